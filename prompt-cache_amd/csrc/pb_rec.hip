// Matrix-state recurrences in chunks of 16 tokens: linear attention with a constant decay per head (retention) or with a decay per key
// channel and token, with or without the delta rule's correction (see pcb_rec_args for the recurrence).
//
// Prompts (pcb_rec_prompt) run as two launches.  Within a chunk let G_t be the running sum of the log decays (per key channel), and
//   A[t][j] = sum_d k_t k_j exp(G_t - G_j),  B[t][j] = sum_d q_t k_j exp(G_t - G_j)          (j <= t: every exponent is <= 0)
//   T = (1 + diag(beta) strictly_lower(A))^-1 diag(beta),  M = B T                           (no correction: T = 1, M = B)
// Then, with S the state before the chunk, K~ = k exp(G), Q~ = q exp(G), K^ = k exp(G_end - G),
//   U = T V - (T K~) S      O = M V + (Q~ - M K~) S      S <- exp(G_end) S + K^T U           (no correction: U = V, O = M V + Q~ S)
// rec_prep_kernel, one workgroup per (chunk, head), computes everything that does not depend on S -- the heads' unit norms or rotary
// turns, decays, A, B, T, M -- and leaves T K~, Q~ - M K~ and K^ in the order in which the second kernel's lanes want them.
// rec_scan_kernel, one workgroup per (request, head, 16 value columns), walks the request's chunks: each of its four waves keeps a
// quarter of the key rows of S as result tiles, which ARE the operand fragments of the products with S; the waves' parts of U and O
// meet in LDS behind one barrier per chunk, the next chunk's operands are in flight meanwhile.  All products are fp32 (matrix cores).
//
// One-token steps (pcb_rec_step): one workgroup per (request, head) reads the state once, and goes on to the head's output norm and
// gate.  States, decays, step sizes, unit norms, rotations and all products are fp32.
#include "pb_common.h"

namespace {
using namespace pcb;

constexpr int CT = 16;            // tokens per chunk
constexpr float LOG2E = 1.44269504088896f;

__device__ __forceinline__ f4 mma4(float a, float b, f4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float exp2_(float x) { return __builtin_amdgcn_exp2f(x); }
// decay^n for a small non-negative integer n
__device__ __forceinline__ float decay_pow(float log2_decay, int n) { return n <= 0 ? 1.0f : exp2f((float)n * log2_decay); }
__device__ __forceinline__ float log2_of(float decay) { return decay > 0.0f ? log2f(decay) : -__builtin_inff(); }
// ln(1 + e^z) = max(z, 0) + ln(1 + x), x = e^-|z| <= 1, and ln(1 + x) = 2 artanh(y), y = x / (2 + x) <= 1/3, by artanh's odd power series
__device__ __forceinline__ float softplus(float z) {
    const float x = __builtin_amdgcn_exp2f(-fabsf(z) * 1.44269504088896f);
    const float y = x * __builtin_amdgcn_rcpf(2.0f + x), y2 = y * y;
    float p = 1.0f / 17.0f;
    p = p * y2 + 1.0f / 15.0f;
    p = p * y2 + 1.0f / 13.0f;
    p = p * y2 + 1.0f / 11.0f;
    p = p * y2 + 1.0f / 9.0f;
    p = p * y2 + 1.0f / 7.0f;
    p = p * y2 + 1.0f / 5.0f;
    p = p * y2 + 1.0f / 3.0f;
    p = p * y2 + 1.0f;
    return fmaxf(z, 0.0f) + 2.0f * y * p;
}
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// the log decay (in units of ln 2) a row of `ld` stands for
__device__ __forceinline__ float log2_decay(const pcb_rec_args& a, float x, float coef) {
    return (a.ld_softplus ? softplus(x) : x) * coef * LOG2E;
}

// one (chunk, head) record of `tiles` 16-column tiles (the key size filled up to 64, 128 or 256 columns): Q~ - M K~, K^ and -T K~ as
// fragments, the end decays, M and T; and its floats
__host__ __device__ constexpr int rec_columns(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : 256; }
__host__ __device__ constexpr int rec_record(int tiles) { return tiles * (3 * 256 + 16) + 512; }

// DM: key columns the workgroup holds (>= dim); DELTA: with the correction; ROWS: decays per key channel and token
template <typename E, int DM, bool DELTA, bool ROWS>
__global__ __launch_bounds__(256) void rec_prep_kernel(pcb_rec_args a) {
    constexpr int LD = DM + 4;
    __shared__ __attribute__((aligned(16))) float Qs[CT][LD], Ks[CT][LD], Gs[ROWS ? CT : 1][LD];
    __shared__ __attribute__((aligned(16))) float As[CT][CT], Bs[CT][CT], Ts[CT][CT], Ms[CT][CT];
    const int tid = threadIdx.x, h = blockIdx.x, hk = h / (a.H / a.Hk), D = a.dim;
    const int32_t* ck = a.chunks + 4 * blockIdx.y;
    const int64_t row0 = ck[0];
    const int n = ck[1];
    const int t = tid >> 4, s = tid & 15;                  // a token and one of 16 threads that share it
    constexpr int NT = DM / 16;
    float* rec = a.scratch + ((int64_t)blockIdx.y * a.H + h) * rec_record(NT);
    float* rq = rec;
    float* rk = rq + NT * 256;
    float* rw = rk + NT * 256;
    float* rd = rw + NT * 256;
    float* rm = rd + NT * 16;
    float* rt = rm + 256;
    const float lg = ROWS ? 0.0f : log2_of(a.decay[h]);

    // ---- the chunk's queries and keys: unit length, scales, rotary turns
    {
        const E* q = (const E*)a.q + (row0 + t) * a.ldq + (int64_t)hk * D;
        const E* k = (const E*)a.k + (row0 + t) * a.ldk + (int64_t)hk * D;
        constexpr int A4 = 4 * sizeof(E);
        const bool vec = D % 4 == 0 && a.ldq % 4 == 0 && a.ldk % 4 == 0 && (uintptr_t)a.q % A4 == 0 && (uintptr_t)a.k % A4 == 0;
        constexpr int NV = DM / 64;
        float qv[NV][4], kv[NV][4], sq = 0.0f, sk = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int d0 = 4 * s + 64 * i, valid = t < n ? D - d0 : 0;
            load4(q + d0, vec, valid, qv[i]);
            load4(k + d0, vec, valid, kv[i]);
#pragma unroll
            for (int e = 0; e < 4; ++e) sq += qv[i][e] * qv[i][e], sk += kv[i][e] * kv[i][e];
        }
        float fq = a.q_scale, fk = a.k_scale;
        if (a.unit_norm) {
#pragma unroll
            for (int o = 1; o < 16; o <<= 1) sq += __shfl_xor(sq, o, 64), sk += __shfl_xor(sk, o, 64);
            fq /= sqrtf(sq + a.unit_eps);
            fk /= sqrtf(sk + a.unit_eps);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            *reinterpret_cast<f4*>(&Qs[t][4 * s + 64 * i]) = f4{qv[i][0] * fq, qv[i][1] * fq, qv[i][2] * fq, qv[i][3] * fq};
            *reinterpret_cast<f4*>(&Ks[t][4 * s + 64 * i]) = f4{kv[i][0] * fk, kv[i][1] * fk, kv[i][2] * fk, kv[i][3] * fk};
        }
    }
    if (ROWS) {
        // log decays (tokens past the end and columns past dim: none), then their running sums, a thread per key channel
        const float coef = a.ld_coef ? a.ld_coef[h] : 1.0f;
        const float* ld = a.ld + (row0 + t) * a.ldld + (int64_t)h * D;
        const bool vec = D % 4 == 0 && a.ldld % 4 == 0 && (uintptr_t)a.ld % 16 == 0;
#pragma unroll
        for (int i = 0; i < DM / 64; ++i) {
            const int d0 = 4 * s + 64 * i;
            float l[4];
            load4(ld + d0, vec, t < n ? D - d0 : 0, l);
            f4 v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = t < n && d0 + e < D ? log2_decay(a, l[e], coef) : 0.0f;
            *reinterpret_cast<f4*>(&Gs[ROWS ? t : 0][d0]) = v;
        }
        __syncthreads();
        if (tid < DM) {
            float l[CT], cum = 0.0f;
#pragma unroll
            for (int i = 0; i < CT; ++i) l[i] = Gs[ROWS ? i : 0][tid];
#pragma unroll
            for (int i = 0; i < CT; ++i) Gs[ROWS ? i : 0][tid] = cum += l[i];
        }
    }
    __syncthreads();
    if (a.rot_dims > 0) {
        const int np = a.rot_dims / 2;
        const float* cs = a.rot + (row0 + (t < n ? t : 0)) * a.rot_dims;
        for (int i = s; i < np; i += 16) {
            const float c = cs[i], sn = cs[np + i];
            const float qu = Qs[t][i], qw = Qs[t][i + np], ku = Ks[t][i], kw = Ks[t][i + np];
            Qs[t][i] = qu * c - qw * sn, Qs[t][i + np] = qw * c + qu * sn;
            Ks[t][i] = ku * c - kw * sn, Ks[t][i + np] = kw * c + ku * sn;
        }
        __syncthreads();
    }

    // ---- A and B.  The 120 pairs j < t take two threads each (neighbours, each half of the key columns), the 16 tokens with themselves
    // one each (no decay, and A is not needed)
    {
        const bool self = tid >= 240;
        int pt, pj, d_lo = 0, d_hi = DM;
        if (self) {
            pt = pj = tid - 240;
        } else {
            const int pr = tid >> 1;                       // pair t (t - 1) / 2 + j
            pt = (int)((1.0f + sqrtf(1.0f + 8.0f * (float)pr)) * 0.5f);
            if (pt * (pt - 1) / 2 > pr) --pt;
            if (pt * (pt + 1) / 2 <= pr) ++pt;
            pj = pr - pt * (pt - 1) / 2;
            d_lo = tid & 1 ? DM / 2 : 0;
            d_hi = d_lo + DM / 2;
        }
        float pa = 0.0f, pb = 0.0f;
        if (pt < n) {
#pragma unroll 4
            for (int d = d_lo; d < d_hi; d += 4) {
                const f4 kj = *reinterpret_cast<const f4*>(&Ks[pj][d]), qt = *reinterpret_cast<const f4*>(&Qs[pt][d]);
                f4 kt = kj, ex = kj;
                if (DELTA) kt = *reinterpret_cast<const f4*>(&Ks[pt][d]);
                if (ROWS && !self) {
                    const f4 gt = *reinterpret_cast<const f4*>(&Gs[ROWS ? pt : 0][d]), gj = *reinterpret_cast<const f4*>(&Gs[ROWS ? pj : 0][d]);
#pragma unroll
                    for (int e = 0; e < 4; ++e) ex[e] = kj[e] * exp2_(gt[e] - gj[e]);
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    pb += qt[e] * ex[e];
                    if (DELTA) pa += kt[e] * ex[e];
                }
            }
        }
        const float pa2 = pa + __shfl_xor(pa, 1, 64), pb2 = pb + __shfl_xor(pb, 1, 64);
        if (self) {
            Bs[pt][pt] = pb;
            if (DELTA) {
                const float beta = pt < n ? sigmoid(a.beta[(row0 + pt) * a.ldbeta + h]) : 0.0f;
                As[pt][pt] = beta;                         // (the diagonal carries the step sizes)
            }
        } else if ((tid & 1) == 0) {
            const float f = ROWS ? 1.0f : decay_pow(lg, pt - pj);
            Bs[pt][pj] = pb2 * f;
            Bs[pj][pt] = 0.0f;
            if (DELTA) As[pt][pj] = pa2 * f;
        }
    }
    __syncthreads();

    // ---- T by forward substitution, a thread per column; meanwhile the other waves turn q, k into Q~, K~ and store K^
    if (DELTA && tid < CT) {
        // (1 + diag(beta) A) T = diag(beta), row by row: T[r] = beta_r (e_r - sum over j < r of A[r][j] T[j])
        float x[CT];
#pragma unroll
        for (int r = 0; r < CT; ++r) {
            float v = r == tid ? 1.0f : 0.0f;
#pragma unroll
            for (int j = 0; j < r; ++j) v -= As[r][j] * x[j];
            x[r] = v * As[r][r];
            Ts[r][tid] = x[r];
        }
    }
    for (int i = tid; i < 4 * DM; i += 256) {
        const int d = i % DM, g = i / DM;                  // key column, run of four tokens
        const int b = d >> 4, c = d & 15;
        float g_end = 0.0f;
        if (ROWS) g_end = Gs[ROWS ? CT - 1 : 0][d];
        f4 kh;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int j = 4 * g + e;
            const float kv = Ks[j][d];
            float f_in, f_end;
            if (ROWS) {
                const float gj = Gs[ROWS ? j : 0][d];
                f_in = exp2_(gj);
                f_end = exp2_(g_end - gj);
            } else {
                f_in = decay_pow(lg, j + 1);
                f_end = decay_pow(lg, n - 1 - j);          // (tokens past the end: their key is zero)
            }
            kh[e] = kv * f_end;
            Ks[j][d] = kv * f_in;
            Qs[j][d] *= f_in;
        }
        *reinterpret_cast<f4*>(rk + (b * 64 + g * 16 + c) * 4) = kh;
        if (g == 0) rd[d] = ROWS ? exp2_(g_end) : decay_pow(lg, n);
    }
    __syncthreads();

    // ---- M = B T, then the fragments of Q~ - M K~ and of T K~
    if (DELTA) {
        float m = 0.0f;
#pragma unroll
        for (int j = 0; j < CT; ++j) m += Bs[t][j] * Ts[j][s];
        Ms[t][s] = m;
        __syncthreads();
        rt[(s & 3) * 64 + (s >> 2) * 16 + t] = Ts[t][s];
    }
    // wave w takes tokens 4 g + w: element (token t, token j) of M and T sits at [j & 3][j >> 2][t]
    rm[(s & 3) * 64 + (s >> 2) * 16 + t] = DELTA ? Ms[t][s] : Bs[t][s];
    {
        const int tt = tid & 15;
        float tr[DELTA ? CT : 1], mr[DELTA ? CT : 1];
        if (DELTA) {
#pragma unroll
            for (int j = 0; j < CT; ++j) tr[j] = Ts[tt][j], mr[j] = Ms[tt][j];
        }
        for (int dq = tid >> 4; dq < 4 * NT; dq += 16) {   // four key columns
            f4 qf = *reinterpret_cast<const f4*>(&Qs[tt][4 * dq]), wf = f4{0.f, 0.f, 0.f, 0.f};
            if (DELTA) {
#pragma unroll
                for (int j = 0; j < CT; ++j) {
                    const f4 kt = *reinterpret_cast<const f4*>(&Ks[j][4 * dq]);
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        wf[e] -= tr[j] * kt[e];
                        qf[e] -= mr[j] * kt[e];
                    }
                }
                *reinterpret_cast<f4*>(rw + (dq * 16 + tt) * 4) = wf;
            }
            *reinterpret_cast<f4*>(rq + (dq * 16 + tt) * 4) = qf;
        }
    }
}

// a value at a uniform address plus a lane's 32-bit byte offset
template <typename T>
__device__ __forceinline__ T at(const void* base, uint32_t bytes) {
    return *reinterpret_cast<const T*>(reinterpret_cast<const char*>(base) + bytes);
}

// NBW: 16-row tiles of S a wave holds (4 NBW tiles in all); ROWS: the end decays come with the records (else decay[h]^tokens)
template <typename E, int NBW, bool DELTA, bool ROWS>
__global__ __launch_bounds__(256) void rec_scan_kernel(pcb_rec_args a) {
    constexpr int NT = 4 * NBW, REC = rec_record(NT);
    __shared__ f4 red_u[DELTA ? 2 : 1][4][64];
    __shared__ float red_o[2][4][4][64];
    const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int32_t* rq = a.reqs + 4 * blockIdx.z;
    const int slot = rq[0], pos0 = rq[1], count = rq[2];
    const int64_t row0 = rq[3];
    const int h = blockIdx.x, D = a.dim, vdim = a.vdim, vcol = blockIdx.y * 16 + c;
    const bool v_ok = vcol < vdim;
    float* st = a.state + (int64_t)slot * a.slot_stride + (int64_t)h * D * vdim;
    f4 S[NBW];
#pragma unroll
    for (int i = 0; i < NBW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (w * NBW + i) + 4 * g + r;
            S[i][r] = (pos0 > 0 && d < D && v_ok) ? st[(int64_t)d * vdim + vcol] : 0.0f;
        }
    const int n_chunk = (count + CT - 1) / CT, n_last = count - CT * (n_chunk - 1);
    const float lg = ROWS ? 0.0f : log2_of(a.decay[h]);
    const float dec_full = ROWS ? 0.0f : decay_pow(lg, CT), dec_last = ROWS ? 0.0f : decay_pow(lg, n_last);
    const int64_t stride = (int64_t)a.H * REC;
    const float* rec = a.scratch + ((int64_t)a.chunk0[blockIdx.z] * a.H + h) * REC + w * NBW * 256;
    const int w_dec = w * NBW * 16 - w * NBW * 256, w_mt = w * 64 - w * NBW * 256;
    const E* V = (const E*)a.v + row0 * a.ldv + (int64_t)h * vdim;
    // a ring of PF chunks' operands, read without branches: chunk i waits in slot i % PF and is replaced, part by part, by chunk i + PF once
    // it has been used.  Chunks, tokens and columns past the end repeat the last one (their K^, M and T are zero, or nothing of theirs
    // is stored).  Part 0: what U needs (T K~, T, the values); part 1: what O needs (Q~ - M K~, M); part 2: what moves S (K^, decays)
    constexpr int PF = NBW <= 2 ? 4 : 3, VN = DELTA ? 1 : 4, NW = DELTA ? NBW : 1;
    f4 rq_[PF][NBW], rk_[PF][NBW], rw_[PF][NW], rd_[PF][ROWS ? NBW : 1];
    float rm_[PF], rt_[PF];
    E rv_[PF][VN];
    uint32_t v_off[VN], v_end[VN];                         // the lane's values within a chunk, and within the last one
#pragma unroll
    for (int e = 0; e < VN; ++e) {
        const int tok = 4 * g + (DELTA ? w : e), col = v_ok ? vcol : vdim - 1;
        v_off[e] = (uint32_t)((tok * a.ldv + col) * sizeof(E));
        v_end[e] = (uint32_t)(((tok < n_last ? tok : n_last - 1) * a.ldv + col) * sizeof(E));
    }
    auto fetch = [&](int i, int u, int part) {
        const bool last = i >= n_chunk - 1;
        i = last ? n_chunk - 1 : i;
        const float* p = rec + i * stride;
        if (part == 0) {
            const E* pv = V + (int64_t)(CT * i) * a.ldv;
#pragma unroll
            for (int e = 0; e < VN; ++e) rv_[u][e] = at<E>(pv, last ? v_end[e] : v_off[e]);
            if (DELTA) {
                rt_[u] = at<float>(p + w_mt + NT * 784 + 256, 4 * lane);
#pragma unroll
                for (int j = 0; j < NW; ++j) rw_[u][j] = at<f4>(p + (2 * NT + j) * 256, 16 * lane);
            }
        } else if (part == 1) {
            rm_[u] = at<float>(p + w_mt + NT * 784, 4 * lane);
#pragma unroll
            for (int j = 0; j < NBW; ++j) rq_[u][j] = at<f4>(p + j * 256, 16 * lane);
        } else {
#pragma unroll
            for (int j = 0; j < NBW; ++j) {
                rk_[u][j] = at<f4>(p + (NT + j) * 256, 16 * lane);
                if (ROWS) rd_[u][ROWS ? j : 0] = at<f4>(p + w_dec + NT * 768 + j * 16, 16 * g);
            }
        }
        // (the loads stay in order: a wait for one chunk's must not cover the chunks behind it)
        __builtin_amdgcn_sched_barrier(0);
    };
#pragma unroll
    for (int u = 0; u < PF; ++u)
#pragma unroll
        for (int part = 0; part < 3; ++part) fetch(u, u, part);
    const uint32_t o_off = (uint32_t)(((4 * g + w) * a.ldo + vcol) * 4);
    const f4 zero = f4{0.f, 0.f, 0.f, 0.f};
    // the outputs of chunk i, whose parts the waves left in LDS before the last barrier: wave w writes the tokens 4 g + w
    auto parts_of = [&](int i, float (&r)[4]) {
#pragma unroll
        for (int x = 0; x < 4; ++x) r[x] = red_o[i & 1][w][x][lane];
    };
    auto emit = [&](int i, const float (&r)[4]) {
        const float ov = (r[0] + r[1]) + (r[2] + r[3]);
        float* po = a.out + (row0 + CT * i) * a.ldo + (int64_t)h * vdim;
        if (CT * i + 4 * g + w < count && v_ok) *reinterpret_cast<float*>(reinterpret_cast<char*>(po) + o_off) = ov;
    };
    auto work = [&](int i, int u, bool refill) {           // chunk i out of slot u
        const int buf = i & 1;
        float cv[VN];
#pragma unroll
        for (int e = 0; e < VN; ++e) cv[e] = to_f32(rv_[u][e]);
        const float v_w = DELTA ? cv[0] : (w == 0 ? cv[0] : w == 1 ? cv[VN > 1 ? 1 : 0] : w == 2 ? cv[VN > 2 ? 2 : 0] : cv[VN > 3 ? 3 : 0]);
        f4 U;
        if (DELTA) {
            // this wave's part of U -- four of the tokens' values and its rows of S -- meets the others' in LDS ...
            f4 part = mma4(rt_[u], v_w, zero);
#pragma unroll
            for (int j = 0; j < NW; ++j)
#pragma unroll
                for (int e = 0; e < 4; ++e) part = mma4(rw_[u][j][e], S[j][e], part);
            red_u[DELTA ? buf : 0][w][lane] = part;
        }
        __syncthreads();                                   // (red_u[buf] was last read two barriers ago, red_o[buf] is written after this one)
        f4 u4[4];
        float before[4];                                   // (of the chunk before; the first chunk's are not used)
        parts_of(i - 1, before);
        if (DELTA) {
#pragma unroll
            for (int x = 0; x < 4; ++x) u4[x] = red_u[DELTA ? buf : 0][x][lane];
        }
        // ... while its part of O is under way
        f4 o = mma4(rm_[u], v_w, zero);
#pragma unroll
        for (int j = 0; j < NBW; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                o = mma4(rq_[u][j][e], S[j][e], o);
                if (refill && j == 0 && e == 3) fetch(i + PF, u, 0);       // (loads go out between products: a wave's queue of them is short)
            }
        if (refill) fetch(i + PF, u, 1);
        if (i > 0) emit(i - 1, before);
        if (DELTA) {
            U = (u4[0] + u4[1]) + (u4[2] + u4[3]);
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) U[r] = cv[DELTA ? 0 : r];
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) red_o[buf][r][w][lane] = o[r];
        const float dec = i == n_chunk - 1 ? dec_last : dec_full;
#pragma unroll
        for (int j = 0; j < NBW; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[j][r] *= ROWS ? rd_[u][ROWS ? j : 0][r] : dec;
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int j = 0; j < NBW; ++j) S[j] = mma4(rk_[u][j][e], U[e], S[j]);
        if (refill) fetch(i + PF, u, 2);
    };
    // (whole rounds of the ring without a branch between them, then the chunks that are left)
    int i0 = 0;
    for (; i0 + PF <= n_chunk; i0 += PF) {
#pragma unroll
        for (int u = 0; u < PF; ++u) work(i0 + u, u, true);
    }
#pragma unroll
    for (int u = 0; u < PF - 1; ++u)
        if (i0 + u < n_chunk) work(i0 + u, u, false);
    __syncthreads();
    float before[4];
    parts_of(n_chunk - 1, before);
    emit(n_chunk - 1, before);
    if (!v_ok) return;
#pragma unroll
    for (int i = 0; i < NBW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = 16 * (w * NBW + i) + 4 * g + r;
            if (d < D) st[(int64_t)d * vdim + vcol] = S[i][r];
        }
}

// ---- one token per request ------------------------------------------------------------------------------------------------------------
constexpr int ST = 512;           // threads of a step's workgroup

template <int VW>
struct Cols {
    float v[VW];
};

// VW: neighbouring value columns of a thread; RPT: key rows of a thread (at most)
template <typename E, int VW, int RPT>
__global__ __launch_bounds__(ST) void rec_step_kernel(pcb_rec_args a) {
    __shared__ float qs[256], ks[256], ds[256], us[512], red[8];
    __shared__ __attribute__((aligned(16))) float part[ST * VW];
    const int tid = threadIdx.x, h = blockIdx.x, hk = h / (a.H / a.Hk), D = a.dim, vdim = a.vdim;
    const int32_t* rq = a.reqs + 4 * blockIdx.y;
    const int slot = rq[0], pos0 = rq[1];
    const int64_t row = rq[3];
    const int CG = vdim / VW, RG = ST / CG;                // column groups, row groups
    const int rg = tid / CG, cg = tid % CG;
    const bool busy = rg < RG;
    float* st = a.state + (int64_t)slot * a.slot_stride + (int64_t)h * D * vdim + cg * VW;
    Cols<VW> S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int d = rg + RG * i;
        const bool ok = busy && d < D && pos0 > 0;
        if (VW == 4) {
            f4 x = f4{0.f, 0.f, 0.f, 0.f};
            if (ok) x = *reinterpret_cast<const f4*>(st + (int64_t)d * vdim);
#pragma unroll
            for (int e = 0; e < VW; ++e) S[i].v[e] = x[e & 3];
        } else {
            S[i].v[0] = ok ? st[(int64_t)d * vdim] : 0.0f;
        }
    }
    // threads 0 .. 255 bring the query, 256 .. 511 the key; all of them the decays
    const bool key = tid >= 256;
    const int d = tid & 255;
    float x = 0.0f;
    if (d < D) x = to_f32(key ? ((const E*)a.k)[row * a.ldk + (int64_t)hk * D + d] : ((const E*)a.q)[row * a.ldq + (int64_t)hk * D + d]);
    const bool delta = a.beta != nullptr;
    float vj = 0.0f, gj = 1.0f, wj = 1.0f, beta = 1.0f;    // this thread's value column, its gate and gain
    if (tid < vdim) {
        vj = to_f32(((const E*)a.v)[row * a.ldv + (int64_t)h * vdim + tid]);
        if (a.gate) gj = to_f32(((const E*)a.gate)[row * a.ldg + (int64_t)h * vdim + tid]);
        if (a.gain) wj = a.gain[tid];
        if (delta) beta = sigmoid(a.beta[row * a.ldbeta + h]);
    }
    if (!key && d < D) {
        if (a.ld) {
            ds[d] = exp2_(log2_decay(a, a.ld[row * a.ldld + (int64_t)h * D + d], a.ld_coef ? a.ld_coef[h] : 1.0f));
        } else {
            ds[d] = a.decay[h];
        }
    }
    float f = key ? a.k_scale : a.q_scale;
    if (a.unit_norm) {
        const float ss = wave_sum(x * x);
        if ((tid & 63) == 0) red[tid >> 6] = ss;
        __syncthreads();
        const int b = key ? 4 : 0;
        f /= sqrtf((red[b] + red[b + 1]) + (red[b + 2] + red[b + 3]) + a.unit_eps);
    }
    (key ? ks : qs)[d] = x * f;
    __syncthreads();
    if (a.rot_dims > 0) {
        const int np = a.rot_dims / 2;
        float* vec = key ? ks : qs;
        if (d < np) {
            const float cs = a.rot[row * a.rot_dims + d], sn = a.rot[row * a.rot_dims + np + d];
            const float u = vec[d], v = vec[d + np];
            vec[d] = u * cs - v * sn;
            vec[d + np] = v * cs + u * sn;
        }
        __syncthreads();
    }
    // forget; what the key reads
    float acc[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) acc[e] = 0.0f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + RG * i;
        if (busy && r < D) {
            const float f = ds[r], kk = ks[r];
#pragma unroll
            for (int e = 0; e < VW; ++e) {
                S[i].v[e] *= f;
                acc[e] += S[i].v[e] * kk;
            }
        }
    }
    if (delta) {
        if (busy)
#pragma unroll
            for (int e = 0; e < VW; ++e) part[(rg * CG + cg) * VW + e] = acc[e];
        __syncthreads();
        if (tid < vdim) {
            float s = 0.0f;
            for (int r = 0; r < RG; ++r) s += part[r * vdim + tid];
            us[tid] = beta * (vj - s);
        }
    } else if (tid < vdim) {
        us[tid] = vj;
    }
    __syncthreads();
    // write, then read with the query
    float uu[VW];
#pragma unroll
    for (int e = 0; e < VW; ++e) uu[e] = busy ? us[cg * VW + e] : 0.0f, acc[e] = 0.0f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + RG * i;
        if (busy && r < D) {
            const float kk = ks[r], qq = qs[r];
#pragma unroll
            for (int e = 0; e < VW; ++e) {
                S[i].v[e] += kk * uu[e];
                acc[e] += S[i].v[e] * qq;
            }
            if (VW == 4)
                *reinterpret_cast<f4*>(st + (int64_t)r * vdim) = f4{S[i].v[0], S[i].v[1 % VW], S[i].v[2 % VW], S[i].v[3 % VW]};
            else
                st[(int64_t)r * vdim] = S[i].v[0];
        }
    }
    if (busy)
#pragma unroll
        for (int e = 0; e < VW; ++e) part[(rg * CG + cg) * VW + e] = acc[e];
    __syncthreads();
    float o = 0.0f;
    if (tid < vdim)
        for (int r = 0; r < RG; ++r) o += part[r * vdim + tid];
    // the head's output norm and gate
    const float ss = wave_sum(o * o);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    if (tid < vdim) {
        float sum = 0.0f;
#pragma unroll
        for (int i = 0; i < ST / 64; ++i) sum += red[i];
        const float inv = 1.0f / sqrtf(sum / (float)vdim + a.eps);
        ((E*)a.y)[row * a.ldy + (int64_t)h * vdim + tid] = from_f32<E>(o * inv * wj * gj);
    }
}

template <typename E, int DM>
void launch_prep(const pcb_rec_args& a, hipStream_t stream) {
    const dim3 grid(a.H, a.n_chunks), block(256);
    if (a.beta) {
        if (a.ld)
            hipLaunchKernelGGL((rec_prep_kernel<E, DM, true, true>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_prep_kernel<E, DM, true, false>), grid, block, 0, stream, a);
    } else {
        if (a.ld)
            hipLaunchKernelGGL((rec_prep_kernel<E, DM, false, true>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_prep_kernel<E, DM, false, false>), grid, block, 0, stream, a);
    }
}

template <typename E, int NBW>
void launch_scan(const pcb_rec_args& a, hipStream_t stream) {
    // (heads run fastest: a head's column blocks meet its records in one XCD's L2)
    const dim3 grid(a.H, pcb_ceil_div(a.vdim, 16), a.n_reqs), block(256);
    if (a.beta) {
        if (a.ld)
            hipLaunchKernelGGL((rec_scan_kernel<E, NBW, true, true>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_scan_kernel<E, NBW, true, false>), grid, block, 0, stream, a);
    } else {
        if (a.ld)
            hipLaunchKernelGGL((rec_scan_kernel<E, NBW, false, true>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_scan_kernel<E, NBW, false, false>), grid, block, 0, stream, a);
    }
}

template <typename E>
int prompt(const pcb_rec_args& a, hipStream_t stream) {
    if (a.dim <= 64) {
        launch_prep<E, 64>(a, stream);
        launch_scan<E, 1>(a, stream);
    } else if (a.dim <= 128) {
        launch_prep<E, 128>(a, stream);
        launch_scan<E, 2>(a, stream);
    } else {
        launch_prep<E, 256>(a, stream);
        launch_scan<E, 4>(a, stream);
    }
    return pcb_check_launch("rec_prep_kernel / rec_scan_kernel");
}

// key rows a thread of a one-token step holds, 0: the head does not fit
int step_rows(int dim, int vdim) {
    if (dim > 256 || vdim > 512) return 0;
    const int vw = vdim % 4 == 0 ? 4 : 1;
    const int rg = ST / (vdim / vw), rpt = (dim + rg - 1) / rg;
    return rpt <= (vw == 4 ? 32 : 64) ? rpt : 0;
}

template <typename E>
int step(const pcb_rec_args& a, hipStream_t stream) {
    const dim3 grid(a.H, a.n_reqs), block(ST);
    const int rpt = step_rows(a.dim, a.vdim);
    if (a.vdim % 4 == 0) {
        if (rpt <= 2)
            hipLaunchKernelGGL((rec_step_kernel<E, 4, 2>), grid, block, 0, stream, a);
        else if (rpt <= 8)
            hipLaunchKernelGGL((rec_step_kernel<E, 4, 8>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_step_kernel<E, 4, 32>), grid, block, 0, stream, a);
    } else {
        if (rpt <= 16)
            hipLaunchKernelGGL((rec_step_kernel<E, 1, 16>), grid, block, 0, stream, a);
        else
            hipLaunchKernelGGL((rec_step_kernel<E, 1, 64>), grid, block, 0, stream, a);
    }
    return pcb_check_launch("rec_step_kernel");
}

int check(const pcb_rec_args* a, const char* what) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_rec_args), PCB_ERR_ARG, "%s: struct size mismatch", what);
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "%s: unknown dtype", what);
    PCB_REQUIRE(a->n_reqs >= 0 && a->n_reqs <= 65535 && a->H > 0 && a->H <= 65535 && a->Hk > 0 && a->H % a->Hk == 0 && a->dim > 0 && a->dim <= 256 &&
                    a->vdim > 0 && a->ldq >= (int64_t)a->Hk * a->dim && a->ldk >= (int64_t)a->Hk * a->dim && a->ldv >= (int64_t)a->H * a->vdim &&
                    a->slot_stride >= (int64_t)a->H * a->dim * a->vdim,
                PCB_ERR_ARG, "%s: bad sizes (up to 256 key columns per head)", what);
    PCB_REQUIRE(a->ldv < (1 << 26) && a->ldo < (1 << 24), PCB_ERR_ARG, "%s: rows too long", what);
    PCB_REQUIRE(a->rot_dims >= 0 && a->rot_dims % 2 == 0 && a->rot_dims <= a->dim && (a->rot_dims == 0 || a->rot || a->n_reqs == 0), PCB_ERR_ARG,
                "%s: rotated columns come in pairs inside the head, with their table of cosines and sines", what);
    PCB_REQUIRE(a->n_reqs == 0 || ((a->decay != nullptr) != (a->ld != nullptr)), PCB_ERR_ARG,
                "%s: a decay per head or rows of log decays, one of them", what);
    PCB_REQUIRE((!a->ld || a->ldld >= (int64_t)a->H * a->dim) && (!a->beta || a->ldbeta >= a->H), PCB_ERR_ARG, "%s: rows too short", what);
    return PCB_OK;
}

}  // namespace

PCB_EXPORT int64_t pcb_rec_scratch(int32_t n_chunks, int32_t H, int32_t dim) {
    return n_chunks > 0 && H > 0 && dim > 0 && dim <= 256 ? (int64_t)n_chunks * H * rec_record(rec_columns(dim) / 16) : 0;
}

PCB_EXPORT int pcb_rec_prompt(const pcb_rec_args* a, void* stream) {
    const int rc = check(a, "pcb_rec_prompt");
    if (rc != PCB_OK) return rc;
    PCB_REQUIRE(a->ldo >= (int64_t)a->H * a->vdim && a->n_chunks >= a->n_reqs && a->n_chunks <= 65535 && pcb_ceil_div(a->vdim, 16) <= 65535 &&
                    a->scratch_floats >= pcb_rec_scratch(a->n_chunks, a->H, a->dim),
                PCB_ERR_ARG, "pcb_rec_prompt: bad sizes (up to 65 535 chunks of 16 tokens, with their scratch)");
    if (a->n_reqs == 0) return PCB_OK;
    PCB_REQUIRE(a->q && a->k && a->v && a->reqs && a->chunks && a->chunk0 && a->state && a->scratch && (uintptr_t)a->scratch % 16 == 0 && a->out,
                PCB_ERR_ARG, "pcb_rec_prompt: null pointer");
    return a->dtype == PCB_BF16 ? prompt<pcb::bf16_t>(*a, (hipStream_t)stream) : prompt<float>(*a, (hipStream_t)stream);
}

PCB_EXPORT int32_t pcb_rec_step_fits(int32_t dim, int32_t vdim) { return dim > 0 && vdim > 0 && step_rows(dim, vdim) > 0; }

PCB_EXPORT int pcb_rec_step(const pcb_rec_args* a, void* stream) {
    const int rc = check(a, "pcb_rec_step");
    if (rc != PCB_OK) return rc;
    PCB_REQUIRE(pcb_rec_step_fits(a->dim, a->vdim), PCB_ERR_ARG, "pcb_rec_step: a head's state must fit the registers of 512 threads");
    PCB_REQUIRE(a->ldy >= (int64_t)a->H * a->vdim && (!a->gate || a->ldg >= (int64_t)a->H * a->vdim), PCB_ERR_ARG, "pcb_rec_step: rows too short");
    if (a->n_reqs == 0) return PCB_OK;
    PCB_REQUIRE(a->q && a->k && a->v && a->reqs && a->state && a->y, PCB_ERR_ARG, "pcb_rec_step: null pointer");
    PCB_REQUIRE(a->vdim % 4 != 0 || ((uintptr_t)a->state % 16 == 0 && a->slot_stride % 4 == 0), PCB_ERR_ARG,
                "pcb_rec_step: states of four-column rows start at multiples of 16 bytes");
    return a->dtype == PCB_BF16 ? step<pcb::bf16_t>(*a, (hipStream_t)stream) : step<float>(*a, (hipStream_t)stream);
}
