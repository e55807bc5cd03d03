// pcb_attn_rows: causal softmax attention of single rows over a slot's cached keys and values, row by row (decoding with grouped key
// heads: the query heads of a key head are the rows of one tile, so a key or value is read once for all of them).
//
// One workgroup = one query row x up to 16 query heads of one key head x one run of the keys.  The run is walked in blocks of BK rows:
// keys and values go global -> registers -> LDS once, the next block's loads in flight.  Scores S^T = K Q^T: wave w takes the 16 keys
// 16 w .. of the block and leaves its 16 x 16 scores in LDS; then every wave takes all of the block's scores and a quarter of the value
// columns, O^T = V^T P^T with transposed reads of the row-major values.  No wave holds more than a quarter of the accumulator and nothing
// is merged between waves; runs of the keys are merged by a second launch, which also takes the sink and the gate.
#include "pb_attn_common.h"

namespace {
using namespace pcb;

constexpr int LW = 4;          // waves of a workgroup

// the oldest key the query at position i sees
__device__ __forceinline__ int oldest(const pcb_attn_rows_args& a, int i) {
    int lo = a.window > 0 && i - a.window + 1 > 0 ? i - a.window + 1 : 0;
    if (a.block > 0) lo = max(lo, i / a.block * a.block);
    return lo;
}

// one 16-byte chunk of a row of `cols` elements, element by element
template <typename E>
__device__ __forceinline__ u32x4 odd_chunk(const E* p, int col, int cols) {
    constexpr int CE = 16 / sizeof(E);
    __attribute__((aligned(16))) E tmp[CE];
#pragma unroll
    for (int e = 0; e < CE; ++e) tmp[e] = col + e < cols ? p[col + e] : from_f32<E>(0.0f);
    return *reinterpret_cast<u32x4*>(tmp);
}

// KSQ: 32-element k-steps of a key; VBW: 16-column value blocks per wave; BK: keys per block
template <typename E, int KSQ, int VBW, int BK>
__global__ __launch_bounds__(64 * LW) void attn_rows_kernel(pcb_attn_rows_args a) {
    constexpr int CE = 16 / sizeof(E);
    constexpr int KC = KSQ * 32, VC = VBW * 16 * LW, KLD = KC + CE, VLD = v_ld<E>(VC), NKT = BK / 16, NK2 = BK / 32;
    constexpr int LPR = 64 * LW / BK;                                // threads that share a row: thread t loads row t / LPR, chunks t % LPR + i LPR
    constexpr int KCH = KC / CE / LPR, VCH = VC / CE / LPR;
    static_assert(KC / CE % LPR == 0 && VC / CE % LPR == 0, "whole chunks per thread");
    __shared__ __attribute__((aligned(16))) E Ks[BK * KLD];
    __shared__ __attribute__((aligned(16))) E Vs[BK * VLD];
    __shared__ f4 Ss[NKT][64];                                       // scores of key tile kt as the result tile's lanes hold them
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
    const int32_t* tile = a.tiles + 4 * blockIdx.x;
    const int slot = tile[0], pos = tile[1];
    const int64_t qrow = tile[3];
    const int per = a.H / a.Hkv, hb = (per + 15) / 16;               // query heads of a key head, workgroups they take
    const int hk = blockIdx.y / hb, j0 = blockIdx.y % hb * 16;
    const int n_h = per - j0 < 16 ? per - j0 : 16;
    const int h = hk * per + j0 + (c < n_h ? c : n_h - 1);           // (lanes past the last head repeat it; nothing of theirs is stored)
    const int dim = a.dim, vdim = a.vdim;
    const E* K = (const E*)a.k + (int64_t)slot * a.k_slot_stride + (int64_t)hk * a.k_head_stride;
    const E* V = (const E*)a.v + (int64_t)slot * a.v_slot_stride + (int64_t)hk * a.v_head_stride;
    const bool vec = (((uintptr_t)a.k | (uintptr_t)a.v) % 16 == 0) && a.k_slot_stride % CE == 0 && a.k_head_stride % CE == 0 && a.k_row_stride % CE == 0 &&
                     a.v_slot_stride % CE == 0 && a.v_head_stride % CE == 0 && a.v_row_stride % CE == 0 && dim % CE == 0 && vdim % CE == 0;
    const bool qvec = ((uintptr_t)a.q % 16 == 0) && (a.ldq % CE == 0) && (dim % CE == 0);
    const float sc = a.scale * 1.44269504088896f;                    // scores in units of ln 2
    const float NEG = -__builtin_inff();

    const int lo = oldest(a, pos);
    int kb_lo = lo / BK, kb_hi = pos / BK;
    if (a.n_splits > 1) {                                            // this workgroup's run of the blocks (it may be empty)
        const int run = (kb_hi - kb_lo + a.n_splits) / a.n_splits;
        kb_lo += (int)blockIdx.z * run;
        kb_hi = kb_lo + run - 1 < kb_hi ? kb_lo + run - 1 : kb_hi;
    }
    u32x4 rk[KCH], rv[VCH];
    const int lr = tid / LPR, lc = tid % LPR * CE;                   // this thread's row and first column
    auto fetch = [&](int kb) {
        int j = kb * BK + lr;
        j = j > pos ? pos : j;                                       // (keys past the end repeat the last one: finite, and masked)
        const E* kp = K + (int64_t)j * a.k_row_stride;
        const E* vp = V + (int64_t)j * a.v_row_stride;
        if (vec) {
#pragma unroll
            for (int i = 0; i < KCH; ++i) {
                const int col = lc + i * LPR * CE;
                rk[i] = u32x4{0u, 0u, 0u, 0u};
                if (col < dim) rk[i] = *reinterpret_cast<const u32x4*>(kp + col);
            }
#pragma unroll
            for (int i = 0; i < VCH; ++i) {
                const int col = lc + i * LPR * CE;
                rv[i] = u32x4{0u, 0u, 0u, 0u};
                if (col < vdim) rv[i] = *reinterpret_cast<const u32x4*>(vp + col);
            }
        } else {
#pragma unroll 1
            for (int i = 0; i < KCH; ++i) *reinterpret_cast<u32x4*>(&Ks[lr * KLD + lc + i * LPR * CE]) = odd_chunk<E>(kp, lc + i * LPR * CE, dim);
#pragma unroll 1
            for (int i = 0; i < VCH; ++i) *reinterpret_cast<u32x4*>(&Vs[lr * VLD + lc + i * LPR * CE]) = odd_chunk<E>(vp, lc + i * LPR * CE, vdim);
        }
    };
    if (vec && kb_lo <= kb_hi) fetch(kb_lo);
    Frag<E> qf[KSQ];
    const E* qp = (const E*)a.q + qrow * a.ldq + (int64_t)h * dim;
#pragma unroll
    for (int ks = 0; ks < KSQ; ++ks) qf[ks] = load_frag(qp + 32 * ks, g, dim - 32 * ks, qvec);

    float m = NEG, l = 0.0f;
    f4 o[VBW];
#pragma unroll
    for (int vb = 0; vb < VBW; ++vb) o[vb] = f4{0.f, 0.f, 0.f, 0.f};
    for (int kb = kb_lo; kb <= kb_hi; ++kb) {
        __syncthreads();                                             // the previous block's reads are done
        if (vec) {
#pragma unroll
            for (int i = 0; i < KCH; ++i) *reinterpret_cast<u32x4*>(&Ks[lr * KLD + lc + i * LPR * CE]) = rk[i];
#pragma unroll
            for (int i = 0; i < VCH; ++i) *reinterpret_cast<u32x4*>(&Vs[lr * VLD + lc + i * LPR * CE]) = rv[i];
        } else {
            fetch(kb);                                               // (odd sizes: element by element, straight into LDS)
        }
        __syncthreads();
        if (vec && kb < kb_hi) fetch(kb + 1);
        for (int kt = wave; kt < NKT; kt += LW) {
            f4 acc = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KSQ; ++ks) acc = mma(load_frag(&Ks[(kt * 16 + c) * KLD + 32 * ks], g, 32, true), qf[ks], acc);
            Ss[kt][lane] = acc;
        }
        __syncthreads();
        float s[NKT][4], bm = NEG;
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
            const f4 acc = Ss[kt][lane];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = kb * BK + kt * 16 + 4 * g + r;
                s[kt][r] = key <= pos && key >= lo ? acc[r] * sc : NEG;
                bm = fmaxf(bm, s[kt][r]);
            }
        }
        bm = fmaxf(bm, __shfl_xor(bm, 16, 64));
        bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
        const float m_new = fmaxf(m, bm);
        const float m_use = m_new == NEG ? 0.0f : m_new;
        const float alpha = __builtin_amdgcn_exp2f(m - m_use);       // (m = -inf: 0)
        float psum = 0.0f;
        PFrag<E> pf[NK2];
#pragma unroll
        for (int k2 = 0; k2 < NK2; ++k2) {
            float p[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                p[e] = __builtin_amdgcn_exp2f(s[2 * k2 + (e >> 2)][e & 3] - m_use);
                psum += p[e];
            }
            make_p(pf[k2], p);
        }
        l = l * alpha + psum;
        m = m_new;
#pragma unroll
        for (int vb = 0; vb < VBW; ++vb) {
            const int col = (wave * VBW + vb) * 16;
            if (col >= vdim) break;
#pragma unroll
            for (int r = 0; r < 4; ++r) o[vb][r] *= alpha;
#pragma unroll
            for (int k2 = 0; k2 < NK2; ++k2) o[vb] = mma_p(load_v_lds(&Vs[k2 * 32 * VLD + col], VLD, g, c), pf[k2], o[vb]);
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (c >= n_h) return;
    float f = 1.0f;
    float* pp = nullptr;
    E* op = nullptr;
    const E* gp = nullptr;                                           // an element-wise gate
    if (a.n_splits > 1) {
        const int64_t run = ((int64_t)blockIdx.x * a.H + h) * a.n_splits + blockIdx.z;
        pp = a.part + run * vdim;
        if (wave == 0 && g == 0) *reinterpret_cast<float2*>(a.part + (int64_t)a.n_rows * a.H * a.n_splits * vdim + 2 * run) = float2{m, l};
    } else {
        float keep = 1.0f;
        if (a.sink) {
            const float sk = a.sink[h] * 1.44269504088896f;
            const float top = fmaxf(m, sk);
            keep = __builtin_amdgcn_exp2f(m - top);
            l = l * keep + __builtin_amdgcn_exp2f(sk - top);
        }
        f = keep / l;
        if (a.gate && a.gate_per_head) f *= to_f32(((const E*)a.gate)[qrow * a.ldg + h]);
        if (a.gate && !a.gate_per_head) gp = (const E*)a.gate + qrow * a.ldg + (int64_t)h * vdim;
        op = (E*)a.out + qrow * a.ldo + (int64_t)h * vdim;
    }
    const bool quads = vdim % 4 == 0 && (pp || (((uintptr_t)a.out % 16 == 0) && a.ldo % 4 == 0));
#pragma unroll
    for (int vb = 0; vb < VBW; ++vb) {
        const int col = (wave * VBW + vb) * 16 + 4 * g;
        if (pp && quads && col < vdim) {
            *reinterpret_cast<f4*>(pp + col) = o[vb];
            continue;
        }
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = pp ? o[vb][r] : o[vb][r] * f * (gp && col + r < vdim ? to_f32(gp[col + r]) : 1.0f);
        if (quads && col < vdim) {
            store4(op + col, v[0], v[1], v[2], v[3]);
            continue;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (col + r < vdim) {
                if (pp)
                    pp[col + r] = v[r];
                else
                    op[col + r] = from_f32<E>(v[r]);
            }
    }
}

// one workgroup per (row, head): the runs' factors once, then their partial results rescaled to the common maximum and summed
template <typename E>
__global__ __launch_bounds__(256) void attn_rows_merge_kernel(pcb_attn_rows_args a) {
    __shared__ float fac[64];
    const int64_t qrow = a.tiles[4 * blockIdx.x + 3];
    const int h = blockIdx.y, vdim = a.vdim, Z = a.n_splits, lane = threadIdx.x & 63;
    const int64_t run = ((int64_t)blockIdx.x * a.H + h) * Z;
    const float* pp = a.part + run * vdim;
    const float* ml = a.part + (int64_t)a.n_rows * a.H * Z * vdim + 2 * run;
    const E* gate = (const E*)a.gate;
    if (threadIdx.x < 64) {
        const float NEG = -__builtin_inff();
        const float mz = lane < Z ? ml[2 * lane] : NEG;
        const float lz = lane < Z ? ml[2 * lane + 1] : 0.0f;
        float top = wave_max(mz);                                    // (the row sees itself: a number)
        const float sk = a.sink ? a.sink[h] * 1.44269504088896f : NEG;
        top = fmaxf(top, sk);
        const float w = __builtin_amdgcn_exp2f(mz - top);
        const float den = wave_sum(w * lz) + (a.sink ? __builtin_amdgcn_exp2f(sk - top) : 0.0f);
        float f = w / den;
        if (gate && a.gate_per_head) f *= to_f32(gate[qrow * a.ldg + h]);
        fac[lane] = f;
    }
    __syncthreads();
    for (int c = threadIdx.x; c < vdim; c += 256) {
        float o = 0.0f;
#pragma unroll 8
        for (int z = 0; z < Z; ++z) o += fac[z] * pp[(int64_t)z * vdim + c];       // (an empty run left zeros)
        if (gate && !a.gate_per_head) o *= to_f32(gate[qrow * a.ldg + (int64_t)h * vdim + c]);
        ((E*)a.out)[qrow * a.ldo + (int64_t)h * vdim + c] = from_f32<E>(o);
    }
}

template <typename E>
int dispatch(const pcb_attn_rows_args& a, hipStream_t stream) {
    constexpr int BK = sizeof(E) == 2 ? 64 : 32;
    const int per = a.H / a.Hkv;
    const dim3 grid(a.n_rows, a.Hkv * ((per + 15) / 16), a.n_splits > 1 ? a.n_splits : 1), block(64 * LW);
    if (a.dim <= 64 && a.vdim <= 64)
        hipLaunchKernelGGL((attn_rows_kernel<E, 2, 1, BK>), grid, block, 0, stream, a);
    else if (a.dim <= 128 && a.vdim <= 128)
        hipLaunchKernelGGL((attn_rows_kernel<E, 4, 2, BK>), grid, block, 0, stream, a);
    else
        hipLaunchKernelGGL((attn_rows_kernel<E, 8, 4, BK>), grid, block, 0, stream, a);
    if (a.n_splits > 1) hipLaunchKernelGGL(attn_rows_merge_kernel<E>, dim3(a.n_rows, a.H), dim3(256), 0, stream, a);
    return pcb_check_launch("attn_rows_kernel");
}

}  // namespace

PCB_EXPORT int pcb_attn_rows(const pcb_attn_rows_args* a, void* stream) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_attn_rows_args), PCB_ERR_ARG, "pcb_attn_rows: struct size mismatch");
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "pcb_attn_rows: unknown dtype");
    PCB_REQUIRE(a->n_rows >= 0 && a->H > 0 && a->H <= 65535 && a->Hkv > 0 && a->H % a->Hkv == 0 && a->dim > 0 && a->dim <= 256 && a->vdim > 0 &&
                    a->vdim <= 256 && a->ldq >= (int64_t)a->H * a->dim && a->ldo >= (int64_t)a->H * a->vdim && a->k_row_stride >= a->dim &&
                    a->v_row_stride >= a->vdim && a->k_slot_stride >= 0 && a->k_head_stride >= 0 && a->v_slot_stride >= 0 && a->v_head_stride >= 0,
                PCB_ERR_ARG, "pcb_attn_rows: bad sizes (keys and values of up to 256 columns)");
    if (a->n_rows == 0) return PCB_OK;
    PCB_REQUIRE(a->q && a->tiles && a->k && a->v && a->out && (!a->gate || a->ldg >= (a->gate_per_head ? (int64_t)a->H : (int64_t)a->H * a->vdim)),
                PCB_ERR_ARG, "pcb_attn_rows: null pointer");
    PCB_REQUIRE(a->n_splits <= 1 || (a->part && (uintptr_t)a->part % 16 == 0 && a->n_splits <= 64), PCB_ERR_ARG,
                "pcb_attn_rows: up to 64 runs, with their scratch");
    return a->dtype == PCB_BF16 ? dispatch<pcb::bf16_t>(*a, (hipStream_t)stream) : dispatch<float>(*a, (hipStream_t)stream);
}
