// pcb_linear: Y = A W^T for row-major activations and nn.Linear-layout weights in bf16 or fp32, with what decoder layers fuse
// around a projection: bias, gathered and scaled input rows, per-group weights (experts), a gated-unit epilogue, and the
// layer-scaled accumulation into an fp32 residual stream.
//
// Tiling: workgroup = 4 waves in a 2 x 2 grid, a wave owns TM x TN result tiles of 16 x 16, so the workgroup covers
// (32 TM) x (32 TN) of Y.  Per stage of two 32-element k-steps the A and B panels go global -> registers -> LDS (the next stage's
// loads are in flight while this stage's MFMAs run); waves read their operand fragments from LDS with one 16-byte read per fragment (bf16).
// bf16 operands that can be read in 16-byte chunks take linear_dma_kernel below instead; fp32, odd sizes and scaled rows this one.
#include <type_traits>

#include "pb_common.h"

namespace {
using namespace pcb;

template <typename E>
struct Tile {
    static constexpr int KS = sizeof(E) == 2 ? 2 : 1;   // 32-element k-steps per LDS stage (fp32 panels are twice as large)
    static constexpr int CE = 16 / sizeof(E);       // elements per 16-byte chunk
    static constexpr int CPR = 32 * KS / CE;         // chunks per staged row
    static constexpr int LD = 32 * KS + CE;          // LDS row stride in elements (16-byte aligned rows, skewed banks)
};

__device__ __forceinline__ u32x4 zero_chunk() { return u32x4{0u, 0u, 0u, 0u}; }

// one 16-byte chunk of row `p` (null: a row outside the matrix) starting at k element k, K elements in the row
template <typename E>
__device__ __forceinline__ u32x4 load_chunk(const E* p, int k, int K, bool vec, float scale, bool scaled) {
    constexpr int CE = Tile<E>::CE;
    u32x4 c = zero_chunk();
    if (p == nullptr || k >= K) return c;
    if (vec) {
        c = *reinterpret_cast<const u32x4*>(p + k);
    } else {
        __attribute__((aligned(16))) E tmp[CE];
#pragma unroll
        for (int e = 0; e < CE; ++e) tmp[e] = k + e < K ? p[k + e] : from_f32<E>(0.0f);
        c = *reinterpret_cast<u32x4*>(tmp);
    }
    if (scaled) {
        __attribute__((aligned(16))) E tmp[CE];
        *reinterpret_cast<u32x4*>(tmp) = c;
#pragma unroll
        for (int e = 0; e < CE; ++e) tmp[e] = from_f32<E>(scale * to_f32(tmp[e]));
        c = *reinterpret_cast<u32x4*>(tmp);
    }
    return c;
}

__device__ __forceinline__ float apply_act(int act, float v, float param) {
    switch (act) {
        case PCB_ACT_SILU: return v / (1.0f + expf(-v));
        case PCB_ACT_SIGMOID: return 1.0f / (1.0f + expf(-v));
        case PCB_ACT_RELU2: return v > 0.0f ? v * v : 0.0f;
        case PCB_ACT_SOFTPLUS: return v > 20.0f ? v : log1pf(expf(v));
        case PCB_ACT_SOFTCAP: return param * tanhf(v / param);
        case PCB_ACT_RELU: return v > 0.0f ? v : 0.0f;
        case PCB_ACT_GELU_TANH: return 0.5f * v * (1.0f + tanhf(0.7978845608028654f * (v + 0.044715f * v * v * v)));
        case PCB_ACT_LOGSIGMOID: return param * (fminf(v, 0.0f) - log1pf(expf(-fabsf(v))));
        case PCB_ACT_SCALE: return param * v;
        default: return v;
    }
}

// the gated epilogue's function: silu (the default), relu or the tanh-form gelu, which is z sigmoid(2 u) for tanh's argument u.  Kept short:
// an epilogue too long to unroll would index the accumulators, which throws them out of the registers.
__device__ __forceinline__ float gate_act(int act, float v) {
    const float t = act == PCB_ACT_GELU_TANH ? 1.5957691216057308f * (v + 0.044715f * v * v * v) : v;
    const float s = v / (1.0f + expf(-t));
    return act == PCB_ACT_RELU ? fmaxf(v, 0.0f) : s;
}

// where one finished element goes (see pcb_linear_args)
template <typename E, int EPI>
__device__ __forceinline__ void put(const pcb_linear_args& a, int m, int n, float v, float cs) {
    if (EPI == PCB_EPI_SCALE_ADD) {
        float* y = (float*)a.y + (int64_t)m * a.ldy + n;
        const float b0 = a.base ? a.base[(int64_t)m * a.ldbase + n] : *y;
        *y = b0 + cs * v;
        return;
    }
    if (a.split_n3 > 0 && n >= a.split_n3) {
        ((E*)a.y3)[a.row_off3[m] + (int64_t)(n - a.split_n3) * a.col_stride3] = from_f32<E>(v);
        return;
    }
    if (a.split_n > 0 && n >= a.split_n) {
        const int c = n - a.split_n;
        if (a.y2_f32) {
            ((float*)a.y2)[m * a.head_stride2 + c] = v;
            return;
        }
        E* y = (E*)a.y2 + a.row_off2[m] + (int64_t)(c / a.head_dim2) * a.head_stride2 + c % a.head_dim2;
        *y = from_f32<E>(v);
        return;
    }
    const int64_t at = (int64_t)(a.row_dst ? a.row_dst[m] : m) * a.ldy + n + (a.n_batch > 0 ? (int64_t)blockIdx.z * a.y_batch_stride : 0);
    if (a.out_f32)
        ((float*)a.y)[at] = v;
    else
        ((E*)a.y)[at] = from_f32<E>(v);
}

// columns that pass through act / act2 of a plain store: the split-off parts are stored as they are
__device__ __forceinline__ int act_end(const pcb_linear_args& a) {
    return a.split_n > 0 ? a.split_n : (a.split_n3 > 0 ? a.split_n3 : a.N);
}

// one result element through the epilogue
template <typename E, int EPI>
__device__ __forceinline__ void emit(const pcb_linear_args& a, int m, int n, float acc, float acc2, float bv, float cs, float bv2 = 0.0f) {
    float v = acc + bv;
    if (EPI == PCB_EPI_STORE && (a.act | a.act2) && n < act_end(a))
        v = apply_act((a.act_split > 0 && n >= a.act_split) ? a.act2 : a.act, v, a.act_param);
    if (EPI == PCB_EPI_SILU_MUL) {
        v = gate_act(a.act, v) * (acc2 + bv2);
        if (a.row_gate) v *= to_f32(((const E*)a.row_gate)[m * a.ld_row_gate]);
    }
    put<E, EPI>(a, m, n, v, cs);
}

template <typename E, int EPI, int TM, int TN>
__global__ __launch_bounds__(256) void linear_kernel(pcb_linear_args a) {
    constexpr bool TWO = EPI == PCB_EPI_SILU_MUL;
    constexpr int BM = 32 * TM, BN = 32 * TN, BROWS = TWO ? 2 * BN : BN;
    constexpr int CE = Tile<E>::CE, CPR = Tile<E>::CPR, LD = Tile<E>::LD, KS = Tile<E>::KS;
    constexpr int A_CH = (BM * CPR + 255) / 256, B_CH = (BROWS * CPR + 255) / 256;
    __shared__ __attribute__((aligned(16))) E As[BM * LD];
    __shared__ __attribute__((aligned(16))) E Bs[BROWS * LD];

    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int wm = wave >> 1, wn = wave & 1, group = lane >> 4, l15 = lane & 15;
    const int K = a.K, N = a.N;

    // which rows: a plain launch tiles [0, M); a grouped launch walks the group offsets to find its group and tile
    int g = 0, m_lo, m_hi;
    if (a.n_groups > 0) {
        int t = blockIdx.y;
        m_lo = -1;
        for (g = 0; g < a.n_groups; ++g) {
            const int lo = a.group_off[g], hi = a.group_off[g + 1];
            const int nt = (hi - lo + BM - 1) / BM;
            if (t < nt) {
                m_lo = lo + t * BM;
                m_hi = hi;
                break;
            }
            t -= nt;
        }
        if (m_lo < 0) return;
    } else {
        m_lo = blockIdx.y * BM;
        m_hi = a.M;
        if (a.n_batch > 0) g = blockIdx.z;
        if (m_lo >= m_hi) return;
    }
    const int n_lo = blockIdx.x * BN;
    const E* W = (const E*)a.w + (int64_t)g * a.w_group_stride;
    const E* W2 = TWO ? (const E*)a.w2 + (int64_t)g * a.w_group_stride : nullptr;
    const E* X = (const E*)a.x + (a.n_batch > 0 ? (int64_t)blockIdx.z * a.x_batch_stride : 0);
    const bool vec = (K % CE == 0) && (a.ldx % CE == 0) && (a.ldw % CE == 0) && (((uintptr_t)X | (uintptr_t)W | (uintptr_t)W2) % 16 == 0);
    const bool scaled = a.row_scale != nullptr;

    // this thread's chunks of the two panels
    const E* a_row[A_CH];
    float a_scale[A_CH];
    int a_k[A_CH], a_at[A_CH];
#pragma unroll
    for (int i = 0; i < A_CH; ++i) {
        const int c = tid + 256 * i, r = c / CPR;
        a_k[i] = (c % CPR) * CE;
        a_at[i] = c < BM * CPR ? r * LD + a_k[i] : -1;
        const int m = m_lo + r;
        a_row[i] = nullptr;
        a_scale[i] = 1.0f;
        if (c < BM * CPR && m < m_hi) {
            a_row[i] = X + (int64_t)(a.row_src ? a.row_src[m] : m) * a.ldx;
            if (scaled) a_scale[i] = a.row_scale[m];
        }
    }
    const E* b_row[B_CH];
    int b_k[B_CH], b_at[B_CH];
#pragma unroll
    for (int i = 0; i < B_CH; ++i) {
        const int c = tid + 256 * i, r = c / CPR;
        b_k[i] = (c % CPR) * CE;
        b_at[i] = c < BROWS * CPR ? r * LD + b_k[i] : -1;
        const E* base = (TWO && r >= BN) ? W2 : W;
        const int n = n_lo + (TWO && r >= BN ? r - BN : r);
        b_row[i] = (c < BROWS * CPR && n < N) ? base + (int64_t)n * a.ldw : nullptr;
    }

    f4 acc[TM][TN], acc2[TWO ? TM : 1][TWO ? TN : 1];
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j) {
            acc[i][j] = f4{0.f, 0.f, 0.f, 0.f};
            if (TWO) acc2[i][j] = f4{0.f, 0.f, 0.f, 0.f};
        }

    u32x4 ra[A_CH], rb[B_CH];
#pragma unroll
    for (int i = 0; i < A_CH; ++i) ra[i] = load_chunk<E>(a_row[i], a_k[i], K, vec, a_scale[i], scaled);
#pragma unroll
    for (int i = 0; i < B_CH; ++i) rb[i] = load_chunk<E>(b_row[i], b_k[i], K, vec, 1.0f, false);

    for (int k0 = 0; k0 < K; k0 += 32 * KS) {
        __syncthreads();                           // the previous stage's fragment reads are done
#pragma unroll
        for (int i = 0; i < A_CH; ++i)
            if (a_at[i] >= 0) *reinterpret_cast<u32x4*>(&As[a_at[i]]) = ra[i];
#pragma unroll
        for (int i = 0; i < B_CH; ++i)
            if (b_at[i] >= 0) *reinterpret_cast<u32x4*>(&Bs[b_at[i]]) = rb[i];
        __syncthreads();
        if (k0 + 32 * KS < K) {
#pragma unroll
            for (int i = 0; i < A_CH; ++i) ra[i] = load_chunk<E>(a_row[i], k0 + 32 * KS + a_k[i], K, vec, a_scale[i], scaled);
#pragma unroll
            for (int i = 0; i < B_CH; ++i) rb[i] = load_chunk<E>(b_row[i], k0 + 32 * KS + b_k[i], K, vec, 1.0f, false);
        }
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            Frag<E> fa[TM];
#pragma unroll
            for (int i = 0; i < TM; ++i) fa[i] = load_frag(&As[((wm * TM + i) * 16 + l15) * LD + 32 * ks], group, 32, true);
#pragma unroll
            for (int j = 0; j < TN; ++j) {
                const Frag<E> fb = load_frag(&Bs[((wn * TN + j) * 16 + l15) * LD + 32 * ks], group, 32, true);
#pragma unroll
                for (int i = 0; i < TM; ++i) acc[i][j] = mma(fa[i], fb, acc[i][j]);
                if (TWO) {
                    const Frag<E> fb2 = load_frag(&Bs[(BN + (wn * TN + j) * 16 + l15) * LD + 32 * ks], group, 32, true);
#pragma unroll
                    for (int i = 0; i < TM; ++i) acc2[i][j] = mma(fa[i], fb2, acc2[i][j]);
                }
            }
        }
    }

    const E* bias = (const E*)a.bias;
#pragma unroll
    for (int j = 0; j < TN; ++j) {
        const int n = n_lo + (wn * TN + j) * 16 + l15;
        if (n >= N) continue;
        const float bv = bias ? to_f32(bias[n]) : 0.0f;
        const float bv2 = (TWO && a.bias2) ? to_f32(((const E*)a.bias2)[n]) : 0.0f;
        const float cs = (EPI == PCB_EPI_SCALE_ADD) ? a.col_scale[n] : 0.0f;
#pragma unroll
        for (int i = 0; i < TM; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int m = m_lo + (wm * TM + i) * 16 + 4 * group + r;
                if (m < m_hi) emit<E, EPI>(a, m, n, acc[i][j][r], TWO ? acc2[i][j][r] : 0.0f, bv, cs, bv2);
            }
    }
}

// ---- few rows: the weights stream once, straight from memory into the matrix cores --------------------------------------------
// Workgroup = 16 result columns x up to 16 rows; its SKW waves split the k range (k-step s goes to wave s % SKW) and add their
// partial tiles through LDS.  No LDS staging: a lane's B fragment is 16 contiguous bytes of its weight row, its A fragment 16
// bytes of its activation row (a handful of rows that stay in cache).
template <typename E>
__device__ __forceinline__ void scale_frag(Frag<E>& f, float s);
template <>
__device__ __forceinline__ void scale_frag<bf16_t>(Frag<bf16_t>& f, float s) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const uint32_t w = f.v[e];
        const uint32_t lo = bf16_bits(s * __uint_as_float(w << 16)), hi = bf16_bits(s * __uint_as_float(w & 0xffff0000u));
        f.v[e] = lo | (hi << 16);
    }
}
template <>
__device__ __forceinline__ void scale_frag<float>(Frag<float>& f, float s) {
#pragma unroll
    for (int e = 0; e < 8; ++e) f.v[e] *= s;
}

// the lane's elements of a whole k-step; p points at the first of them
__device__ __forceinline__ Frag<bf16_t> whole_frag(const bf16_t* p) {
    Frag<bf16_t> f;
    f.v = *reinterpret_cast<const u32x4*>(p);
    return f;
}
__device__ __forceinline__ Frag<float> whole_frag(const float* p) {
    Frag<float> f;
#pragma unroll
    for (int e = 0; e < 8; ++e) f.v[e] = p[4 * e];
    return f;
}

// SKW: waves of a workgroup (eight, or sixteen where few workgroups walk a long k range)
template <typename E, int EPI, int SKW>
__global__ __launch_bounds__(64 * SKW) void linear_skinny_kernel(pcb_linear_args a) {
    constexpr bool TWO = EPI == PCB_EPI_SILU_MUL;
    constexpr int CE = Tile<E>::CE;
    __shared__ f4 red[TWO ? 2 : 1][SKW][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, group = lane >> 4, l15 = lane & 15;
    const int K = a.K, N = a.N;
    int g = 0, m_lo, m_hi;
    if (a.n_groups > 0) {
        int t = blockIdx.y;
        m_lo = -1;
        for (g = 0; g < a.n_groups; ++g) {
            const int lo = a.group_off[g], hi = a.group_off[g + 1];
            const int nt = (hi - lo + 15) / 16;
            if (t < nt) {
                m_lo = lo + t * 16;
                m_hi = hi;
                break;
            }
            t -= nt;
        }
        if (m_lo < 0) return;
    } else {
        m_lo = blockIdx.y * 16;
        m_hi = a.M;
        if (a.n_batch > 0) g = blockIdx.z;
        if (m_lo >= m_hi) return;
    }
    const int n_lo = blockIdx.x * 16;
    const E* W = (const E*)a.w + (int64_t)g * a.w_group_stride;
    const E* W2 = TWO ? (const E*)a.w2 + (int64_t)g * a.w_group_stride : nullptr;
    const E* X = (const E*)a.x + (a.n_batch > 0 ? (int64_t)blockIdx.z * a.x_batch_stride : 0);
    const bool vec = (K % CE == 0) && (a.ldx % CE == 0) && (a.ldw % CE == 0) && (((uintptr_t)X | (uintptr_t)W | (uintptr_t)W2) % 16 == 0);
    const int n_b = n_lo + l15, m_a = m_lo + l15;
    const bool b_ok = n_b < N, a_ok = m_a < m_hi;
    const E* wrow = W + (int64_t)(b_ok ? n_b : 0) * a.ldw;
    const E* wrow2 = TWO ? W2 + (int64_t)(b_ok ? n_b : 0) * a.ldw : nullptr;
    const E* xrow = X + (int64_t)(a_ok ? (a.row_src ? a.row_src[m_a] : m_a) : 0) * a.ldx;
    const bool scaled = a.row_scale != nullptr;
    const float xs = (scaled && a_ok) ? a.row_scale[m_a] : 1.0f;
    f4 acc = f4{0.f, 0.f, 0.f, 0.f}, acc2 = f4{0.f, 0.f, 0.f, 0.f};
    const int nsteps = (K + 31) / 32;
    // whole k-steps of rows that can be read in 16-byte pieces: nothing between the loads.  (Lanes past the last row or column read row 0
    // or column 0 instead: what they multiply is not stored.)
    int st = wave;
    if (vec && !scaled) {
        const int whole = K / 32;
        const E* xp = xrow + (sizeof(E) == 2 ? 8 * group : group);
        const E* wp = wrow + (sizeof(E) == 2 ? 8 * group : group);
        const E* wp2 = TWO ? wrow2 + (sizeof(E) == 2 ? 8 * group : group) : nullptr;
#pragma unroll 8
        for (; st < whole; st += SKW) {
            const Frag<E> fa = whole_frag(xp + 32 * st), fb = whole_frag(wp + 32 * st);
            acc = mma(fa, fb, acc);
            if (TWO) acc2 = mma(fa, whole_frag(wp2 + 32 * st), acc2);
        }
    }
#pragma unroll 2
    for (; st < nsteps; st += SKW) {
        const int k0 = 32 * st;
        Frag<E> fa = load_frag(xrow + k0, group, a_ok ? K - k0 : 0, vec);
        if (scaled) scale_frag<E>(fa, xs);
        const Frag<E> fb = load_frag(wrow + k0, group, b_ok ? K - k0 : 0, vec);
        acc = mma(fa, fb, acc);
        if (TWO) {
            const Frag<E> fb2 = load_frag(wrow2 + k0, group, b_ok ? K - k0 : 0, vec);
            acc2 = mma(fa, fb2, acc2);
        }
    }
    red[0][wave][lane] = acc;
    if (TWO) red[1][wave][lane] = acc2;
    __syncthreads();
    if (wave != 0) return;
    acc = red[0][0][lane];
    if (TWO) acc2 = red[1][0][lane];
#pragma unroll
    for (int w = 1; w < SKW; ++w) {
        acc += red[0][w][lane];
        if (TWO) acc2 += red[1][w][lane];
    }
    const int n = n_lo + l15;
    if (n >= N) return;
    const E* bias = (const E*)a.bias;
    const float bv = bias ? to_f32(bias[n]) : 0.0f;
    const float bv2 = (TWO && a.bias2) ? to_f32(((const E*)a.bias2)[n]) : 0.0f;
    const float cs = (EPI == PCB_EPI_SCALE_ADD) ? a.col_scale[n] : 0.0f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int m = m_lo + 4 * group + r;
        if (m < m_hi) emit<E, EPI>(a, m, n, acc[r], acc2[r], bv, cs, bv2);
    }
}

// ---- many rows in bf16: both panels travel to LDS by themselves --------------------------------------------------------------------
// The same tiles (2 x 2 waves of TM x TN result tiles) for operands whose rows can be read in 16-byte chunks: global_load_lds carries a
// stage of 64 k elements (1 KiB per wave instruction: 8 rows x 128 bytes) straight into a ring of two or three images, one barrier per stage, so
// no register and no branch stands between the loads.  Rows past the end repeat the last one (their results are not stored); chunks
// past K come from a block of zeros.  The 16-byte chunk c of row r sits at position c ^ ((r >> 1) & 7) of its 128-byte row, which spreads
// a fragment read over all banks; the loads write lane by lane, so the permutation is applied to each lane's source.
// A plain launch numbers its tiles panel by panel (all row blocks of a column panel in turn) and gives each XCD one run of them: a
// panel's weights are fetched into one L2.
__device__ const u32x4 zero_row = {0u, 0u, 0u, 0u};

__device__ __forceinline__ void dma16(const void* g, void* lds_wave_base) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)g, (__attribute__((address_space(3))) void*)lds_wave_base, 16,
                                     0, 0);
}

template <int EPI, int TM, int TN, int STAGES>
__global__ __launch_bounds__(256) void linear_dma_kernel(pcb_linear_args a) {
    typedef bf16_t E;
    constexpr bool TWO = EPI == PCB_EPI_SILU_MUL;
    constexpr int BM = 32 * TM, BN = 32 * TN, ROWS = BM + (TWO ? 2 : 1) * BN, BK = 64;
    constexpr int NI = ROWS / 32;                                    // wave instructions per wave and stage
    __shared__ __attribute__((aligned(16))) E img[STAGES][ROWS * BK];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int wm = wave >> 1, wn = wave & 1, group = lane >> 4, l15 = lane & 15;
    const int K = a.K, N = a.N;

    int g = 0, m_lo = -1, m_hi = 0, n_lo;
    if (a.n_groups > 0) {
        int t = blockIdx.y;
        for (g = 0; g < a.n_groups; ++g) {
            const int lo = a.group_off[g], hi = a.group_off[g + 1];
            const int nt = (hi - lo + BM - 1) / BM;
            if (t < nt) {
                m_lo = lo + t * BM;
                m_hi = hi;
                break;
            }
            t -= nt;
        }
        if (m_lo < 0) return;
        n_lo = blockIdx.x * BN;
    } else {
        const int mb = (a.M + BM - 1) / BM, total = mb * ((N + BN - 1) / BN), per = (total + 7) / 8;
        const int t = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
        if ((int)(blockIdx.x >> 3) >= per || t >= total) return;
        m_lo = t % mb * BM;
        m_hi = a.M;
        n_lo = t / mb * BN;
        if (a.n_batch > 0) g = blockIdx.z;
    }
    const E* W = (const E*)a.w + (int64_t)g * a.w_group_stride;
    const E* W2 = TWO ? (const E*)a.w2 + (int64_t)g * a.w_group_stride : nullptr;
    const E* X = (const E*)a.x + (a.n_batch > 0 ? (int64_t)blockIdx.z * a.x_batch_stride : 0);

    // instruction i of this wave fills rows 8 (4 i + wave) .. + 7 of the image: A rows, then W rows, then W2 rows
    const E* src[NI];
    int kc[NI];                                                      // the lane's k offset within the stage
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int r = 8 * (4 * i + wave) + (lane >> 3);
        kc[i] = ((lane & 7) ^ ((r >> 1) & 7)) * 8;
        if (32 * i < BM) {
            int m = m_lo + r;
            m = m < m_hi ? m : m_hi - 1;
            src[i] = X + (int64_t)(a.row_src ? a.row_src[m] : m) * a.ldx;
        } else {
            const bool second = TWO && 32 * i >= BM + BN;
            int n = n_lo + r - BM - (second ? BN : 0);
            n = n < N ? n : N - 1;
            src[i] = (second ? W2 : W) + (int64_t)n * a.ldw;
        }
    }
    auto fetch = [&](int k0, int buf) {
        if (k0 + BK <= K) {
#pragma unroll
            for (int i = 0; i < NI; ++i) dma16(src[i] + k0 + kc[i], &img[buf][(4 * i + wave) * 8 * BK]);
        } else {
#pragma unroll
            for (int i = 0; i < NI; ++i)
                dma16(k0 + kc[i] < K ? (const void*)(src[i] + k0 + kc[i]) : (const void*)&zero_row, &img[buf][(4 * i + wave) * 8 * BK]);
        }
    };
    f4 acc[TM][TN], acc2[TWO ? TM : 1][TWO ? TN : 1];
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j) {
            acc[i][j] = f4{0.f, 0.f, 0.f, 0.f};
            if (TWO) acc2[i][j] = f4{0.f, 0.f, 0.f, 0.f};
        }
    auto frag = [&](int buf, int r, int ks) {
        Frag<E> f;
        f.v = *reinterpret_cast<const u32x4*>(&img[buf][r * BK + ((4 * ks + group) ^ ((r >> 1) & 7)) * 8]);
        return f;
    };
    // STAGES - 1 stages are in flight: at the top of a step the wave waits for its own part of the stage at hand (loads land in order),
    // the barrier then says that everyone's has landed and that the buffer of the step before is read out
#pragma unroll
    for (int p = 0; p < STAGES - 1; ++p)
        if (p * BK < K) fetch(p * BK, p);
    int buf = 0;
    for (int k0 = 0; k0 < K; k0 += BK, buf = buf + 1 == STAGES ? 0 : buf + 1) {
        if (STAGES > 2 && k0 + BK < K)
            asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"((STAGES - 2) * NI) : "memory");
        else
            asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        if (k0 + (STAGES - 1) * BK < K) fetch(k0 + (STAGES - 1) * BK, buf == 0 ? STAGES - 1 : buf - 1);
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            Frag<E> fa[TM];
#pragma unroll
            for (int i = 0; i < TM; ++i) fa[i] = frag(buf, (wm * TM + i) * 16 + l15, ks);
#pragma unroll
            for (int j = 0; j < TN; ++j) {
                const Frag<E> fb = frag(buf, BM + (wn * TN + j) * 16 + l15, ks);
#pragma unroll
                for (int i = 0; i < TM; ++i) acc[i][j] = mma(fb, fa[i], acc[i][j]);
                if (TWO) {
                    const Frag<E> fb2 = frag(buf, BM + BN + (wn * TN + j) * 16 + l15, ks);
#pragma unroll
                    for (int i = 0; i < TM; ++i) acc2[i][j] = mma(fb2, fa[i], acc2[i][j]);
                }
            }
        }
    }

    // (the weights are the products' first operand: a lane ends up with four neighbouring columns of one row.)
    // Bias, gate and activation first, in the accumulators -- an activation is chosen once, around the loop over them --, then the stores
    const E* bias = (const E*)a.bias;
    const E* bias2 = TWO ? (const E*)a.bias2 : nullptr;
#pragma unroll
    for (int j = 0; j < TN; ++j) {
        const int n = n_lo + (wn * TN + j) * 16 + 4 * group;
        if (bias || TWO) {
            float bv[4], bv2[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const bool in = n + e < N;
                bv[e] = bias && in ? to_f32(bias[n + e]) : 0.0f;
                bv2[e] = TWO && bias2 && in ? to_f32(bias2[n + e]) : 0.0f;
            }
#pragma unroll
            for (int i = 0; i < TM; ++i) {
                float rg = 1.0f;
                if (TWO && a.row_gate) {
                    const int m = m_lo + (wm * TM + i) * 16 + l15;
                    rg = to_f32(((const E*)a.row_gate)[(m < m_hi ? m : m_hi - 1) * a.ld_row_gate]);
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    acc[i][j][e] += bv[e];
                    if (TWO) acc[i][j][e] = gate_act(a.act, acc[i][j][e]) * (acc2[TWO ? i : 0][TWO ? j : 0][e] + bv2[e]) * rg;
                }
            }
        }
    }
    if (EPI == PCB_EPI_STORE && (a.act | a.act2)) {
        const int end = act_end(a), mid = a.act_split > 0 && a.act_split < end ? a.act_split : end;
        auto run = [&](auto code, int lo, int hi) {
            constexpr int A = decltype(code)::value;
#pragma unroll
            for (int j = 0; j < TN; ++j) {
                const int n = n_lo + (wn * TN + j) * 16 + 4 * group;
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e >= lo && n + e < hi) {
#pragma unroll
                        for (int i = 0; i < TM; ++i) acc[i][j][e] = apply_act(A, acc[i][j][e], a.act_param);
                    }
            }
        };
        auto pass = [&](int act, int lo, int hi) {
            if (n_lo >= hi || n_lo + BN <= lo) return;
            switch (act) {
                case PCB_ACT_SILU: run(std::integral_constant<int, PCB_ACT_SILU>{}, lo, hi); break;
                case PCB_ACT_SIGMOID: run(std::integral_constant<int, PCB_ACT_SIGMOID>{}, lo, hi); break;
                case PCB_ACT_RELU2: run(std::integral_constant<int, PCB_ACT_RELU2>{}, lo, hi); break;
                case PCB_ACT_SOFTPLUS: run(std::integral_constant<int, PCB_ACT_SOFTPLUS>{}, lo, hi); break;
                case PCB_ACT_SOFTCAP: run(std::integral_constant<int, PCB_ACT_SOFTCAP>{}, lo, hi); break;
                case PCB_ACT_RELU: run(std::integral_constant<int, PCB_ACT_RELU>{}, lo, hi); break;
                case PCB_ACT_GELU_TANH: run(std::integral_constant<int, PCB_ACT_GELU_TANH>{}, lo, hi); break;
                case PCB_ACT_LOGSIGMOID: run(std::integral_constant<int, PCB_ACT_LOGSIGMOID>{}, lo, hi); break;
                case PCB_ACT_SCALE: run(std::integral_constant<int, PCB_ACT_SCALE>{}, lo, hi); break;
                default: break;
            }
        };
#pragma unroll 1
        for (int part = 0; part < 2; ++part) pass(part ? a.act2 : a.act, part ? mid : 0, part ? end : mid);
    }
    const int whole = act_end(a);                                    // columns that go to y
    const int esz = (EPI == PCB_EPI_SCALE_ADD || a.out_f32) ? 4 : 2;
    const bool quads = a.ldy % 4 == 0 && (uintptr_t)a.y % (4 * esz) == 0 && a.y_batch_stride % 4 == 0 &&
                       (EPI != PCB_EPI_SCALE_ADD || !a.base || (a.ldbase % 4 == 0 && (uintptr_t)a.base % 16 == 0));
    const int64_t y0 = a.n_batch > 0 ? (int64_t)blockIdx.z * a.y_batch_stride : 0;
#pragma unroll
    for (int j = 0; j < TN; ++j) {
        const int n = n_lo + (wn * TN + j) * 16 + 4 * group;
        float cs[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) cs[e] = EPI == PCB_EPI_SCALE_ADD && n + e < N ? a.col_scale[n + e] : 0.0f;
        const bool quad = quads && n + 4 <= whole;
#pragma unroll
        for (int i = 0; i < TM; ++i) {
            const int m = m_lo + (wm * TM + i) * 16 + l15;
            if (m >= m_hi) continue;
            const f4 v = acc[i][j];
            if (quad) {
                if (EPI == PCB_EPI_SCALE_ADD) {
                    f4* y = reinterpret_cast<f4*>((float*)a.y + (int64_t)m * a.ldy + n);
                    const f4 b0 = a.base ? *reinterpret_cast<const f4*>(a.base + (int64_t)m * a.ldbase + n) : *y;
                    *y = f4{b0[0] + cs[0] * v[0], b0[1] + cs[1] * v[1], b0[2] + cs[2] * v[2], b0[3] + cs[3] * v[3]};
                } else {
                    const int64_t at = (int64_t)(a.row_dst ? a.row_dst[m] : m) * a.ldy + n + y0;
                    if (a.out_f32)
                        *reinterpret_cast<f4*>((float*)a.y + at) = v;
                    else
                        *reinterpret_cast<uint2*>((E*)a.y + at) = uint2{(uint32_t)bf16_bits(v[0]) | ((uint32_t)bf16_bits(v[1]) << 16),
                                                                        (uint32_t)bf16_bits(v[2]) | ((uint32_t)bf16_bits(v[3]) << 16)};
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < N) put<E, EPI>(a, m, n + e, v[e], cs[e]);
            }
        }
    }
}

template <int EPI, int TM, int TN, int STAGES>
int launch_dma(const pcb_linear_args& a, hipStream_t stream) {
    constexpr int BM = 32 * TM, BN = 32 * TN;
    const int nb = pcb_ceil_div(a.N, BN), mb = pcb_ceil_div(a.M, BM);
    const dim3 grid = a.n_groups > 0 ? dim3(nb, mb + a.n_groups) : dim3(8 * pcb_ceil_div(nb * mb, 8), 1, a.n_batch > 0 ? a.n_batch : 1);
    hipLaunchKernelGGL((linear_dma_kernel<EPI, TM, TN, STAGES>), grid, dim3(256), 0, stream, a);
    return pcb_check_launch("linear_dma_kernel");
}

// whether every operand row can be read in 16-byte chunks (bf16)
bool dma_ok(const pcb_linear_args& a) {
    return a.dtype == PCB_BF16 && !a.row_scale && a.K % 8 == 0 && a.ldx % 8 == 0 && a.ldw % 8 == 0 && a.w_group_stride % 8 == 0 &&
           a.x_batch_stride % 8 == 0 && ((uintptr_t)a.x | (uintptr_t)a.w | (uintptr_t)a.w2) % 16 == 0 &&
           (int64_t)pcb_ceil_div(a.N, 32) * pcb_ceil_div(a.M, 32) < (1 << 30);
}

template <int EPI>
int dispatch_dma(const pcb_linear_args& a, int rows, hipStream_t stream) {
    // the largest tile that still gives every CU a workgroup; grouped launches count the tiles their rows fill
    constexpr int TNW = EPI == PCB_EPI_SILU_MUL ? 2 : 4;
    const int64_t batch = a.n_batch > 0 ? a.n_batch : 1;
    auto tiles = [&](int bm, int bn) { return batch * pcb_ceil_div(a.M, bm) * pcb_ceil_div(a.N, bn); };
    // (two workgroups of a CU hide each other's loads behind their products; a lone one needs a stage more in flight)
    if (rows > 64 && tiles(128, 32 * TNW) > 256) return launch_dma<EPI, 4, TNW, 2>(a, stream);
    if (rows > 64 && tiles(128, 32 * TNW) == 256) return launch_dma<EPI, 4, TNW, 3>(a, stream);
    if (rows > 32 && tiles(64, 32 * TNW) >= 400) return launch_dma<EPI, 2, TNW, 3>(a, stream);
    if (rows > 32) return launch_dma<EPI, 2, TNW / 2, 3>(a, stream);
    return launch_dma<EPI, 1, TNW / 2, 3>(a, stream);
}

template <typename E, int EPI, int TM, int TN>
int launch(const pcb_linear_args& a, hipStream_t stream) {
    constexpr int BM = 32 * TM, BN = 32 * TN;
    const dim3 grid(pcb_ceil_div(a.N, BN), pcb_ceil_div(a.M, BM) + (a.n_groups > 0 ? a.n_groups : 0), a.n_batch > 0 ? a.n_batch : 1);
    hipLaunchKernelGGL((linear_kernel<E, EPI, TM, TN>), grid, dim3(256), 0, stream, a);
    return pcb_check_launch("linear_kernel");
}

template <typename E>
int dispatch(const pcb_linear_args& a, hipStream_t stream) {
    // rows per group decide the row tile: many rows -> 128-row panels, few -> 32-row panels (the weights stream once)
    const int rows = a.n_groups > 0 ? pcb_ceil_div(a.M, a.n_groups) : a.M;
    // (a narrow result -- router logits, step sizes: N <= 64 -- takes the 32-row panels too: 128-row panels would leave M / 128
    // workgroups on the chip, each walking all of K)
    const bool big = rows > 64 && a.N > 64;
    if (rows <= 16) {
        const dim3 grid(pcb_ceil_div(a.N, 16), pcb_ceil_div(a.M, 16) + (a.n_groups > 0 ? a.n_groups : 0), a.n_batch > 0 ? a.n_batch : 1);
        const bool deep = a.K >= 2048 && (int64_t)grid.x * grid.y * grid.z <= 192;
        auto go = [&](auto epi) {
            constexpr int EPI = decltype(epi)::value;
            if (deep)
                hipLaunchKernelGGL((linear_skinny_kernel<E, EPI, 16>), grid, dim3(64 * 16), 0, stream, a);
            else
                hipLaunchKernelGGL((linear_skinny_kernel<E, EPI, 8>), grid, dim3(64 * 8), 0, stream, a);
        };
        switch (a.epilogue) {
            case PCB_EPI_STORE: go(std::integral_constant<int, PCB_EPI_STORE>{}); break;
            case PCB_EPI_SILU_MUL: go(std::integral_constant<int, PCB_EPI_SILU_MUL>{}); break;
            default: go(std::integral_constant<int, PCB_EPI_SCALE_ADD>{});
        }
        return pcb_check_launch("linear_skinny_kernel");
    }
    if (sizeof(E) == 2 && dma_ok(a)) {
        switch (a.epilogue) {
            case PCB_EPI_STORE: return dispatch_dma<PCB_EPI_STORE>(a, rows, stream);
            case PCB_EPI_SILU_MUL: return dispatch_dma<PCB_EPI_SILU_MUL>(a, rows, stream);
            default: return dispatch_dma<PCB_EPI_SCALE_ADD>(a, rows, stream);
        }
    }
    switch (a.epilogue) {
        case PCB_EPI_STORE:
            return big ? launch<E, PCB_EPI_STORE, 4, 4>(a, stream) : launch<E, PCB_EPI_STORE, 1, 2>(a, stream);
        case PCB_EPI_SILU_MUL:
            return big ? launch<E, PCB_EPI_SILU_MUL, 4, 2>(a, stream) : launch<E, PCB_EPI_SILU_MUL, 1, 1>(a, stream);
        default:
            return big ? launch<E, PCB_EPI_SCALE_ADD, 4, 4>(a, stream) : launch<E, PCB_EPI_SCALE_ADD, 1, 2>(a, stream);
    }
}

}  // namespace

PCB_EXPORT int pcb_linear(const pcb_linear_args* a, void* stream) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_linear_args), PCB_ERR_ARG, "pcb_linear: struct size mismatch");
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "pcb_linear: unknown dtype");
    PCB_REQUIRE(a->M >= 0 && a->N > 0 && a->K > 0 && a->ldx >= a->K && a->ldw >= a->K, PCB_ERR_ARG, "pcb_linear: bad sizes");
    PCB_REQUIRE(a->epilogue >= PCB_EPI_STORE && a->epilogue <= PCB_EPI_SCALE_ADD, PCB_ERR_ARG, "pcb_linear: unknown epilogue");
    PCB_REQUIRE(a->act >= PCB_ACT_NONE && a->act <= PCB_ACT_SCALE && a->act2 >= PCB_ACT_NONE && a->act2 <= PCB_ACT_SCALE &&
                    a->act_split >= 0 &&
                    ((a->act | a->act2) == 0 || a->epilogue == PCB_EPI_STORE ||
                     (a->epilogue == PCB_EPI_SILU_MUL && a->act2 == 0 &&
                      (a->act == PCB_ACT_SILU || a->act == PCB_ACT_RELU || a->act == PCB_ACT_GELU_TANH))),
                PCB_ERR_ARG, "pcb_linear: an activation goes with the plain store epilogue (the gated one takes silu, relu or gelu_tanh)");
    PCB_REQUIRE((a->act != PCB_ACT_SOFTCAP && a->act2 != PCB_ACT_SOFTCAP) || a->act_param > 0.0f, PCB_ERR_ARG,
                "pcb_linear: the soft cap must be positive");
    if (a->M == 0) return PCB_OK;
    PCB_REQUIRE(a->x && a->w && a->y, PCB_ERR_ARG, "pcb_linear: null pointer");
    PCB_REQUIRE(a->n_groups >= 0 && (a->n_groups == 0 || a->group_off), PCB_ERR_ARG, "pcb_linear: groups need their offsets");
    PCB_REQUIRE(a->n_batch >= 0 && a->n_batch <= 65535 &&
                    (a->n_batch == 0 || (a->n_groups == 0 && a->epilogue == PCB_EPI_STORE && a->split_n == 0 && a->split_n3 == 0 && !a->bias &&
                                         !a->row_scale && a->x_batch_stride >= 0 && a->y_batch_stride >= 0 && a->w_group_stride >= 0)),
                PCB_ERR_ARG, "pcb_linear: a batch goes with plain stores (no groups, no split destinations, no bias)");
    PCB_REQUIRE(!a->row_gate || (a->epilogue == PCB_EPI_SILU_MUL && a->n_groups == 0 && a->ld_row_gate >= 1), PCB_ERR_ARG,
                "pcb_linear: a gate per row goes with the gated epilogue of a plain (ungrouped) launch");
    PCB_REQUIRE(a->epilogue != PCB_EPI_SILU_MUL || a->w2, PCB_ERR_ARG, "pcb_linear: the gated epilogue takes w2");
    PCB_REQUIRE(a->epilogue == PCB_EPI_SILU_MUL || !a->bias2, PCB_ERR_ARG, "pcb_linear: a second bias goes with the gated epilogue");
    PCB_REQUIRE(a->epilogue != PCB_EPI_SCALE_ADD || (a->col_scale && a->ldy >= a->N && !a->row_dst), PCB_ERR_ARG,
                "pcb_linear: scale-add needs col_scale and a plain fp32 destination");
    PCB_REQUIRE(a->split_n == 0 || (a->epilogue == PCB_EPI_STORE && a->split_n > 0 && a->split_n < a->N && a->y2 && a->row_off2 &&
                                    a->head_dim2 > 0 && a->ldy >= a->split_n) ||
                    (a->epilogue == PCB_EPI_STORE && a->split_n > 0 && a->split_n < a->N && a->y2 && a->y2_f32 && a->split_n3 == 0 &&
                     a->n_groups == 0 && a->head_stride2 >= a->N - a->split_n && a->ldy >= a->split_n),
                PCB_ERR_ARG, "pcb_linear: bad split destination");
    PCB_REQUIRE(a->split_n3 == 0 || (a->epilogue == PCB_EPI_STORE && a->split_n3 > a->split_n && a->split_n3 < a->N && a->y3 && a->row_off3 &&
                                     a->col_stride3 > 0 && (a->split_n > 0 || a->ldy >= a->split_n3)),
                PCB_ERR_ARG, "pcb_linear: bad column-wise destination");
    PCB_REQUIRE(a->split_n > 0 || a->split_n3 > 0 || a->epilogue == PCB_EPI_SCALE_ADD || a->ldy >= a->N, PCB_ERR_ARG, "pcb_linear: ldy < N");
    return a->dtype == PCB_BF16 ? dispatch<pcb::bf16_t>(*a, (hipStream_t)stream) : dispatch<float>(*a, (hipStream_t)stream);
}
