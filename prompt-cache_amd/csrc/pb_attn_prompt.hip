// pcb_attn_prompt: causal softmax attention of prompt rows over keys and values that lie as plain rows (a step's own, or rebuilt from
// a cached latent), tiled through LDS.
//
// One workgroup = 64 QT consecutive queries of one request x one query head; each of its four waves owns QT tiles of 16 queries.  The
// workgroup walks the keys in blocks of BK: the block's keys and values go global -> registers -> LDS (the next block's loads are in
// flight while this one is worked on) and serve all 64 QT queries.  Both products are "swapped" as in pb_attn_soft.hip:
//   S^T = K Q^T   K operand: 16-byte reads of LDS key rows; the lane's column is its query,
//   O^T = V^T P^T V operand: transposed LDS reads of the same row-major value tile (bf16), P straight from the lane's registers.
// A wave's queries are its own from start to end, so nothing is merged at the end.  Waves whose queries all precede a block skip its
// products; only blocks that straddle a query's own position or a window's edge pay for masks.  The keys' last tail_dim columns may be
// shared by all heads (one rotated part per token): they are then fetched from rows of their own, through an index table if given.
// Keys and values may also lie in a slot's cache, and a query may see its window or its block of positions only.
// Workgroups of one head are neighbours eight apart in launch order: they share that head's keys and values in one XCD's L2.
#include "pb_attn_common.h"

namespace {
using namespace pcb;

constexpr int PW = 4;          // waves of a workgroup

// one 16-byte chunk of E starting at column c of a row whose columns [c_lo, c_hi) lie at p; others read as zero
template <typename E>
__device__ __forceinline__ u32x4 part_chunk(const E* p, int c, int c_lo, int c_hi) {
    constexpr int CE = 16 / sizeof(E);
    __attribute__((aligned(16))) E tmp[CE];
#pragma unroll
    for (int e = 0; e < CE; ++e) tmp[e] = (c + e >= c_lo && c + e < c_hi) ? p[c + e - c_lo] : from_f32<E>(0.0f);
    return *reinterpret_cast<u32x4*>(tmp);
}

// the oldest key the query at position i sees (it never moves back as i grows)
__device__ __forceinline__ int oldest(const pcb_attn_prompt_args& a, int i) {
    int lo = a.window > 0 && i - a.window + 1 > 0 ? i - a.window + 1 : 0;
    if (a.block > 0) lo = max(lo, i / a.block * a.block);
    return lo;
}

// KSQ: 32-element k-steps of the key size; VB: 16-column blocks of the value size; BK: keys per block
template <typename E, int KSQ, int VB, int QT, int BK>
__global__ __launch_bounds__(64 * PW) void attn_prompt_kernel(pcb_attn_prompt_args a) {
    constexpr int CE = 16 / sizeof(E);
    constexpr int KC = KSQ * 32, VC = VB * 16;                       // columns of the tiles
    constexpr int KLD = KC + CE, VLD = v_ld<E>(VC);
    constexpr int LPR = 64 * PW / BK;                                // threads that share a row: thread t loads row t / LPR, chunks t % LPR + i LPR
    constexpr int KCH = KC / CE / LPR, VCH = VC / CE / LPR;          // 16-byte chunks per thread
    static_assert(KC / CE % LPR == 0 && VC / CE % LPR == 0, "whole chunks per thread");
    constexpr int NKT = BK / 16, NK2 = BK / 32;
    __shared__ __attribute__((aligned(16))) E Ks[BK * KLD];
    __shared__ __attribute__((aligned(16))) E Vs[BK * VLD];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
    const int h = blockIdx.x, hk = h / (a.H / a.Hkv);
    // (tiles from the last to the first: within a request later tiles see more keys, and the long ones should not start last)
    const int32_t* tile = a.tiles + 4 * (gridDim.y - 1 - blockIdx.y);
    const int base = tile[0], pos0 = tile[1], rows = tile[2], row0 = tile[3];
    const int dim = a.dim, vdim = a.vdim, split = dim - a.tail_dim;  // columns [0, split) per head, [split, dim) shared
    const int last = pos0 + rows - 1;
    const E* K = (const E*)a.k + (int64_t)base * (a.slots ? a.k_slot_stride : a.k_row_stride) + (int64_t)hk * a.k_head_stride;
    const E* V = (const E*)a.v + (int64_t)base * (a.slots ? a.v_slot_stride : a.v_row_stride) + (int64_t)hk * a.v_head_stride;
    const E* KT = (const E*)a.k_tail;
    const int32_t* trow = a.tail_rows ? a.tail_rows + base : nullptr;
    // whether every 16-byte chunk of a row lies in one part and can be read at once
    const bool plain = ((uintptr_t)a.k % 16 == 0) && a.k_row_stride % CE == 0 && a.k_head_stride % CE == 0 && ((uintptr_t)a.v % 16 == 0) &&
                       a.v_row_stride % CE == 0 && a.v_head_stride % CE == 0 && dim % CE == 0 && vdim % CE == 0 && split % CE == 0 &&
                       (!a.slots || (a.k_slot_stride % CE == 0 && a.v_slot_stride % CE == 0)) &&
                       (a.tail_dim == 0 || ((uintptr_t)a.k_tail % 16 == 0 && a.tail_row_stride % CE == 0));

    // this wave's queries
    const int w0 = wave * 16 * QT;                                   // first row of the wave within the tile
    const bool busy = w0 < rows;
    const int w_first = pos0 + w0, w_last = pos0 + (w0 + 16 * QT < rows ? w0 + 16 * QT : rows) - 1;
    const bool qvec = ((uintptr_t)a.q % 16 == 0) && (a.ldq % CE == 0) && (dim % CE == 0);
    Frag<E> qf[QT][KSQ];
    int qpos[QT], qlo[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        int qi = w0 + 16 * qt + c;
        qi = qi < rows ? qi : rows - 1;                              // (lanes past the tile repeat its last query; nothing of theirs is stored)
        qpos[qt] = pos0 + qi;
        qlo[qt] = oldest(a, pos0 + qi);
        const E* qp = (const E*)a.q + (int64_t)(row0 + qi) * a.ldq + (int64_t)h * dim;
#pragma unroll
        for (int ks = 0; ks < KSQ; ++ks) qf[qt][ks] = load_frag(qp + 32 * ks, g, dim - 32 * ks, qvec);
    }
    const float sc = a.scale * 1.44269504088896f;                    // scores in units of ln 2: every exponential is one v_exp_f32
    const float NEG = -__builtin_inff();
    float m[QT], l[QT];
    f4 o[QT][VB];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        m[qt] = NEG;
        l[qt] = 0.0f;
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) o[qt][vb] = f4{0.f, 0.f, 0.f, 0.f};
    }

    const int kb_lo = oldest(a, pos0) / BK;
    const int w_lo = oldest(a, w_first), w_lo_last = oldest(a, w_last);
    const int kb_hi = last / BK;
    u32x4 rk[KCH], rv[VCH];
    const int lr = tid / LPR, lc = tid % LPR * CE;                   // this thread's row and first column
    auto fetch = [&](int kb) {
        int j = kb * BK + lr;
        j = j > last ? last : j;                                     // (keys past the end repeat the last one: finite, and masked)
        const E* kp = K + (int64_t)j * a.k_row_stride;
        const E* vp = V + (int64_t)j * a.v_row_stride;
        const E* tp = a.tail_dim ? KT + (int64_t)(trow ? trow[j] : base + j) * a.tail_row_stride : kp;
        if (plain) {
#pragma unroll
            for (int i = 0; i < KCH; ++i) {
                const int col = lc + i * LPR * CE;
                rk[i] = u32x4{0u, 0u, 0u, 0u};
                if (col < dim) rk[i] = *reinterpret_cast<const u32x4*>(col < split ? kp + col : tp + (col - split));
            }
#pragma unroll
            for (int i = 0; i < VCH; ++i) {
                const int col = lc + i * LPR * CE;
                rv[i] = u32x4{0u, 0u, 0u, 0u};
                if (col < vdim) rv[i] = *reinterpret_cast<const u32x4*>(vp + col);
            }
        } else {
#pragma unroll 1
            for (int i = 0; i < KCH; ++i) {
                const int col = lc + i * LPR * CE;
                *reinterpret_cast<u32x4*>(&Ks[lr * KLD + col]) = part_chunk<E>(kp, col, 0, split) | part_chunk<E>(tp, col, split, dim);
            }
#pragma unroll 1
            for (int i = 0; i < VCH; ++i) {
                const int col = lc + i * LPR * CE;
                *reinterpret_cast<u32x4*>(&Vs[lr * VLD + col]) = part_chunk<E>(vp, col, 0, vdim);
            }
        }
    };
    if (plain) fetch(kb_lo);
    for (int kb = kb_lo; kb <= kb_hi; ++kb) {
        __syncthreads();                                             // the previous block's reads are done
        if (plain) {
#pragma unroll
            for (int i = 0; i < KCH; ++i) *reinterpret_cast<u32x4*>(&Ks[lr * KLD + lc + i * LPR * CE]) = rk[i];
#pragma unroll
            for (int i = 0; i < VCH; ++i) *reinterpret_cast<u32x4*>(&Vs[lr * VLD + lc + i * LPR * CE]) = rv[i];
        } else {
            fetch(kb);                                               // (odd sizes: element by element, straight into LDS)
        }
        __syncthreads();
        if (plain && kb < kb_hi) fetch(kb + 1);
        const int k0 = kb * BK;
        if (!busy || k0 > w_last || k0 + BK - 1 < w_lo) continue;

        f4 s[QT][NKT];
#pragma unroll
        for (int kt = 0; kt < NKT; ++kt) {
#pragma unroll
            for (int qt = 0; qt < QT; ++qt) s[qt][kt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KSQ; ++ks) {
                const Frag<E> kf = load_frag(&Ks[(kt * 16 + c) * KLD + 32 * ks], g, 32, true);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt) s[qt][kt] = mma(kf, qf[qt][ks], s[qt][kt]);
            }
        }
        const bool masked = k0 + BK - 1 > w_first || k0 < w_lo_last;
        PFrag<E> pf[QT][NK2];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            float bm = NEG;
#pragma unroll
            for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[qt][kt][r] * sc;
                    if (masked) {
                        const int key = k0 + kt * 16 + 4 * g + r;
                        if (key > qpos[qt] || key < qlo[qt]) v = NEG;
                    }
                    s[qt][kt][r] = v;
                    bm = fmaxf(bm, v);
                }
            bm = fmaxf(bm, __shfl_xor(bm, 16, 64));
            bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
            const float m_new = fmaxf(m[qt], bm);
            const float m_use = m_new == NEG ? 0.0f : m_new;
            const float alpha = __builtin_amdgcn_exp2f(m[qt] - m_use);          // (m = -inf: 0)
            float psum = 0.0f;
#pragma unroll
            for (int k2 = 0; k2 < NK2; ++k2) {
                float p[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    p[e] = __builtin_amdgcn_exp2f(s[qt][2 * k2 + (e >> 2)][e & 3] - m_use);
                    psum += p[e];
                }
                make_p(pf[qt][k2], p);
            }
            l[qt] = l[qt] * alpha + psum;
            if (__any(m_new != m[qt])) {                             // (a running maximum rarely moves after the first blocks)
#pragma unroll
                for (int vb = 0; vb < VB; ++vb)
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[qt][vb][r] *= alpha;
            }
            m[qt] = m_new;
        }
#pragma unroll
        for (int k2 = 0; k2 < NK2; ++k2)
#pragma unroll
            for (int vb = 0; vb < VB; ++vb) {
                const Frag<E> vf = load_v_lds(&Vs[k2 * 32 * VLD + vb * 16], VLD, g, c);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt) o[qt][vb] = mma_p(vf, pf[qt][k2], o[qt][vb]);
            }
    }
    if (!busy) return;
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        float lt = l[qt];
        lt += __shfl_xor(lt, 16, 64);
        lt += __shfl_xor(lt, 32, 64);
        if (w0 + 16 * qt + c >= rows) continue;
        float keep = 1.0f;
        if (a.sink) {
            // one more term exp(sink) without a value: the sum moves to the larger of the two maxima
            const float sk = a.sink[h] * 1.44269504088896f;
            const float top = fmaxf(m[qt], sk);
            keep = __builtin_amdgcn_exp2f(m[qt] - top);
            lt = lt * keep + __builtin_amdgcn_exp2f(sk - top);
        }
        const int64_t qrow = row0 + w0 + 16 * qt + c;
        float f = keep / lt;
        if (a.gate && !a.gate_cols) f *= to_f32(((const E*)a.gate)[qrow * a.ldg + h]);
        const E* gp = a.gate && a.gate_cols ? (const E*)a.gate + qrow * a.ldg + (int64_t)h * vdim : nullptr;
        E* op = (E*)a.out + qrow * a.ldo + (int64_t)h * vdim;
        const bool ovec = ((uintptr_t)a.out % 16 == 0) && a.ldo % 4 == 0 && vdim % 4 == 0;
        const bool gvec = gp && ((uintptr_t)a.gate % (4 * sizeof(E)) == 0) && a.ldg % 4 == 0 && vdim % 4 == 0;
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
            const int col = vb * 16 + 4 * g;
            float gv[4] = {f, f, f, f};
            if (gp) {
                load4(gp + col, gvec, vdim - col, gv);
#pragma unroll
                for (int r = 0; r < 4; ++r) gv[r] *= f;
            }
            if (ovec && col + 4 <= vdim) {
                store4(op + col, o[qt][vb][0] * gv[0], o[qt][vb][1] * gv[1], o[qt][vb][2] * gv[2], o[qt][vb][3] * gv[3]);
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (col + r < vdim) op[col + r] = from_f32<E>(o[qt][vb][r] * gv[r]);
            }
        }
    }
}

template <typename E, int KSQ, int VB, int BK>
int launch(const pcb_attn_prompt_args& a, hipStream_t stream) {
    const dim3 grid(a.H, a.n_tiles), block(64 * PW);
    if (sizeof(E) == 2 && a.tile_rows == 128)
        hipLaunchKernelGGL((attn_prompt_kernel<E, KSQ, VB, sizeof(E) == 2 ? 2 : 1, BK>), grid, block, 0, stream, a);
    else
        hipLaunchKernelGGL((attn_prompt_kernel<E, KSQ, VB, 1, BK>), grid, block, 0, stream, a);
    return pcb_check_launch("attn_prompt_kernel");
}

template <typename E>
int dispatch(const pcb_attn_prompt_args& a, hipStream_t stream) {
    constexpr bool B16 = sizeof(E) == 2;
    if (a.dim <= 64 && a.vdim <= 64) return launch<E, 2, 4, B16 ? 64 : 32>(a, stream);
    if (a.dim <= 128 && a.vdim <= 128) return launch<E, 4, 8, B16 ? 64 : 32>(a, stream);
    if (a.dim <= 192 && a.vdim <= 128) return launch<E, 6, 8, B16 ? 64 : 32>(a, stream);
    return launch<E, 8, 16, 32>(a, stream);
}

}  // namespace

PCB_EXPORT int pcb_attn_prompt(const pcb_attn_prompt_args* a, void* stream) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_attn_prompt_args), PCB_ERR_ARG, "pcb_attn_prompt: struct size mismatch");
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "pcb_attn_prompt: unknown dtype");
    PCB_REQUIRE(a->n_tiles >= 0 && a->n_tiles <= 65535 && a->H > 0 && a->Hkv > 0 && a->H % a->Hkv == 0 && a->dim > 0 && a->dim <= 256 &&
                    a->vdim > 0 && a->vdim <= 256 && a->tail_dim >= 0 && a->tail_dim < a->dim && a->ldq >= (int64_t)a->H * a->dim &&
                    a->ldo >= (int64_t)a->H * a->vdim && a->k_row_stride > 0 && a->k_head_stride >= 0 && a->v_row_stride > 0 &&
                    a->v_head_stride >= 0,
                PCB_ERR_ARG, "pcb_attn_prompt: bad sizes (key and value sizes up to 256, the shared part less than the key)");
    PCB_REQUIRE(a->tile_rows == 64 || (a->tile_rows == 128 && a->dtype == PCB_BF16), PCB_ERR_ARG,
                "pcb_attn_prompt: tiles of 64 rows, or 128 in bf16");
    if (a->n_tiles == 0) return PCB_OK;
    PCB_REQUIRE(a->q && a->tiles && a->k && a->v && a->out && (a->tail_dim == 0 || (a->k_tail && a->tail_row_stride >= a->tail_dim)) &&
                    (!a->gate || a->ldg >= (a->gate_cols ? (int64_t)a->H * a->vdim : (int64_t)a->H)),
                PCB_ERR_ARG, "pcb_attn_prompt: null pointer");
    PCB_REQUIRE(!a->slots || (a->tail_dim == 0 && a->k_slot_stride >= 0 && a->v_slot_stride >= 0), PCB_ERR_ARG,
                "pcb_attn_prompt: keys in slots have no shared part");
    return a->dtype == PCB_BF16 ? dispatch<pcb::bf16_t>(*a, (hipStream_t)stream) : dispatch<float>(*a, (hipStream_t)stream);
}
