// pcb_attn_latent: causal softmax attention of single rows over ONE key head whose values are the leading columns of the key rows
// themselves (decoding over a shared latent: a cached row is latent | rotated key part, the queries come folded into that space).
//
// One workgroup = 16 heads of one query row x one run of the keys.  The run is walked in blocks of BK rows that go global -> registers
// -> LDS once (the next block's loads in flight) and are then read in both roles:
//   scores   S^T = K Q^T: wave w takes the 16 keys 16 w .. of the block (row-wise 16-byte reads), and leaves its 16 x 16 scores in LDS;
//   values   every wave takes all of the block's scores (the softmax weights of a head are in its lanes' column) and a quarter of the
//            value columns: O^T = V^T P^T with transposed reads of the same rows.
// So the weights are computed four times over (they are few), and no wave ever holds more than a quarter of the accumulator: latents of
// 512 columns fit, and nothing is merged between waves.
#include "pb_attn_common.h"

namespace {
using namespace pcb;

constexpr int LW = 4;          // waves of a workgroup

// KSQ: 32-element k-steps of a row; VBW: 16-column value blocks per wave; BK: rows per block
template <typename E, int KSQ, int VBW, int BK>
__global__ __launch_bounds__(64 * LW) void attn_latent_kernel(pcb_attn_latent_args a) {
    constexpr int CE = 16 / sizeof(E);
    constexpr int KC = KSQ * 32, LD = v_ld<E>(KC), NKT = BK / 16, NK2 = BK / 32;
    constexpr int LPR = 64 * LW / BK, NCH = KC / CE / LPR;           // threads that share a row: thread t loads row t / LPR, chunks t % LPR + i LPR
    static_assert(KC / CE % LPR == 0, "whole chunks per thread");
    __shared__ __attribute__((aligned(16))) E Ks[BK * LD];
    __shared__ f4 Ss[NKT][64];                                       // scores of key tile kt as the result tile's lanes hold them
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, c = lane & 15;
    const int32_t* tile = a.tiles + 4 * blockIdx.x;
    const int slot = tile[0], pos = tile[1];
    const int64_t qrow = tile[3];
    const int h0 = 16 * blockIdx.y;
    const int n_h = a.H - h0 < 16 ? a.H - h0 : 16;
    const int h = h0 + (c < n_h ? c : n_h - 1);                      // (lanes past the last head repeat it; nothing of theirs is stored)
    const int dim = a.dim, vdim = a.vdim;
    const E* K = (const E*)a.cache + (int64_t)slot * a.slot_stride;
    const bool kvec = ((uintptr_t)a.cache % 16 == 0) && a.slot_stride % CE == 0 && a.row_stride % CE == 0 && dim % CE == 0;
    const bool qvec = ((uintptr_t)a.q % 16 == 0) && (a.ldq % CE == 0) && (dim % CE == 0);
    const float sc = a.scale * 1.44269504088896f;                    // scores in units of ln 2
    const float NEG = -__builtin_inff();

    const int lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;     // the oldest key the row sees
    int kb_lo = lo / BK, kb_hi = pos / BK;
    if (a.n_splits > 1) {                                            // this workgroup's run of the blocks (it may be empty)
        const int per = (kb_hi - kb_lo + a.n_splits) / a.n_splits;
        kb_lo += (int)blockIdx.z * per;
        kb_hi = kb_lo + per - 1 < kb_hi ? kb_lo + per - 1 : kb_hi;
    }
    u32x4 rk[NCH];
    const int lr = tid / LPR, lc = tid % LPR * CE;                   // this thread's row and first column
    auto fetch = [&](int kb) {
        int j = kb * BK + lr;
        j = j > pos ? pos : j;                                       // (keys past the end repeat the last one: finite, and masked)
        const E* p = K + (int64_t)j * a.row_stride;
        if (kvec) {
#pragma unroll
            for (int i = 0; i < NCH; ++i) {
                const int col = lc + i * LPR * CE;
                rk[i] = u32x4{0u, 0u, 0u, 0u};
                if (col < dim) rk[i] = *reinterpret_cast<const u32x4*>(p + col);
            }
        } else {
#pragma unroll 1
            for (int i = 0; i < NCH; ++i) {
                const int col = lc + i * LPR * CE;
                __attribute__((aligned(16))) E tmp[CE];
#pragma unroll
                for (int e = 0; e < CE; ++e) tmp[e] = col + e < dim ? p[col + e] : from_f32<E>(0.0f);
                *reinterpret_cast<u32x4*>(&Ks[lr * LD + col]) = *reinterpret_cast<u32x4*>(tmp);
            }
        }
    };
    if (kvec && kb_lo <= kb_hi) fetch(kb_lo);
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
        if (kvec) {
#pragma unroll
            for (int i = 0; i < NCH; ++i) *reinterpret_cast<u32x4*>(&Ks[lr * LD + lc + i * LPR * CE]) = rk[i];
        } else {
            fetch(kb);                                               // (odd sizes: element by element, straight into LDS)
        }
        __syncthreads();
        if (kvec && kb < kb_hi) fetch(kb + 1);
        for (int kt = wave; kt < NKT; kt += LW) {
            f4 acc = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KSQ; ++ks) acc = mma(load_frag(&Ks[(kt * 16 + c) * LD + 32 * ks], g, 32, true), qf[ks], acc);
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
            for (int k2 = 0; k2 < NK2; ++k2) o[vb] = mma_p(load_v_lds(&Ks[k2 * 32 * LD + col], LD, g, c), pf[k2], o[vb]);
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (c >= n_h) return;
    float f = 1.0f;
    float* pp = nullptr;
    E* op = nullptr;
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
        if (a.gate) f *= to_f32(((const E*)a.gate)[qrow * a.ldg + h]);
        op = (E*)a.out + qrow * a.ldo + (int64_t)h * vdim;
    }
    const bool quads = vdim % 4 == 0 && (pp || (((uintptr_t)a.out % 16 == 0) && a.ldo % 4 == 0));
#pragma unroll
    for (int vb = 0; vb < VBW; ++vb) {
        const int col = (wave * VBW + vb) * 16 + 4 * g;
        if (quads && col < vdim) {
            if (pp)
                *reinterpret_cast<f4*>(pp + col) = o[vb];
            else
                store4(op + col, o[vb][0] * f, o[vb][1] * f, o[vb][2] * f, o[vb][3] * f);
            continue;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (col + r < vdim) {
                if (pp)
                    pp[col + r] = o[vb][r];
                else
                    op[col + r] = from_f32<E>(o[vb][r] * f);
            }
    }
}

// one workgroup per (row, head): the runs' factors once, then their partial results rescaled to the common maximum and summed
template <typename E>
__global__ __launch_bounds__(256) void attn_latent_merge_kernel(pcb_attn_latent_args a) {
    __shared__ float fac[64];
    const int64_t qrow = a.tiles[4 * blockIdx.x + 3];
    const int h = blockIdx.y, vdim = a.vdim, Z = a.n_splits, lane = threadIdx.x & 63;
    const int64_t run = ((int64_t)blockIdx.x * a.H + h) * Z;
    const float* pp = a.part + run * vdim;
    const float* ml = a.part + (int64_t)a.n_rows * a.H * Z * vdim + 2 * run;
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
        if (a.gate) f *= to_f32(((const E*)a.gate)[qrow * a.ldg + h]);
        fac[lane] = f;
    }
    __syncthreads();
    for (int c = threadIdx.x; c < vdim; c += 256) {
        float o = 0.0f;
#pragma unroll 8
        for (int z = 0; z < Z; ++z) o += fac[z] * pp[(int64_t)z * vdim + c];       // (an empty run left zeros)
        ((E*)a.out)[qrow * a.ldo + (int64_t)h * vdim + c] = from_f32<E>(o);
    }
}

template <typename E>
int dispatch(const pcb_attn_latent_args& a, hipStream_t stream) {
    constexpr int BK = sizeof(E) == 2 ? 64 : 32;
    const dim3 grid(a.n_rows, (a.H + 15) / 16, a.n_splits > 1 ? a.n_splits : 1), block(64 * LW);
    if (a.dim <= 128 && a.vdim <= 128)
        hipLaunchKernelGGL((attn_latent_kernel<E, 4, 2, BK>), grid, block, 0, stream, a);
    else if (a.dim <= 256 && a.vdim <= 256)
        hipLaunchKernelGGL((attn_latent_kernel<E, 8, 4, BK>), grid, block, 0, stream, a);
    else if (a.dim <= 384 && a.vdim <= 320)
        hipLaunchKernelGGL((attn_latent_kernel<E, 12, 5, BK>), grid, block, 0, stream, a);
    else if (a.dim <= 576)
        hipLaunchKernelGGL((attn_latent_kernel<E, 18, 8, BK>), grid, block, 0, stream, a);
    else
        hipLaunchKernelGGL((attn_latent_kernel<E, 24, 8, sizeof(E) == 2 ? 64 : 32>), grid, block, 0, stream, a);
    if (a.n_splits > 1) hipLaunchKernelGGL(attn_latent_merge_kernel<E>, dim3(a.n_rows, a.H), dim3(256), 0, stream, a);
    return pcb_check_launch("attn_latent_kernel");
}

}  // namespace

PCB_EXPORT int pcb_attn_latent(const pcb_attn_latent_args* a, void* stream) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_attn_latent_args), PCB_ERR_ARG, "pcb_attn_latent: struct size mismatch");
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "pcb_attn_latent: unknown dtype");
    PCB_REQUIRE(a->n_rows >= 0 && a->H > 0 && a->H <= 65535 && a->dim > 0 && a->dim <= 768 && a->vdim > 0 && a->vdim <= 512 &&
                    a->vdim <= a->dim && a->ldq >= (int64_t)a->H * a->dim && a->ldo >= (int64_t)a->H * a->vdim && a->row_stride >= a->dim &&
                    a->slot_stride >= 0,
                PCB_ERR_ARG, "pcb_attn_latent: bad sizes (rows of up to 768 columns, of which up to 512 are the value)");
    if (a->n_rows == 0) return PCB_OK;
    PCB_REQUIRE(a->q && a->tiles && a->cache && a->out && (!a->gate || a->ldg >= a->H), PCB_ERR_ARG, "pcb_attn_latent: null pointer");
    PCB_REQUIRE(a->n_splits <= 1 || (a->part && (uintptr_t)a->part % 16 == 0 && a->n_splits <= 64), PCB_ERR_ARG,
                "pcb_attn_latent: up to 64 runs, with their scratch");
    return a->dtype == PCB_BF16 ? dispatch<pcb::bf16_t>(*a, (hipStream_t)stream) : dispatch<float>(*a, (hipStream_t)stream);
}
