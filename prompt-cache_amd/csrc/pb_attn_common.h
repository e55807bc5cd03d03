// Pieces the attention kernels of libpromptcache_blocks.so share: softmax weights as an operand of the second product.
#pragma once
#include "pb_common.h"

#ifdef __HIPCC__
namespace pcb {

// eight softmax weights of a lane.  bf16: a hi + lo pair of bf16 values (two MFMAs), so that they are not rounded to 8 bits; fp32: as
// they are
template <typename E>
struct PFrag;
template <>
struct PFrag<bf16_t> {
    Frag<bf16_t> hi, lo;
};
template <>
struct PFrag<float> {
    Frag<float> hi;
};

__device__ __forceinline__ void make_p(PFrag<bf16_t>& f, const float (&p)[8]) {
    // hi = the upper 16 bits of p as they stand, lo = the rest, cut to 16 bits: hi + lo carries 16 bits of p's mantissa (p is a
    // finite non-negative weight, so no rounding carry or NaN needs care)
    uint32_t h[8], l[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const uint32_t u = __float_as_uint(p[e]);
        h[e] = u >> 16;
        l[e] = __float_as_uint(p[e] - __uint_as_float(u & 0xffff0000u)) >> 16;
    }
    f.hi.v = u32x4{h[0] | (h[1] << 16), h[2] | (h[3] << 16), h[4] | (h[5] << 16), h[6] | (h[7] << 16)};
    f.lo.v = u32x4{l[0] | (l[1] << 16), l[2] | (l[3] << 16), l[4] | (l[5] << 16), l[6] | (l[7] << 16)};
}
__device__ __forceinline__ void make_p(PFrag<float>& f, const float (&p)[8]) {
#pragma unroll
    for (int e = 0; e < 8; ++e) f.hi.v[e] = p[e];
}

__device__ __forceinline__ f4 mma_p(const Frag<bf16_t>& v, const PFrag<bf16_t>& p, f4 c) {
    c = mma(v, p.hi, c);
    return mma(v, p.lo, c);
}
__device__ __forceinline__ f4 mma_p(const Frag<float>& v, const PFrag<float>& p, f4 c) { return mma(v, p.hi, c); }

// ---- value operands out of an LDS tile kept key by key ([key][column], ld elements per key) ------------------------------------------
// The second product is O^T = V^T P^T: its A operand wants, per lane (value column l & 15, group l >> 4), eight keys of that column.  Key
// k index (group g, e) stands for key 4 g + e (e < 4) and 16 + 4 g + e - 4 (e >= 4) of the 32-key step -- what the lanes hold of the
// weights after S^T = K Q^T.
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

// `t` points at (key 0 of the step, column 0 of the 16-column block); transposed 8-byte reads: the 16 lanes of a group give the addresses
// of a 4-key x 16-column block (lane i: key i / 4, columns 4 (i % 4) ..) and receive its columns
__device__ __forceinline__ Frag<bf16_t> load_v_lds(const bf16_t* t, int ld, int g, int i) {
    const bf16_t* p = t + (4 * g + (i >> 2)) * ld + 4 * (i & 3);
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)p);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p + 16 * ld));
    Frag<bf16_t> f;
    const uint2 ua = __builtin_bit_cast(uint2, a), ub = __builtin_bit_cast(uint2, b);
    f.v = u32x4{ua.x, ua.y, ub.x, ub.y};
    return f;
}
__device__ __forceinline__ Frag<float> load_v_lds(const float* t, int ld, int g, int i) {
    Frag<float> f;
#pragma unroll
    for (int e = 0; e < 8; ++e) f.v[e] = t[(e < 4 ? 4 * g + e : 16 + 4 * g + e - 4) * ld + i];
    return f;
}

// elements per LDS row for `cols` columns (a multiple of 16): rows 8 (mod 16) dwords apart, so that four neighbouring keys of a transposed
// read fall on different banks
template <typename E>
__host__ __device__ constexpr int v_ld(int cols) {
    return sizeof(E) == 2 ? cols + (cols / 2 % 16 == 8 ? 0 : 16) : cols + 8;
}

}  // namespace pcb
#endif
