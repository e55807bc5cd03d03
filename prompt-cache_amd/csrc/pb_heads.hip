// pcb_head_prep: what happens to projected rows between the projection and the attention -- a unit-RMS norm per head (with or
// without a gain), a blend with another layer's values, rotary positions on neighbouring column pairs or on halves, and the store into a row
// matrix or a slot's cache (row by row or column by column).  Up to four segments (queries, keys, values, ...) per launch.
//
// One workgroup per (row, segment), or several that share the heads when rows are few.  The turn of every column pair depends on the row's position only, so the workgroup first
// fills a cos / sin table in LDS -- the angle is the float64 product position x frequency, reduced by float64 sincos, so a
// position in the thousands costs no bits of the angle -- and its waves then take the heads in turn: one pass for the sum of
// squares, one that norms, blends, turns and stores.  A lane owns the two columns of a pair, so a rotation never crosses lanes
// (and a segment may work in place).
#include "pb_common.h"

namespace {
using namespace pcb;

constexpr int MAX_PAIRS = 512;   // rotated column pairs per head

// the heads of one segment for one row: a wave takes a head (lanes step through its pairs), or -- LONE, a segment of one head: a latent of
// hundreds of columns -- the whole workgroup does
template <typename E, bool LONE>
__device__ __forceinline__ void prep_heads(const pcb_head_prep_args& a, const pcb_head_prep_seg& s, int64_t row, const float* cs, const float* sn,
                                           float* red) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int D = s.head_dim, np = s.rot_dims / 2;
    const int first = LONE ? (int)threadIdx.x : lane;
    constexpr int STEP = LONE ? 256 : 64;
    const float lam = s.blend ? s.blend[0] : 0.0f;
    for (int h = LONE ? 0 : wave + 4 * (int)blockIdx.z; h < s.heads; h += 4 * (int)gridDim.z) {
        const E* x = (const E*)s.src + row * s.ld_src + (int64_t)h * s.src_head_stride;
        float inv = 1.0f;
        if (s.norm) {
            float ss = 0.0f;
            for (int c = first; c < D; c += STEP) {
                const float v = to_f32(x[c]);
                ss += v * v;
            }
            ss = wave_sum(ss);
            if (LONE) {
                if (lane == 0) red[wave] = ss;
                __syncthreads();                             // (also: every column is read before one is written in place)
                ss = red[0] + red[1] + red[2] + red[3];
            }
            inv = 1.0f / sqrtf(ss / (float)D + a.eps);
        }
        const float* __restrict__ other = s.blend ? s.other + row * s.ld_other + (int64_t)h * D : nullptr;
        float* __restrict__ keep = s.keep ? s.keep + row * s.ld_keep + (int64_t)h * D : nullptr;
        E* dst = (E*)s.dst + (s.row_off ? s.row_off[row] : row * s.ld_dst) + (int64_t)h * s.head_stride;
        // a lane owns whole pairs: pair i < np turns by the position; of the columns that do not turn, pair i >= np is the next two
        // (interleaved rotation: the pairs in memory order, np of them from rot_off on)
        for (int i0 = first; 2 * i0 < D + 1; i0 += STEP) {
            int c[2];
            int i = -1;                                      // which angle, or none
            if (a.rot_half && np > 0) {
                if (i0 < np) {
                    c[0] = s.rot_off + i0;
                    c[1] = c[0] + np;
                    i = i0;
                } else {
#pragma unroll
                    for (int e = 0; e < 2; ++e) {
                        const int k = 2 * (i0 - np) + e;
                        c[e] = k < s.rot_off ? k : k + 2 * np;
                    }
                }
            } else {
                c[0] = 2 * i0;
                c[1] = c[0] + 1;
                const int k = (c[0] - s.rot_off) >> 1;       // (rot_off is even: a pair never straddles the rotated range's edge)
                if (c[0] >= s.rot_off && k < np) i = k;
            }
            float v[2];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                float t = 0.0f;
                if (c[e] < D) {
                    t = to_f32(x[c[e]]) * inv;
                    if (s.gain) t *= s.gain[c[e]];
                    if (other) t = (1.0f - lam) * t + lam * other[c[e]];
                    if (keep) keep[c[e]] = t;
                }
                v[e] = t;
            }
            if (i >= 0) {
                const float u = v[0], w = v[1];
                v[0] = u * cs[i] - w * sn[i];
                v[1] = w * cs[i] + u * sn[i];
            }
#pragma unroll
            for (int e = 0; e < 2; ++e)
                if (c[e] < D) dst[(int64_t)c[e] * s.col_stride] = from_f32<E>(v[e]);
        }
    }
}

template <typename E>
__global__ __launch_bounds__(256) void head_prep_kernel(pcb_head_prep_args a) {
    __shared__ float cs[MAX_PAIRS], sn[MAX_PAIRS], red[4];
    const pcb_head_prep_seg& s = a.seg[blockIdx.y];
    const int64_t row = blockIdx.x;
    const int np = s.rot_dims / 2;
    if (np > 0 && a.table) {
        for (int i = threadIdx.x; i < np; i += 256) {
            cs[i] = a.table[row * s.rot_dims + i];
            sn[i] = a.table[row * s.rot_dims + np + i];
        }
        __syncthreads();
    } else if (np > 0) {
        const double p = (double)a.pos[row];
        for (int i = threadIdx.x; i < np; i += 256) {
            double sv, cv;
            sincos(p * a.freqs[i], &sv, &cv);
            cs[i] = (float)cv * a.rot_mag;
            sn[i] = (float)sv * a.rot_mag;
        }
        __syncthreads();
    }
    if (s.heads == 1 && blockIdx.z > 0) return;
    if (s.heads == 1)
        prep_heads<E, true>(a, s, row, cs, sn, red);
    else
        prep_heads<E, false>(a, s, row, cs, sn, red);
}

__global__ __launch_bounds__(256) void rot_table_kernel(const int32_t* __restrict__ pos, const double* __restrict__ freqs, float mag,
                                                        float* __restrict__ out, int n_rows, int np) {
    const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (e >= (int64_t)n_rows * np) return;
    const int64_t r = e / np;
    const int i = (int)(e % np);
    double sv, cv;
    sincos((double)pos[r] * freqs[i], &sv, &cv);
    out[r * 2 * np + i] = (float)cv * mag;
    out[r * 2 * np + np + i] = (float)sv * mag;
}

}  // namespace

PCB_EXPORT int pcb_rot_table(const int32_t* pos, const double* freqs, float mag, float* out, int32_t n_rows, int32_t n_pairs, void* stream) {
    PCB_REQUIRE(n_rows >= 0 && n_pairs > 0 && n_pairs <= MAX_PAIRS, PCB_ERR_ARG, "pcb_rot_table: bad sizes (up to 512 pairs)");
    if (n_rows == 0) return PCB_OK;
    PCB_REQUIRE(pos && freqs && out, PCB_ERR_ARG, "pcb_rot_table: null pointer");
    const int64_t blocks = ((int64_t)n_rows * n_pairs + 255) / 256;
    hipLaunchKernelGGL(rot_table_kernel, dim3((uint32_t)blocks), dim3(256), 0, (hipStream_t)stream, pos, freqs, mag, out, n_rows, n_pairs);
    return pcb_check_launch("rot_table_kernel");
}

PCB_EXPORT int pcb_head_prep(const pcb_head_prep_args* a, void* stream) {
    PCB_REQUIRE(a && a->struct_bytes == sizeof(pcb_head_prep_args), PCB_ERR_ARG, "pcb_head_prep: struct size mismatch");
    PCB_REQUIRE(a->dtype == PCB_BF16 || a->dtype == PCB_F32, PCB_ERR_ARG, "pcb_head_prep: unknown dtype");
    PCB_REQUIRE(a->n_rows >= 0 && a->n_segs >= 1 && a->n_segs <= 4, PCB_ERR_ARG, "pcb_head_prep: one to four segments");
    int rot = 0;
    for (int i = 0; i < a->n_segs; ++i) {
        const pcb_head_prep_seg& s = a->seg[i];
        PCB_REQUIRE(s.heads > 0 && s.head_dim > 0 && s.head_dim <= 16384 && s.src_head_stride >= 0 && s.ld_src >= (int64_t)(s.heads - 1) * s.src_head_stride + s.head_dim && s.col_stride > 0,
                    PCB_ERR_ARG, "pcb_head_prep: bad segment sizes (heads of up to 16384 columns)");
        PCB_REQUIRE(s.rot_dims >= 0 && s.rot_dims % 2 == 0 && s.rot_off >= 0 && s.rot_off % 2 == 0 && s.rot_off + s.rot_dims <= s.head_dim &&
                        s.rot_dims <= 2 * MAX_PAIRS && (s.rot_dims == 0 || rot == 0 || rot == s.rot_dims),
                    PCB_ERR_ARG, "pcb_head_prep: rotated columns come in pairs inside the head, the same number in every segment that rotates");
        if (s.rot_dims) rot = s.rot_dims;
        PCB_REQUIRE(!s.blend || (s.other && s.ld_other >= (int64_t)s.heads * s.head_dim), PCB_ERR_ARG, "pcb_head_prep: a blend needs the other rows");
        PCB_REQUIRE(!s.keep || s.ld_keep >= (int64_t)s.heads * s.head_dim, PCB_ERR_ARG, "pcb_head_prep: keep rows too short");
        PCB_REQUIRE(a->n_rows == 0 || (s.src && s.dst), PCB_ERR_ARG, "pcb_head_prep: null pointer");
    }
    if (a->n_rows == 0) return PCB_OK;
    PCB_REQUIRE(rot == 0 || a->table || (a->pos && a->freqs), PCB_ERR_ARG, "pcb_head_prep: a rotation needs positions and frequencies");
    // (few rows: a row's heads are spread over workgroups, so that a wave has one)
    int most = 1;
    for (int i = 0; i < a->n_segs; ++i) most = a->seg[i].heads > most ? a->seg[i].heads : most;
    const dim3 grid(a->n_rows, a->n_segs, a->n_rows <= 64 ? pcb_ceil_div(most < 64 ? most : 64, 4) : 1);
    if (a->dtype == PCB_BF16)
        hipLaunchKernelGGL(head_prep_kernel<pcb::bf16_t>, grid, dim3(256), 0, (hipStream_t)stream, *a);
    else
        hipLaunchKernelGGL(head_prep_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, *a);
    return pcb_check_launch("head_prep_kernel");
}
