// Hyper-connections (ops_hyper.hip; the one-row form is a prologue of engine_stack.hip): s fp32 streams x_1 .. x_s instead of one.
//   a sublayer reads  u = sum_a in[a] x_a  and its output y goes back as  x_b <- sum_a mix[a][b] x_a + out[b] y
// Norms in `groups` equal parts of a row, each over its own root mean square.
#pragma once

#include "latent.hip.h"

namespace pgk {

constexpr int HYPER_MAX_STREAMS = 8, NORM_MAX_GROUPS = 4096;

// One step on rows: the pending sublayer's output goes into the streams (upd given), the next sublayer's normed input comes out.
// The output: y, rows of the element type or nslabs fp32 slabs whose sum is the row, + y_bias, times y_gate[row], + e_top rows of e.
struct HyperArgs {
    const float* src;                     // stream s of row r: src + r * src_row + s * src_stream (stride 0: all streams are equal)
    long long src_row, src_stream;
    float* dst;                           // [row][S][ld]; may be src; null: the new streams are not stored
    int S, W, ld, groups;
    float eps;
    const void* y; int ldy, nslabs;       // null: e alone
    long long slab_stride;
    const float *y_bias, *y_gate;         // [ld], [rows] or null
    const void* e; int e_top;             // [row][e_top][ld], element type, or null
    const float* upd;                     // of the pending sublayer: in [S] | out [S] | mix [S][S]; null: nothing is pending
    const float* in;                      // [S]; null: the sum of the streams
    const float* gamma;                   // [ld]
    void* out;                            // [ld] per workgroup, element type
    const int32_t* rows;                  // workgroup i works on row rows[i] (null: row i) and writes out row i
    const void* gate_w; float* gate_out;  // gate_out[row] = sigmoid(gate_w . normed row), gate_w [ld] in the element type; null: none
};
pgk_status hyper_rows(const HyperArgs& a, int n, pgk_dtype dt, hipStream_t st);

// 1 / root mean square of every group of a row of W elements in LDS -> rs [groups]; 256 threads, ends with a barrier
__device__ __forceinline__ void group_rstd(const float* row, int W, int groups, float eps, float* rs) {
    const int gs = W / groups;
    int lanes = 64;
    while (lanes > 1 && lanes * groups > 256) lanes >>= 1;
    const int lane = threadIdx.x & (lanes - 1);
    for (int g0 = 0; g0 < groups; g0 += 256 / lanes) {             // uniform
        const int g = g0 + (int)threadIdx.x / lanes;
        float ss = 0.f;
        if (g < groups) for (int i = lane; i < gs; i += lanes) { const float v = row[g * gs + i]; ss = fmaf(v, v, ss); }
        for (int off = lanes >> 1; off >= 1; off >>= 1) ss += __shfl_xor(ss, off, 64);
        if (g < groups && lane == 0) rs[g] = 1.0f / sqrtf(ss / gs + eps);
    }
    __syncthreads();
}

// rows of p(z) = a r(z) + b r(z^2) + c r(z^3) + e, r over the row's W elements; columns W .. ld are zero and stay so.  act: a, b, c, e
pgk_status poly_rows(const void* z, void* out, int n, int W, int ld, const float* act, float eps, pgk_dtype dt, hipStream_t st);
// coefficients of z, z^2, z^3 from the sums of z^2, z^4, z^6 over W elements
__device__ __forceinline__ float3 poly_coef(const float* act, float s2, float s4, float s6, int W, float eps) {
    return make_float3(act[0] / sqrtf(s2 / W + eps), act[1] / sqrtf(s4 / W + eps), act[2] / sqrtf(s6 / W + eps));
}
__device__ __forceinline__ float poly_at(const float3& c, float e, float z) { return fmaf(z, fmaf(z, fmaf(z, c.z, c.y), c.x), e); }

// x <- cap * tanh(x / cap)
__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }
pgk_status soft_cap_rows(float* x, size_t n, float cap, hipStream_t st);

}  // namespace pgk
