// Gated linear recurrence (mixers.hip.h): per head a state S [dim][vdim] in fp32, S <- diag(f) S + (1 - f) v^T, o = S^T q.
// Gates, state and the head norm are fp32 whatever the element type.

#include <type_traits>

#include "mixers.hip.h"

namespace pgk {

__device__ __forceinline__ float rc_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// forget gate and write strength: f = l + (1 - l) sigmoid(z), 1 - f = (1 - l) sigmoid(-z) (no cancellation near f = 1)
__device__ __forceinline__ void rc_gate(float z, float lower, float& f, float& k) {
    const float e = expf(-fabsf(z)), big = 1.0f / (1.0f + e), small = e * big;
    f = fmaf(1.0f - lower, z >= 0.f ? big : small, lower);
    k = (1.0f - lower) * (z >= 0.f ? small : big);
}

// -------------------------------------------------------------------------------------------- token by token
// One workgroup per (sequence, head).  A thread owns VEC columns of every NG-th state row (VEC = 4: one 16-byte access each); a
// sequence that starts (position 0) begins with a zero state without reading the slot.
template <class IT, int VEC>
__global__ __launch_bounds__(512) void recur_scan_kernel(unsigned long long* tl, RecurArgs a) {
    const TLStamp tls(tl);
    extern __shared__ float sm[];
    __shared__ float red[16];
    const int tid = threadIdx.x, NT = blockDim.x, h = blockIdx.x, dim = a.dim, vdim = a.vdim;
    const int NC = vdim / VEC, NG = max(NT / NC, 1), c = tid % NC, g = tid / NC;
    float *q = sm, *f = q + dim, *k = f + dim, *v = k + dim, *po = v + vdim;          // po [NG][vdim]
    SeqSpan s;
    if (a.seqs) s = a.seqs[blockIdx.y];
    else { s.row0 = blockIdx.y; s.len = 1; s.start = max(a.positions[blockIdx.y], 0); s.slot = blockIdx.y; }
    float* S = a.state + ((size_t)s.slot * a.H + h) * dim * vdim;
    for (int t = 0; t < s.len; ++t) {
        const IT* in = reinterpret_cast<const IT*>(a.in) + (size_t)(s.row0 + t) * a.ld_in;
        const bool fresh = s.start + t == 0;
        for (int d = tid; d < dim; d += NT) {
            const float zq = to_f(in[a.q_off + h * dim + d]), zf = to_f(in[a.f_off + h * dim + d]) + (a.bias ? a.bias[h * dim + d] : 0.f);
            q[d] = zq * rc_sigmoid(zq);
            rc_gate(zf, a.lower[h * dim + d], f[d], k[d]);
        }
        for (int i = tid; i < vdim; i += NT) v[i] = to_f(in[a.v_off + h * vdim + i]);
        __syncthreads();
        if (g < NG) {
            for (int cc = c; cc < NC; cc += NT) {                  // (one trip unless a head has more columns than the workgroup threads)
                float acc[VEC], vv[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) { acc[e] = 0.f; vv[e] = v[cc * VEC + e]; }
                constexpr int U = 4;
                for (int d0 = g; d0 < dim; d0 += U * NG) {
                    float x[U][VEC];
#pragma unroll
                    for (int u = 0; u < U; ++u) {
                        const int d = min(d0 + u * NG, dim - 1);
                        if (fresh) {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) x[u][e] = 0.f;
                        } else if constexpr (VEC == 4) {
                            const float4 r = *reinterpret_cast<const float4*>(S + (size_t)d * vdim + cc * 4);
                            x[u][0] = r.x; x[u][1] = r.y; x[u][2] = r.z; x[u][3] = r.w;
                        } else x[u][0] = S[(size_t)d * vdim + cc];
                    }
#pragma unroll
                    for (int u = 0; u < U; ++u) {
                        const int d = d0 + u * NG;
                        if (d >= dim) break;
#pragma unroll
                        for (int e = 0; e < VEC; ++e) {
                            x[u][e] = fmaf(f[d], x[u][e], k[d] * vv[e]);
                            acc[e] = fmaf(q[d], x[u][e], acc[e]);
                        }
                        if constexpr (VEC == 4) *reinterpret_cast<float4*>(S + (size_t)d * vdim + cc * 4) = make_float4(x[u][0], x[u][1], x[u][2], x[u][3]);
                        else S[(size_t)d * vdim + cc] = x[u][0];
                    }
                }
#pragma unroll
                for (int e = 0; e < VEC; ++e) po[g * vdim + cc * VEC + e] = acc[e];
            }
        }
        __syncthreads();
        float ss = 0.f;
        for (int i = tid; i < vdim; i += NT) {
            float o = 0.f;
            for (int j = 0; j < NG; ++j) o += po[j * vdim + i];
            v[i] = o;                                              // the column's own thread: read again below
            ss = fmaf(o, o, ss);
        }
        float inv = 1.f;
        if (a.norm) inv = 1.0f / sqrtf(block_sum(ss, red) / a.vdim_true + a.eps);
        IT* out = reinterpret_cast<IT*>(a.out) + (size_t)(s.row0 + t) * a.ld_out;
        for (int i = tid; i < vdim; i += NT) out[h * vdim + i] = from_f<IT>(v[i] * inv * (a.norm ? a.norm[i] : 1.f));
        if (h == a.H - 1)
            for (int i = a.H * vdim + tid; i < a.ld_out; i += NT) out[i] = from_f<IT>(0.f);
        __syncthreads();                                           // q, f, k, v and po are rewritten by the next token
    }
    tls.end();
}

template <class IT>
static pgk_status recur_scan(const RecurArgs& a, hipStream_t st) {
    const int B = a.seqs ? a.n_seqs : a.n, threads = a.dim * a.vdim >= 8192 ? 512 : 256;
    const bool vec = a.vdim % 4 == 0;
    const int cols = vec ? a.vdim / 4 : a.vdim, groups = threads / cols > 0 ? threads / cols : 1;
    const size_t lds = (size_t)(3 * a.dim + a.vdim + groups * a.vdim) * 4;
    PGK_REQUIRE(lds <= 64 * 1024, "recurrence: head widths %d / %d do not fit LDS", a.dim, a.vdim);
    if (vec) PGK_CHECK_HIP(launch_k(&recur_scan_kernel<IT, 4>, dim3(a.H, B), dim3(threads), lds, st, a));
    else PGK_CHECK_HIP(launch_k(&recur_scan_kernel<IT, 1>, dim3(a.H, B), dim3(threads), lds, st, a));
    return PGK_OK;
}

pgk_status recur_rows(const RecurArgs& a, pgk_dtype dt, bool io32, hipStream_t st) {
    PGK_REQUIRE(a.H >= 1 && a.dim >= 1 && a.vdim >= 1 && a.ld_out >= a.H * a.vdim && (a.seqs || a.positions), "recurrence: bad sizes");
    return dt == PGK_F32 || io32 ? recur_scan<float>(a, st) : recur_scan<bf16>(a, st);
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_gated_recurrence(const void* q, const void* f, const void* v, const float* f_bias, const float* lower, const float* norm, float* state, void* out, int n,
                                int fresh, int heads, int dim, int vdim, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(q && f && v && lower && state && out, "pgk_gated_recurrence: null pointer");
    PGK_REQUIRE(n >= 1 && heads >= 1 && dim >= 1 && vdim >= 1, "pgk_gated_recurrence: bad shape %d x %d x %d, %d rows", heads, dim, vdim, n);
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_gated_recurrence: dtype %d (bf16 or f32)", (int)dt);
    hipStream_t st = resolve_stream(s);
    // one row buffer q | f | v, and the portion table behind it
    const size_t E = dtype_size(dt), row = (size_t)heads * (2 * dim + vdim), bytes = ((size_t)n * row * E + 255) & ~(size_t)255;
    char* ws = nullptr;
    if (pgk_status r = pgk_malloc((void**)&ws, bytes + sizeof(SeqSpan))) return r;
    const size_t wq = (size_t)heads * dim * E, wv = (size_t)heads * vdim * E;
    const SeqSpan span{0, n, fresh ? 0 : 1, 0};
    hipError_t e = hipMemcpy2DAsync(ws, row * E, q, wq, wq, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpy2DAsync(ws + wq, row * E, f, wq, wq, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpy2DAsync(ws + 2 * wq, row * E, v, wv, wv, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + bytes, &span, sizeof(span), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    RecurArgs a{};
    a.in = ws; a.ld_in = (int)row; a.f_off = heads * dim; a.v_off = 2 * heads * dim;
    a.bias = f_bias; a.lower = lower; a.norm = norm; a.H = heads; a.dim = dim; a.vdim = a.vdim_true = vdim; a.n = n; a.eps = eps;
    a.state = state; a.seqs = (const SeqSpan*)(ws + bytes); a.n_seqs = 1; a.out = out; a.ld_out = heads * vdim;
    pgk_status r = e == hipSuccess ? recur_rows(a, dt, false, st) : set_error(PGK_ERR_HIP, "pgk_gated_recurrence: %s", hipGetErrorString(e));
    pgk_free(ws);       // stream-ordered reuse: later work on this stream runs after the kernel above
    return r;
}

}  // extern "C"
