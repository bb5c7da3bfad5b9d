// Hyper-connected residual streams, norms in groups, polynomial-norm activation, soft cap (hyper.hip.h).

#include <type_traits>

#include "hyper.hip.h"

namespace pgk {

__device__ __forceinline__ float4 fma_s(float s, const float4& x, const float4& y) { return make_float4(fmaf(s, x.x, y.x), fmaf(s, x.y, y.y), fmaf(s, x.z, y.z), fmaf(s, x.w, y.w)); }

// A workgroup per row, NT float4 per thread, up to SM streams
template <class T, class YT, int NT, int SM>
__global__ __launch_bounds__(256) void hyper_rows_kernel(HyperArgs a) {
    extern __shared__ __attribute__((aligned(16))) float hy_smem[];          // groups > 1: [ld] | [groups]
    __shared__ float red[16];
    const int row = a.rows ? a.rows[blockIdx.x] : blockIdx.x, nt = a.ld, S = a.S;
    const float* src = a.src + (size_t)row * a.src_row;
    float* dst = a.dst ? a.dst + (size_t)row * S * a.ld : nullptr;
    const YT* yr = reinterpret_cast<const YT*>(a.y) + (size_t)row * a.ldy;
    const T* er = reinterpret_cast<const T*>(a.e) + (size_t)row * a.e_top * a.ld;
    const float4 zero = {0.f, 0.f, 0.f, 0.f};
    const float gate = a.y_gate ? a.y_gate[row] : 1.0f;
    float cin[SM], cout[SM], mix[SM][SM];
#pragma unroll
    for (int s = 0; s < SM; ++s) {
        cin[s] = s >= S ? 0.f : a.in ? a.in[s] : 1.0f;
        cout[s] = s < S && a.upd ? a.upd[S + s] : 0.f;
#pragma unroll
        for (int t = 0; t < SM; ++t) mix[s][t] = s < S && t < S && a.upd ? a.upd[2 * S + s * S + t] : 0.f;
    }
    float4 u[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4, ic = min(i, nt - 4);
        float4 x[SM];
#pragma unroll
        for (int s = 0; s < SM; ++s) x[s] = s < S ? *reinterpret_cast<const float4*>(src + s * a.src_stream + ic) : zero;
        u[t] = zero;
        if (a.upd) {
            float4 y = a.y ? load4<YT>(yr + ic) : zero;
#pragma unroll 8
            for (int s = 1; s < a.nslabs; ++s) { const float4 q = load4<YT>(yr + s * a.slab_stride + ic); y.x += q.x; y.y += q.y; y.z += q.z; y.w += q.w; }
            if (a.y_bias) y = fma_s(1.0f, *reinterpret_cast<const float4*>(a.y_bias + ic), y);
            y.x *= gate; y.y *= gate; y.z *= gate; y.w *= gate;
            if (a.e) {
#pragma unroll 4
                for (int k = 0; k < a.e_top; ++k) y = fma_s(1.0f, load4<T>(er + (size_t)k * a.ld + ic), y);
            }
#pragma unroll
            for (int o = 0; o < SM; ++o) {
                if (o >= S) break;
                float4 v = zero;
#pragma unroll
                for (int s = 0; s < SM; ++s) v = fma_s(mix[s][o], x[s], v);
                v = fma_s(cout[o], y, v);
                if (dst && i < nt) *reinterpret_cast<float4*>(dst + (size_t)o * a.ld + i) = v;
                u[t] = fma_s(cin[o], v, u[t]);
            }
        } else {
#pragma unroll
            for (int s = 0; s < SM; ++s) u[t] = fma_s(cin[s], x[s], u[t]);
        }
        if (i >= nt) u[t] = zero;
    }
    if (!a.out) return;
    const int gs = a.W / a.groups;
    float inv1 = 0.f;
    float *lrow = hy_smem, *rs = hy_smem + a.ld;
    if (a.groups == 1) {
        float ss = 0.f;
#pragma unroll
        for (int t = 0; t < NT; ++t) ss += u[t].x * u[t].x + u[t].y * u[t].y + u[t].z * u[t].z + u[t].w * u[t].w;      // (columns W .. ld are zero)
        inv1 = 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps);
    } else {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < nt) *reinterpret_cast<float4*>(lrow + i) = u[t];
        }
        __syncthreads();
        group_rstd(lrow, a.W, a.groups, a.eps, rs);
    }
    T* o = reinterpret_cast<T*>(a.out) + (size_t)blockIdx.x * a.ld;
    const T* gw = reinterpret_cast<const T*>(a.gate_w);
    float dot = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4;
        if (i >= nt) continue;
        float4 r = {inv1, inv1, inv1, inv1};
        if (a.groups > 1) {
            if ((gs & 3) == 0) { const float q = rs[min(i / gs, a.groups - 1)]; r = make_float4(q, q, q, q); }
            else r = make_float4(rs[min(i / gs, a.groups - 1)], rs[min((i + 1) / gs, a.groups - 1)], rs[min((i + 2) / gs, a.groups - 1)], rs[min((i + 3) / gs, a.groups - 1)]);
        }
        const float4 g = *reinterpret_cast<const float4*>(a.gamma + i);      // zero in columns W .. ld
        const float4 v = make_float4(u[t].x * r.x * g.x, u[t].y * r.y * g.y, u[t].z * r.z * g.z, u[t].w * r.w * g.w);
        store4<T>(o + i, v);
        if (gw) { const float4 w = load4<T>(gw + i); dot += (v.x * w.x + v.y * w.y) + (v.z * w.z + v.w * w.w); }
    }
    if (gw) {
        __syncthreads();                                           // (`red` may still be read)
        dot = block_sum(dot, red);
        if (threadIdx.x == 0) a.gate_out[row] = 1.0f / (1.0f + expf(-dot));
    }
}

template <class T, class YT, int NT>
static pgk_status hyper_rows_s(const HyperArgs& a, int n, hipStream_t st) {
    const size_t lds = a.groups > 1 ? (size_t)(a.ld + a.groups) * 4 : 0;
    auto go = [&](auto sm) -> pgk_status {
        auto kfn = &hyper_rows_kernel<T, YT, NT, decltype(sm)::value>;
        static bool done = false;
        if (lds > 48 * 1024 && !done) {
            PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024));
            done = true;
        }
        kfn<<<n, 256, lds, st>>>(a);
        PGK_LAUNCH_CHECK();
        return PGK_OK;
    };
    return a.S <= 2 ? go(std::integral_constant<int, 2>{}) : a.S <= 4 ? go(std::integral_constant<int, 4>{}) : go(std::integral_constant<int, 8>{});
}
template <class T, class YT>
static pgk_status hyper_rows_t(const HyperArgs& a, int n, hipStream_t st) {
    PGK_REQUIRE(a.src && a.S >= 1 && a.S <= HYPER_MAX_STREAMS && a.ld % 4 == 0 && a.W >= 1 && a.W <= a.ld && a.groups >= 1 && a.groups <= NORM_MAX_GROUPS && a.W % a.groups == 0 &&
                    (!a.out || a.gamma) && (!a.y || a.upd) && (!a.upd || a.y || a.e) && (!a.e || (a.upd && a.e_top >= 1)) && (!a.gate_w || (a.out && a.gate_out)) && (!a.rows || !a.dst),
                "hyper_rows: %d streams of %d (stride %d), %d groups", a.S, a.W, a.ld, a.groups);
    if (a.ld <= 1024) return hyper_rows_s<T, YT, 1>(a, n, st);
    if (a.ld <= 2048) return hyper_rows_s<T, YT, 2>(a, n, st);
    if (a.ld <= 4096) return hyper_rows_s<T, YT, 4>(a, n, st);
    if (a.ld <= 16384) return hyper_rows_s<T, YT, 16>(a, n, st);
    return set_error(PGK_ERR_UNSUPPORTED, "hyper_rows: width %d beyond 16384", a.W);
}
pgk_status hyper_rows(const HyperArgs& a, int n, pgk_dtype dt, hipStream_t st) {
    if (dt == PGK_F32) return hyper_rows_t<float, float>(a, n, st);
    PGK_REQUIRE(dt == PGK_BF16, "hyper_rows: dtype %d", (int)dt);
    return a.nslabs > 0 ? hyper_rows_t<bf16, float>(a, n, st) : hyper_rows_t<bf16, bf16>(a, n, st);
}

// -------------------------------------------------------------------------------------------- activation
// NT groups of four per thread stay in registers; NT 0: any width, the row is read twice
template <class T, int NT>
__global__ __launch_bounds__(256) void poly_rows_kernel(const T* z, T* out, int W, int ld, const float* act, float eps) {
    __shared__ float red[3][4];
    const T* zr = z + (size_t)blockIdx.x * ld;
    T* o = out + (size_t)blockIdx.x * ld;
    float4 v[NT > 0 ? NT : 1];
    float s2 = 0.f, s4 = 0.f, s6 = 0.f;
    auto add = [&](float x) { const float x2 = x * x, x4 = x2 * x2; s2 += x2; s4 += x4; s6 = fmaf(x4, x2, s6); };
    auto put = [&](int i, const float4& q, const float3& c, float e) {
        if (i + 3 < W) store4<T>(o + i, make_float4(poly_at(c, e, q.x), poly_at(c, e, q.y), poly_at(c, e, q.z), poly_at(c, e, q.w)));
        else store4<T>(o + i, make_float4(i < W ? poly_at(c, e, q.x) : 0.f, i + 1 < W ? poly_at(c, e, q.y) : 0.f, i + 2 < W ? poly_at(c, e, q.z) : 0.f, i + 3 < W ? poly_at(c, e, q.w) : 0.f));
    };
    if constexpr (NT > 0) {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            v[t] = i < ld ? load4<T>(zr + i) : make_float4(0.f, 0.f, 0.f, 0.f);
            add(v[t].x); add(v[t].y); add(v[t].z); add(v[t].w);
        }
    } else {
        for (int i = threadIdx.x; i < W; i += 256) add(to_f(zr[i]));
    }
    s2 = wave_sum(s2); s4 = wave_sum(s4); s6 = wave_sum(s6);
    if ((threadIdx.x & 63) == 0) { red[0][threadIdx.x >> 6] = s2; red[1][threadIdx.x >> 6] = s4; red[2][threadIdx.x >> 6] = s6; }
    __syncthreads();
    auto total = [&](int i) { return (red[i][0] + red[i][1]) + (red[i][2] + red[i][3]); };
    s2 = total(0); s4 = total(1); s6 = total(2);
    const float3 c = poly_coef(act, s2, s4, s6, W, eps);
    const float e = act[3];
    if constexpr (NT > 0) {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < ld) put(i, v[t], c, e);
        }
    } else {
        for (int i = threadIdx.x; i < ld; i += 256) o[i] = from_f<T>(i < W ? poly_at(c, e, to_f(zr[i])) : 0.f);
    }
}
template <class T>
static void poly_rows_t(const T* z, T* out, int n, int W, int ld, const float* act, float eps, hipStream_t st) {
    if (ld % 4 != 0) poly_rows_kernel<T, 0><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
    else if (ld <= 4096) poly_rows_kernel<T, 4><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
    else if (ld <= 8192) poly_rows_kernel<T, 8><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
    else if (ld <= 12288) poly_rows_kernel<T, 12><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
    else if (ld <= 16384) poly_rows_kernel<T, 16><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
    else poly_rows_kernel<T, 0><<<n, 256, 0, st>>>(z, out, W, ld, act, eps);
}
pgk_status poly_rows(const void* z, void* out, int n, int W, int ld, const float* act, float eps, pgk_dtype dt, hipStream_t st) {
    PGK_REQUIRE(z && out && act && n >= 1 && W >= 1 && W <= ld, "poly_rows: %d rows of %d (stride %d)", n, W, ld);
    if (dt == PGK_F32) poly_rows_t((const float*)z, (float*)out, n, W, ld, act, eps, st);
    else if (dt == PGK_BF16) poly_rows_t((const bf16*)z, (bf16*)out, n, W, ld, act, eps, st);
    else return set_error(PGK_ERR_UNSUPPORTED, "poly_rows: dtype %d", (int)dt);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

__global__ __launch_bounds__(256) void soft_cap_kernel(float* x, size_t n, float cap) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) x[i] = soft_cap(x[i], cap);
}
pgk_status soft_cap_rows(float* x, size_t n, float cap, hipStream_t st) {
    PGK_REQUIRE(x && cap > 0.f, "soft_cap: cap %g", (double)cap);
    if (!n) return PGK_OK;
    const size_t blocks = (n + 255) / 256;
    soft_cap_kernel<<<(unsigned)(blocks > 4096 ? 4096 : blocks), 256, 0, st>>>(x, n, cap);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

// -------------------------------------------------------------------------------------------- operators, any width
// streams [n][S][W]: u = sum_a in[a] x_a
__global__ __launch_bounds__(256) void hyper_read_kernel(const float* x, const float* in, float* u, int S, int W) {
    const float* r = x + (size_t)blockIdx.x * S * W;
    for (int i = threadIdx.x; i < W; i += 256) {
        float t = 0.f;
        for (int s = 0; s < S; ++s) t = fmaf(in ? in[s] : 1.0f, r[(size_t)s * W + i], t);
        u[(size_t)blockIdx.x * W + i] = t;
    }
}
// x_b <- sum_a mix[a][b] x_a + out[b] y, in place
template <class T>
__global__ __launch_bounds__(256) void hyper_write_kernel(float* x, const T* y, const float* out, const float* mix, int S, int W) {
    float* r = x + (size_t)blockIdx.x * S * W;
    for (int i = threadIdx.x; i < W; i += 256) {
        float old[HYPER_MAX_STREAMS];
#pragma unroll
        for (int s = 0; s < HYPER_MAX_STREAMS; ++s) old[s] = s < S ? r[(size_t)s * W + i] : 0.f;
        const float v = to_f(y[(size_t)blockIdx.x * W + i]);
        for (int b = 0; b < S; ++b) {
            float t = out[b] * v;
#pragma unroll
            for (int s = 0; s < HYPER_MAX_STREAMS; ++s) if (s < S) t = fmaf(mix[s * S + b], old[s], t);
            r[(size_t)b * W + i] = t;
        }
    }
}
// a workgroup per (row, group)
template <class T>
__global__ __launch_bounds__(256) void group_norm_kernel(const float* x, const float* w, T* out, int cols, int groups, float eps) {
    __shared__ float red[16];
    const int gs = cols / groups;
    const size_t at = (size_t)blockIdx.x * gs;
    const float* wg = w + (blockIdx.x % groups) * gs;
    float ss = 0.f;
    for (int i = threadIdx.x; i < gs; i += 256) ss = fmaf(x[at + i], x[at + i], ss);
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / gs + eps);
    for (int i = threadIdx.x; i < gs; i += 256) out[at + i] = from_f<T>(x[at + i] * inv * wg[i]);
}
template <class T, int KIND>      // 0: gelu, 1: soft cap
__global__ __launch_bounds__(256) void unary_kernel(const T* x, T* y, size_t n, float p) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) y[i] = from_f<T>(KIND == 0 ? gelu_erf(to_f(x[i])) : soft_cap(to_f(x[i]), p));
}
static unsigned unary_grid(size_t n) { const size_t b = (n + 255) / 256; return (unsigned)(b > 8192 ? 8192 : b); }

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_hyper_read(const float* x, const float* in, float* u, int n, int streams, int width, pgk_stream s) {
    PGK_REQUIRE(x && u && n >= 0 && streams >= 1 && width >= 1, "pgk_hyper_read: %d rows of %d x %d", n, streams, width);
    if (!n) return PGK_OK;
    hyper_read_kernel<<<n, 256, 0, resolve_stream(s)>>>(x, in, u, streams, width);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_hyper_write(float* x, const void* y, const float* out, const float* mix, int n, int streams, int width, pgk_dtype y_dt, pgk_stream s) {
    PGK_REQUIRE(x && y && out && mix && n >= 0 && streams >= 1 && streams <= HYPER_MAX_STREAMS && width >= 1, "pgk_hyper_write: %d rows of %d x %d", n, streams, width);
    if (!n) return PGK_OK;
    PGK_DISPATCH_FLOAT(y_dt, "pgk_hyper_write", (hyper_write_kernel<T><<<n, 256, 0, resolve_stream(s)>>>(x, (const T*)y, out, mix, streams, width)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_group_norm_f32(const float* x, const float* weight, void* out, int rows, int cols, int groups, float eps, pgk_dtype out_dt, pgk_stream s) {
    PGK_REQUIRE(x && weight && out && rows >= 0 && cols >= 1 && groups >= 1 && cols % groups == 0, "pgk_group_norm_f32: %d x %d in %d groups", rows, cols, groups);
    if (!rows) return PGK_OK;
    PGK_DISPATCH_FLOAT(out_dt, "pgk_group_norm_f32", (group_norm_kernel<T><<<rows * groups, 256, 0, resolve_stream(s)>>>(x, weight, (T*)out, cols, groups, eps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_poly_norm(const void* z, void* out, int rows, int cols, const float* act, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(z && out && act && rows >= 0 && cols >= 1, "pgk_poly_norm: %d x %d", rows, cols);
    return rows ? poly_rows(z, out, rows, cols, cols, act, eps, dt, resolve_stream(s)) : PGK_OK;
}

pgk_status pgk_gelu_erf(const void* x, void* y, size_t n, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && y, "pgk_gelu_erf: null pointer");
    if (!n) return PGK_OK;
    PGK_DISPATCH_FLOAT(dt, "pgk_gelu_erf", (unary_kernel<T, 0><<<unary_grid(n), 256, 0, resolve_stream(s)>>>((const T*)x, (T*)y, n, 0.f)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_soft_cap(const void* x, void* y, size_t n, float cap, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && y && cap > 0.f, "pgk_soft_cap: cap %g", (double)cap);
    if (!n) return PGK_OK;
    PGK_DISPATCH_FLOAT(dt, "pgk_soft_cap", (unary_kernel<T, 1><<<unary_grid(n), 256, 0, resolve_stream(s)>>>((const T*)x, (T*)y, n, cap)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

}  // extern "C"
