// Short causal convolution with SiLU over projection rows (prompts; decode steps convolve inside the recurrences, conv_step in
// mixers.hip.h), RMS norm in equal parts of a row, column slices.

#include <type_traits>
#include <vector>

#include "mixers.hip.h"

namespace pgk {

__device__ __forceinline__ float4 fma4(const float4& w, const float4& u, float4 y) {
    y.x = fmaf(w.x, u.x, y.x); y.y = fmaf(w.y, u.y, y.y); y.z = fmaf(w.z, u.z, y.z); y.w = fmaf(w.w, u.w, y.w);
    return y;
}
template <bool EXACT> __device__ __forceinline__ float4 silu4(const float4& y) {
    return make_float4(silu_f<EXACT>(y.x), silu_f<EXACT>(y.y), silu_f<EXACT>(y.z), silu_f<EXACT>(y.w));
}

// Up to four taps: a thread walks `span` rows of four channels; weights and the three rows above stay in registers, RB rows travel at a
// time.  At a portion's first row (and the thread's) the rows above come from the rows above or the slot's ring.
constexpr int CS_MT = 4, CS_RB = 4;
template <class T>
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvSiluArgs a, int span) {
    constexpr bool EXACT = std::is_same<T, float>::value;
    const int c = 4 * (blockIdx.x * 256 + threadIdx.x);
    if (c >= a.channels) return;
    const int begin = blockIdx.y * span, end = min(begin + span, a.n), taps = a.taps;
    const T *in = reinterpret_cast<const T*>(a.in) + c, *conv = reinterpret_cast<const T*>(a.conv) + c, *ring = reinterpret_cast<const T*>(a.ring) + c;
    T* out = reinterpret_cast<T*>(a.out) + c;
    const float4 zero = {0.f, 0.f, 0.f, 0.f}, bias = a.bias ? *reinterpret_cast<const float4*>(a.bias + c) : zero;
    float4 w[CS_MT], h[CS_MT - 1], next[CS_RB];                    // h[k]: the row k + 1 above
#pragma unroll
    for (int m = 0; m < CS_RB; ++m) next[m] = load4<T>(in + (size_t)min(begin + m, end - 1) * a.ld_in);
#pragma unroll
    for (int k = 0; k < CS_MT; ++k) w[k] = k < taps ? load4<T>(conv + (size_t)(taps - 1 - k) * a.channels) : zero;
    for (int r0 = begin; r0 < end; r0 += CS_RB) {
        float4 u[CS_RB];
        RowSrc src[CS_RB];
#pragma unroll
        for (int m = 0; m < CS_RB; ++m) { u[m] = next[m]; src[m] = a.rows[min(r0 + m, end - 1)]; }
#pragma unroll
        for (int m = 0; m < CS_RB; ++m) next[m] = load4<T>(in + (size_t)min(r0 + CS_RB + m, end - 1) * a.ld_in);
#pragma unroll
        for (int m = 0; m < CS_RB; ++m) {
            const int r = r0 + m;
            if (r >= end) break;
            if (r == begin || r == src[m].first) {
#pragma unroll
                for (int k = 0; k < CS_MT - 1; ++k) {
                    const int p = src[m].pos - 1 - k;
                    h[k] = zero;
                    if (p >= 0 && k + 1 < taps)
                        h[k] = r - 1 - k >= src[m].first ? load4<T>(in + (size_t)(r - 1 - k) * a.ld_in) : load4<T>(ring + ((size_t)src[m].slot * taps + p % taps) * a.channels);
                }
            }
            float4 y = fma4(w[0], u[m], bias);
#pragma unroll
            for (int k = 0; k < CS_MT - 1; ++k) y = fma4(w[k + 1], h[k], y);
            store4<T>(out + (size_t)r * a.ld_out, silu4<EXACT>(y));
            h[2] = h[1]; h[1] = h[0]; h[0] = u[m];
        }
    }
}

// any number of taps
template <class T>
__global__ __launch_bounds__(256) void conv_silu_any_kernel(ConvSiluArgs a) {
    constexpr bool EXACT = std::is_same<T, float>::value;
    const int c = 4 * (blockIdx.x * 256 + threadIdx.x), r = blockIdx.y;
    if (c >= a.channels) return;
    const T *in = reinterpret_cast<const T*>(a.in) + c, *conv = reinterpret_cast<const T*>(a.conv) + c, *ring = reinterpret_cast<const T*>(a.ring) + c;
    const RowSrc s = a.rows[r];
    float4 y = a.bias ? *reinterpret_cast<const float4*>(a.bias + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    for (int b = 0; b < a.taps && s.pos - b >= 0; ++b)
        y = fma4(load4<T>(conv + (size_t)(a.taps - 1 - b) * a.channels),
                 r - b >= s.first ? load4<T>(in + (size_t)(r - b) * a.ld_in) : load4<T>(ring + ((size_t)s.slot * a.taps + (s.pos - b) % a.taps) * a.channels), y);
    store4<T>(reinterpret_cast<T*>(a.out) + c + (size_t)r * a.ld_out, silu4<EXACT>(y));
}

template <class T>
static pgk_status conv_silu_t(const ConvSiluArgs& a, hipStream_t st) {
    const int cols = ceil_div(a.channels, 1024);
    if (a.taps <= CS_MT) {
        const int span = a.n >= 2048 ? 16 : a.n >= 256 ? 8 : 4;
        conv_silu_kernel<T><<<dim3(cols, ceil_div(a.n, span)), 256, 0, st>>>(a, span);
    } else {
        PGK_REQUIRE(a.n <= 65535, "conv_silu_rows: %d rows of %d taps", a.n, a.taps);
        conv_silu_any_kernel<T><<<dim3(cols, a.n), 256, 0, st>>>(a);
    }
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}
pgk_status conv_silu_rows(const ConvSiluArgs& a, pgk_dtype dt, hipStream_t st) {
    PGK_REQUIRE(a.n >= 1 && a.taps >= 1 && a.channels >= 4 && a.channels % 4 == 0 && a.ld_in % 4 == 0 && a.ld_out % 4 == 0 && a.rows && a.ring && a.conv,
                "conv_silu_rows: %d rows of %d channels, %d taps", a.n, a.channels, a.taps);
    return dt == PGK_F32 ? conv_silu_t<float>(a, st) : conv_silu_t<bf16>(a, st);
}

// -------------------------------------------------------------------------------------------- norm in parts
// grid (rows, parts); the true elements of a row count through its heads, `vdim` columns apart
template <class T>
__global__ __launch_bounds__(256) void parts_norm_kernel(unsigned long long* tl, T* x, int ld, int vdim, int vdim_true, int len, const float* norm, float eps) {
    const TLStamp tls(tl);
    __shared__ float red[16];
    T* row = x + (size_t)blockIdx.x * ld;
    const int i0 = blockIdx.y * len;
    constexpr int K = 4;                                           // elements a thread keeps; longer parts read them again
    float v[K];
    auto at = [&](int i) { return vdim == vdim_true ? i : i / vdim_true * vdim + i % vdim_true; };
    float ss = 0.f;
    for (int i = threadIdx.x, k = 0; i < len; i += 256, ++k) {
        const float t = to_f(row[at(i0 + i)]);
        if (k < K) v[k] = t;
        ss = fmaf(t, t, ss);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / len + eps);
    for (int i = threadIdx.x, k = 0; i < len; i += 256, ++k) {
        const int c = at(i0 + i);
        row[c] = from_f<T>((k < K ? v[k] : to_f(row[c])) * inv * norm[c]);
    }
    tls.end();
}
pgk_status parts_norm(void* x, int ld, int n, int heads, int vdim, int vdim_true, int parts, const float* norm, float eps, pgk_dtype dt, hipStream_t st) {
    PGK_REQUIRE(n >= 1 && parts >= 1 && (heads * vdim_true) % parts == 0 && ld >= heads * vdim, "parts_norm: %d x %d in %d parts", heads, vdim_true, parts);
    const int len = heads * vdim_true / parts;
    if (dt == PGK_F32) PGK_CHECK_HIP(launch_k(&parts_norm_kernel<float>, dim3(n, parts), dim3(256), 0, st, (float*)x, ld, vdim, vdim_true, len, norm, eps));
    else PGK_CHECK_HIP(launch_k(&parts_norm_kernel<bf16>, dim3(n, parts), dim3(256), 0, st, (bf16*)x, ld, vdim, vdim_true, len, norm, eps));
    return PGK_OK;
}

template <class E>
__global__ __launch_bounds__(256) void rows_slice_kernel(const E* in, int ld, int cols, E* out, size_t total) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t r = i / cols;
        out[i] = in[r * ld + i % cols];
    }
}
pgk_status rows_slice(const void* in, int ld_in, int off, int cols, void* out, int n, pgk_dtype dt, hipStream_t st) {
    const int pack = dt == PGK_F32 ? 4 : 8;                        // 16-byte pieces
    PGK_REQUIRE(ld_in % pack == 0 && off % pack == 0 && cols % pack == 0 && aligned16(in) && aligned16(out), "rows_slice: columns %d + %d of %d", off, cols, ld_in);
    const size_t total = (size_t)n * (cols / pack), blocks = (total + 255) / 256;
    rows_slice_kernel<uint4><<<(int)(blocks > 4096 ? 4096 : blocks), 256, 0, st>>>((const uint4*)in + off / pack, ld_in / pack, cols / pack, (uint4*)out, total);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_conv_silu(const void* u, const void* past, const void* w, const float* bias, void* out, int n, int channels, int taps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(u && w && out && n >= 1 && taps >= 1, "pgk_conv_silu: %d rows of %d channels, %d taps", n, channels, taps);
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_conv_silu: dtype %d (bf16 or f32)", (int)dt);
    hipStream_t st = resolve_stream(s);
    // the past as ring rows of positions 1 .. taps - 1, the rows are positions taps, taps + 1, ...
    const size_t E = dtype_size(dt), row = (size_t)channels * E, o_rows = ((size_t)taps * row + 255) & ~(size_t)255;
    const bool goes_on = past && taps > 1;
    std::vector<RowSrc> src(n);
    for (int i = 0; i < n; ++i) src[i] = RowSrc{(goes_on ? taps : 0) + i, 0, 0};
    char* ws = nullptr;
    if (pgk_status r = pgk_malloc((void**)&ws, o_rows + n * sizeof(RowSrc))) return r;
    hipError_t e = hipSuccess;
    if (goes_on) e = hipMemcpyAsync(ws + row, past, (taps - 1) * row, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_rows, src.data(), n * sizeof(RowSrc), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    const pgk_status r = e != hipSuccess ? set_error(PGK_ERR_HIP, "pgk_conv_silu: %s", hipGetErrorString(e))
                                         : conv_silu_rows(ConvSiluArgs{u, channels, w, bias, taps, channels, n, ws, (const RowSrc*)(ws + o_rows), out, channels}, dt, st);
    pgk_free(ws);       // stream-ordered reuse
    return r;
}

}  // extern "C"
