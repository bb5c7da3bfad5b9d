// Operators of the layer-list models (llm/layers/latent_attention.py, engine_stack.hip): RMSNorm of an fp32 stream with fp32 weights,
// normalised residual add, sliding-window attention with separate key / value widths, per-head sigmoid gate, zero padding.

#include "latent.hip.h"

namespace pgk {

// One workgroup per row; see latent.hip.h.  NT float4 per thread keep the row in registers between the two reductions.
template <class T, class YT, int NT>
__global__ __launch_bounds__(256) void rows_norm_kernel(RowsNormArgs a) {
    __shared__ float red[16];
    const int row = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
    float* hr = a.h + (size_t)row * a.ld;
    float4 v[NT];
    const int nt = a.ld;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4;
        v[t] = i < nt ? *reinterpret_cast<const float4*>(hr + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    if (a.y) {
        const YT* yr = reinterpret_cast<const YT*>(a.y) + (size_t)row * a.ldy;
        float4 y[NT];
        float ss = 0.f;
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            y[t] = i < nt ? load4<YT>(yr + i) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
        if constexpr (std::is_same<YT, float>::value) {
            constexpr int SU = NT <= 4 ? 16 / NT : 2;      // slabs in flight: unconditional loads (clamped), masked adds
            for (int s0 = 1; s0 < a.nslabs; s0 += SU) {
                float4 q[SU][NT];
#pragma unroll
                for (int s = 0; s < SU; ++s)
#pragma unroll
                    for (int t = 0; t < NT; ++t)
                        q[s][t] = load4<float>(reinterpret_cast<const float*>(yr) + min(s0 + s, a.nslabs - 1) * a.slab_stride + min((int)(threadIdx.x + 256 * t) * 4, nt - 4));
#pragma unroll
                for (int s = 0; s < SU; ++s) {
                    const float w = s0 + s < a.nslabs ? 1.f : 0.f;
#pragma unroll
                    for (int t = 0; t < NT; ++t) {
                        const float m = (int)(threadIdx.x + 256 * t) * 4 < nt ? w : 0.f;
                        y[t].x = fmaf(m, q[s][t].x, y[t].x); y[t].y = fmaf(m, q[s][t].y, y[t].y);
                        y[t].z = fmaf(m, q[s][t].z, y[t].z); y[t].w = fmaf(m, q[s][t].w, y[t].w);
                    }
                }
            }
        }
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            ss += y[t].x * y[t].x + y[t].y * y[t].y + y[t].z * y[t].z + y[t].w * y[t].w;
        }
        ss = block_sum(ss, red);
        const float inv = a.mult / sqrtf(ss / a.W + a.eps);
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < nt) {
                const float4 g = *reinterpret_cast<const float4*>(a.g_post + i);
                v[t].x = fmaf(y[t].x * inv, g.x, v[t].x); v[t].y = fmaf(y[t].y * inv, g.y, v[t].y);
                v[t].z = fmaf(y[t].z * inv, g.z, v[t].z); v[t].w = fmaf(y[t].w * inv, g.w, v[t].w);
                if (a.store_h) *reinterpret_cast<float4*>(hr + i) = v[t];
            }
        }
    }
    if (!a.out) return;
    if (!a.gamma) {                                     // the sublayer reads the stream itself
        T* o = reinterpret_cast<T*>(a.out) + (size_t)blockIdx.x * a.ld;
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < nt) store4<T>(o + i, v[t]);
        }
        return;
    }
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) ss += v[t].x * v[t].x + v[t].y * v[t].y + v[t].z * v[t].z + v[t].w * v[t].w;
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / a.W + a.eps);
    T* o = reinterpret_cast<T*>(a.out) + (size_t)blockIdx.x * a.ld;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4;
        if (i < nt) {
            const float4 g = *reinterpret_cast<const float4*>(a.gamma + i);
            store4<T>(o + i, make_float4(v[t].x * inv * g.x, v[t].y * inv * g.y, v[t].z * inv * g.z, v[t].w * inv * g.w));
        }
    }
}

// The plain form: y (or its slabs) and the experts' rows are added, then layer norm or RMS norm, or the row beside its embedding
template <class T, class YT, int NT>
__global__ __launch_bounds__(256) void rows_add_kernel(RowsNormArgs a) {
    __shared__ float red[16];
    const int row = a.rows ? a.rows[blockIdx.x] : blockIdx.x, nt = a.ld;
    float* hr = a.h + (size_t)row * a.ld;
    const float* from = a.base ? a.base : hr;
    const YT* yr = reinterpret_cast<const YT*>(a.y) + (size_t)row * a.ldy;
    const T* er = reinterpret_cast<const T*>(a.e) + (size_t)row * a.e_top * a.ld;
    float4 v[NT];
    float s1 = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = min((int)(threadIdx.x + 256 * t) * 4, nt - 4);
        float4 x = *reinterpret_cast<const float4*>(from + i), y = {0.f, 0.f, 0.f, 0.f};
        auto add = [&](const float4& q) { y.x += q.x; y.y += q.y; y.z += q.z; y.w += q.w; };
        if (a.y) add(load4<YT>(yr + i));
#pragma unroll 4
        for (int s = 1; s < a.nslabs; ++s) add(load4<YT>(yr + s * a.slab_stride + i));
        if (a.e) {
#pragma unroll 4
            for (int k = 0; k < a.e_top; ++k) add(load4<T>(er + (size_t)k * a.ld + i));
        }
        x.x = fmaf(a.mult, y.x, x.x); x.y = fmaf(a.mult, y.y, x.y); x.z = fmaf(a.mult, y.z, x.z); x.w = fmaf(a.mult, y.w, x.w);
        const bool in = (int)(threadIdx.x + 256 * t) * 4 < nt;
        if (in && a.store_h) *reinterpret_cast<float4*>(hr + i) = x;
        v[t] = in ? x : make_float4(0.f, 0.f, 0.f, 0.f);
        s1 += v[t].x + v[t].y + v[t].z + v[t].w;                   // (columns W .. ld are zero)
    }
    if (!a.out) return;
    if (a.embed) {
        const T* er0 = reinterpret_cast<const T*>(a.embed) + (size_t)a.tok[row] * a.W;
        T* o = reinterpret_cast<T*>(a.out) + (size_t)blockIdx.x * 2 * a.ld;
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < nt) store4<T>(o + i, v[t]);
        }
        for (int i = threadIdx.x; i < nt; i += 256) o[nt + i] = i < a.W ? er0[i] : from_f<T>(0.f);
        return;
    }
    const float mean = a.layer_norm ? block_sum(s1, red) / a.W : 0.f;
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4;
        v[t].x -= mean; v[t].y -= mean; v[t].z -= mean; v[t].w -= mean;
        ss += (i < a.W ? v[t].x * v[t].x : 0.f) + (i + 1 < a.W ? v[t].y * v[t].y : 0.f) + (i + 2 < a.W ? v[t].z * v[t].z : 0.f) + (i + 3 < a.W ? v[t].w * v[t].w : 0.f);
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps);
    T* o = reinterpret_cast<T*>(a.out) + (size_t)blockIdx.x * a.ld;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        const int i = (threadIdx.x + 256 * t) * 4;
        if (i < nt) {
            const float4 g = *reinterpret_cast<const float4*>(a.gamma + i);      // zero in columns W .. ld
            store4<T>(o + i, make_float4(v[t].x * inv * g.x, v[t].y * inv * g.y, v[t].z * inv * g.z, v[t].w * inv * g.w));
        }
    }
}

template <class T, class YT>
static pgk_status rows_add_t(const RowsNormArgs& a, int n, hipStream_t st) {
    PGK_REQUIRE(a.ld % 4 == 0 && a.W <= a.ld && (!a.out || a.embed || a.gamma) && !(a.e && a.e_top < 1), "rows_norm: row stride %d / width %d", a.ld, a.W);
    if (a.ld <= 1024) rows_add_kernel<T, YT, 1><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 2048) rows_add_kernel<T, YT, 2><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 4096) rows_add_kernel<T, YT, 4><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 16384) rows_add_kernel<T, YT, 16><<<n, 256, 0, st>>>(a);
    else return set_error(PGK_ERR_UNSUPPORTED, "rows_norm: width %d beyond 16384", a.W);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

template <class T, class YT>
static pgk_status rows_norm_t(const RowsNormArgs& a, int n, hipStream_t st) {
    PGK_REQUIRE(a.ld % 4 == 0 && a.W <= a.ld, "rows_norm: row stride %d / width %d", a.ld, a.W);
    if (a.ld <= 1024) rows_norm_kernel<T, YT, 1><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 2048) rows_norm_kernel<T, YT, 2><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 4096) rows_norm_kernel<T, YT, 4><<<n, 256, 0, st>>>(a);
    else if (a.ld <= 16384) rows_norm_kernel<T, YT, 16><<<n, 256, 0, st>>>(a);
    else return set_error(PGK_ERR_UNSUPPORTED, "rows_norm: width %d beyond 16384", a.W);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status rows_norm(const RowsNormArgs& a, int n, pgk_dtype dt, hipStream_t st) {
    if (a.plain) {
        if (dt == PGK_BF16) return a.nslabs > 0 ? rows_add_t<bf16, float>(a, n, st) : rows_add_t<bf16, bf16>(a, n, st);
        if (dt == PGK_F32) return rows_add_t<float, float>(a, n, st);
    }
    if (dt == PGK_BF16) return a.nslabs > 0 ? rows_norm_t<bf16, float>(a, n, st) : rows_norm_t<bf16, bf16>(a, n, st);
    if (dt == PGK_F32) return rows_norm_t<float, float>(a, n, st);
    return set_error(PGK_ERR_UNSUPPORTED, "rows_norm: dtype %d", (int)dt);
}

// ---- any width (not a multiple of 4, any row stride): the operator form of the same two steps ----
template <class T>
__global__ __launch_bounds__(256) void rmsnorm_f32_kernel(const float* x, const float* w, T* out, int cols, float eps) {
    __shared__ float red[16];
    const float* xr = x + (size_t)blockIdx.x * cols;
    float ss = 0.f;
    for (int i = threadIdx.x; i < cols; i += 256) ss = fmaf(xr[i], xr[i], ss);
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / cols + eps);
    for (int i = threadIdx.x; i < cols; i += 256) out[(size_t)blockIdx.x * cols + i] = from_f<T>(xr[i] * inv * w[i]);
}
template <class T>
__global__ __launch_bounds__(256) void rmsnorm_add_kernel(float* x, const T* y, const float* w, int cols, float eps, float mult) {
    __shared__ float red[16];
    const T* yr = y + (size_t)blockIdx.x * cols;
    float* xr = x + (size_t)blockIdx.x * cols;
    float ss = 0.f;
    for (int i = threadIdx.x; i < cols; i += 256) { const float v = to_f(yr[i]); ss = fmaf(v, v, ss); }
    ss = block_sum(ss, red);
    const float inv = mult / sqrtf(ss / cols + eps);
    for (int i = threadIdx.x; i < cols; i += 256) xr[i] = fmaf(to_f(yr[i]) * inv, w[i], xr[i]);
}

template <class T>
__global__ __launch_bounds__(256) void head_gate_kernel(T* x, const T* gate, size_t total, int heads, int d, long long gs) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t rh = i / d;
        const float g = to_f(gate[(long long)(rh / heads) * gs + (long long)(rh % heads)]);
        x[i] = from_f<T>(to_f(x[i]) / (1.0f + expf(-g)));
    }
}

template <class T>
__global__ __launch_bounds__(256) void xielu_kernel(const T* x, T* y, size_t n, float a, float b) {
    constexpr int N = Vec<T>::N;
    const size_t stride = (size_t)gridDim.x * 256, i0 = blockIdx.x * (size_t)256 + threadIdx.x;
    for (size_t i = i0; i < n / N; i += stride) {
        Vec<T> v;
        v.load(x + i * N);
        float f[N];
        v.to_float(f);
#pragma unroll
        for (int j = 0; j < N; ++j) f[j] = xielu<std::is_same<T, float>::value>(f[j], a, b);
        v.from_float(f);
        v.store(y + i * N);
    }
    for (size_t i = n / N * N + i0; i < n; i += stride) y[i] = from_f<T>(xielu<std::is_same<T, float>::value>(to_f(x[i]), a, b));
}

template <class E>
__global__ __launch_bounds__(256) void pad_2d_kernel(const E* src, E* dst, int rows, int cols, int dcols, size_t total) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const size_t r = i / dcols, c = i % dcols;
        dst[i] = r < (size_t)rows && c < (size_t)cols ? src[r * cols + c] : E(0);
    }
}

// Sliding-window attention for any widths and for fp32: one workgroup per (query row, head), each wave takes every fourth block of
// 64 keys (a lane per key for the scores, a lane per value column for the sum), the four partial softmaxes meet in LDS.
template <class T>
__global__ __launch_bounds__(256) void window_attn_simple_kernel(const T* q, const T* k, const T* v, T* out, int rep, int q_len, int kv_len, int dk, int dv,
                                                                 float scale, int window, WindowStrides sd, OutGate gate, const float* slopes) {
    extern __shared__ float wsm[];
    const int row = blockIdx.x, head = blockIdx.y, kvh = head / rep, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    float* qs = wsm;                          // [dk]
    float* acc = wsm + dk + wid * dv;         // [4][dv]
    float* ps = wsm + dk + 4 * dv + wid * 64; // [4][64]
    float* ml = wsm + dk + 4 * dv + 4 * 64;   // [4][2]
    const T* qr = q + head * sd.qh + row * sd.qs;
    for (int i = threadIdx.x; i < dk; i += 256) qs[i] = to_f(qr[i]);
    for (int i = lane; i < dv; i += 64) acc[i] = 0.f;
    __syncthreads();
    const int qpos = kv_len - q_len + row, lo = max(0, qpos - window + 1);
    const T* kh = k + kvh * sd.kh;
    const T* vh = v + kvh * sd.vh;
    float m = -INFINITY, l = 0.f;
    const float slope = slopes ? slopes[head] : 0.f;
    for (int k0 = lo + 64 * wid; k0 <= qpos; k0 += 256) {          // wave-uniform
        const int key = k0 + lane, kn = min(64, qpos + 1 - k0);
        float s = 0.f;
        const T* kr = kh + (long long)min(key, qpos) * sd.ks;
        for (int d = 0; d < dk; ++d) s = fmaf(qs[d], to_f(kr[d]), s);
        s = lane < kn ? fmaf(s, scale, -slope * (float)(qpos - key)) : -INFINITY;
        const float mn = fmaxf(m, wave_max(s)), alpha = expf(m - mn), p = expf(s - mn);      // mn is finite: kn >= 1
        m = mn;
        l = l * alpha + wave_sum(p);
        ps[lane] = p;
        __builtin_amdgcn_wave_barrier();
        for (int c = lane; c < dv; c += 64) {
            float t = acc[c] * alpha;
            const T* vc = vh + (long long)k0 * sd.vs + c;
            for (int j = 0; j < kn; ++j) t = fmaf(ps[j], to_f(vc[(long long)j * sd.vs]), t);
            acc[c] = t;
        }
        __builtin_amdgcn_wave_barrier();
    }
    if (lane == 0) { ml[2 * wid] = m; ml[2 * wid + 1] = l; }
    __syncthreads();
    float mm = -INFINITY, den = 0.f, w[4];
    for (int i = 0; i < 4; ++i) mm = fmaxf(mm, ml[2 * i]);
    for (int i = 0; i < 4; ++i) { w[i] = ml[2 * i + 1] > 0.f ? expf(ml[2 * i] - mm) : 0.f; den += w[i] * ml[2 * i + 1]; }
    const float f = 1.f / den;
    const float* a0 = wsm + dk;
    T* o = out + head * sd.oh + row * sd.os;
    const T* g = reinterpret_cast<const T*>(gate.p);
    for (int c = threadIdx.x; c < dv; c += 256) {
        const float y = (w[0] * a0[c] + w[1] * a0[dv + c] + w[2] * a0[2 * dv + c] + w[3] * a0[3 * dv + c]) * f;
        o[c] = from_f<T>(g ? y / (1.0f + expf(-to_f(g[(long long)row * gate.gs + head * gate.gh + c * gate.gc]))) : y);
    }
}

pgk_status window_attention(const void* q, const void* k, const void* v, void* out, int hq, int hkv, int q_len, int kv_len, int dk, int dv, float scale,
                            int window, const WindowStrides& sd, const OutGate& gate, const float* slopes, pgk_dtype dt, hipStream_t st) {
    const bool flash = dt == PGK_BF16 && dk == dv && (dk == 64 || dk == 128) && scale > 0.f && sd.kh == sd.vh && sd.ks == sd.vs && aligned16(q) && aligned16(k) && aligned16(v) &&
                       sd.qs % 8 == 0 && sd.qh % 8 == 0 && sd.ks % 8 == 0 && sd.kh % 8 == 0 && (reinterpret_cast<uintptr_t>(out) & 7u) == 0 && sd.os % 4 == 0 && sd.oh % 4 == 0 &&
                       (!gate.gc || (gate.gc == 1 && gate.gs % 4 == 0 && gate.gh % 4 == 0 && (reinterpret_cast<uintptr_t>(gate.p) & 7u) == 0));
    // the whole context in one tile and inside every query's window
    if (flash && dk == 128 && kv_len <= 128 && window >= kv_len && !slopes && !gate.gc && (!gate.p || gate.gh == 1)) return attn_short_gated(q, k, v, out, hq, hkv, q_len, kv_len, scale, sd, gate.p, gate.gs, st);
    if (flash) return flash_window(q, k, v, out, hq, hkv, q_len, kv_len, dk, scale, window, gate, slopes, sd.qh, sd.qs, sd.kh, sd.ks, sd.oh, sd.os, st);
    const size_t lds = ((size_t)dk + 4 * (size_t)dv + 4 * 64 + 8) * 4;
    PGK_REQUIRE(lds <= 64 * 1024, "window_attention: head widths %d / %d do not fit LDS", dk, dv);
    dim3 grid(q_len, hq);
    PGK_DISPATCH_FLOAT(dt, "window_attention", (window_attn_simple_kernel<T><<<grid, 256, lds, st>>>((const T*)q, (const T*)k, (const T*)v, (T*)out, hq / hkv, q_len, kv_len, dk, dv,
                                                                                                     scale, window, sd, gate, slopes)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

}  // namespace pgk

using namespace pgk;

// One wave per row: layer norm, latent rows, rotation of query columns
template <class T>
__global__ __launch_bounds__(256) void layernorm_f32_kernel(const float* x, const float* w, T* out, int rows, int cols, float eps) {
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (row >= rows) return;
    const float* r = x + (size_t)row * cols;
    float s = 0.f, ss = 0.f;
    for (int i = lane; i < cols; i += 64) s += r[i];
    const float mean = wave_sum(s) / cols;
    for (int i = lane; i < cols; i += 64) ss = fmaf(r[i] - mean, r[i] - mean, ss);
    const float inv = 1.0f / sqrtf(wave_sum(ss) / cols + eps);
    for (int i = lane; i < cols; i += 64) out[(size_t)row * cols + i] = from_f<T>((r[i] - mean) * inv * w[i]);
}
template <class T>
__device__ __forceinline__ void turn_pair(const T* src, T* dst, float angle) {
    float s, c;
    sincosf(angle, &s, &c);
    const float u = to_f(src[0]), v = to_f(src[1]);
    dst[0] = from_f<T>(fmaf(u, c, -v * s));
    dst[1] = from_f<T>(fmaf(v, c, u * s));
}
template <class T>
__global__ __launch_bounds__(256) void latent_cache_rows_kernel(const T* x, const float* norm, const float* freq, T* out, int n, int rank, int rot, int first, float eps) {
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (row >= n) return;
    const T* r = x + (size_t)row * (rank + rot);
    T* o = out + (size_t)row * (rank + rot);
    float ss = 0.f;
    for (int i = lane; i < rank; i += 64) { const float v = to_f(r[i]); ss = fmaf(v, v, ss); }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / rank + eps);
    for (int i = lane; i < rank; i += 64) o[i] = from_f<T>(to_f(r[i]) * inv * norm[i]);
    for (int i = lane; i < rot / 2; i += 64) turn_pair<T>(r + rank + 2 * i, o + rank + 2 * i, (float)(first + row) * freq[i]);
}
template <class T>
__global__ __launch_bounds__(256) void rotate_pairs_kernel(T* x, const float* freq, int total, int heads, int dim, int rot, int first) {
    const int i = blockIdx.x * 256 + threadIdx.x, pairs = rot / 2;
    if (i >= total) return;
    T* p = x + (size_t)(i / pairs) * dim + dim - rot + 2 * (i % pairs);
    turn_pair<T>(p, p, (float)(first + i / pairs / heads) * freq[i % pairs]);
}

extern "C" {

pgk_status pgk_layernorm_f32(const float* x, const float* weight, void* out, int rows, int cols, float eps, pgk_dtype out_dt, pgk_stream s) {
    PGK_REQUIRE(x && weight && out && rows >= 0 && cols >= 1, "pgk_layernorm_f32: %d x %d", rows, cols);
    if (!rows) return PGK_OK;
    PGK_DISPATCH_FLOAT(out_dt, "pgk_layernorm_f32", (layernorm_f32_kernel<T><<<ceil_div(rows, 4), 256, 0, resolve_stream(s)>>>(x, weight, (T*)out, rows, cols, eps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_latent_rows(const void* x, const float* norm, const float* freq, void* out, int n, int rank, int rot, int first, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && norm && freq && out && n >= 1 && rank >= 1 && rot >= 2 && rot % 2 == 0 && first >= 0, "pgk_latent_rows: %d rows of %d + %d", n, rank, rot);
    PGK_DISPATCH_FLOAT(dt, "pgk_latent_rows", (latent_cache_rows_kernel<T><<<ceil_div(n, 4), 256, 0, resolve_stream(s)>>>((const T*)x, norm, freq, (T*)out, n, rank, rot, first, eps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_rotate_pairs(void* x, const float* freq, int n, int heads, int dim, int rot, int first, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && freq && n >= 1 && heads >= 1 && rot >= 2 && rot % 2 == 0 && rot <= dim && first >= 0 && (long long)n * heads * rot < (1LL << 31), "pgk_rotate_pairs: %d x %d x %d, %d turned", n, heads, dim, rot);
    const int total = n * heads * (rot / 2);
    PGK_DISPATCH_FLOAT(dt, "pgk_rotate_pairs", (rotate_pairs_kernel<T><<<ceil_div(total, 256), 256, 0, resolve_stream(s)>>>((T*)x, freq, total, heads, dim, rot, first)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_rmsnorm_f32(const float* x, const float* weight, void* out, int rows, int cols, float eps, pgk_dtype out_dt, pgk_stream s) {
    PGK_REQUIRE(x && weight && out && rows >= 0 && cols > 0, "pgk_rmsnorm_f32: bad arguments [%d, %d]", rows, cols);
    if (!rows) return PGK_OK;
    PGK_DISPATCH_FLOAT(out_dt, "pgk_rmsnorm_f32", (rmsnorm_f32_kernel<T><<<rows, 256, 0, resolve_stream(s)>>>(x, weight, (T*)out, cols, eps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_rmsnorm_add_f32(float* x, const void* y, const float* weight, int rows, int cols, float eps, float mult, pgk_dtype y_dt, pgk_stream s) {
    PGK_REQUIRE(x && y && weight && rows >= 0 && cols > 0, "pgk_rmsnorm_add_f32: bad arguments [%d, %d]", rows, cols);
    if (!rows) return PGK_OK;
    PGK_DISPATCH_FLOAT(y_dt, "pgk_rmsnorm_add_f32", (rmsnorm_add_kernel<T><<<rows, 256, 0, resolve_stream(s)>>>(x, (const T*)y, weight, cols, eps, mult)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_window_attention(const void* q, const void* k, const void* v, void* out, int hq, int hkv, int q_len, int kv_len, int dk, int dv, float scale,
                                int window, const void* gate, int64_t gate_stride, int gate_elementwise, const float* slopes, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(q && k && v && out, "pgk_window_attention: null pointer");
    PGK_REQUIRE(hq > 0 && hkv > 0 && hq % hkv == 0, "pgk_window_attention: n_heads mismatch (Hq=%d, Hkv=%d)", hq, hkv);
    PGK_REQUIRE(q_len > 0 && kv_len >= q_len && dk > 0 && dv > 0 && window >= 1, "pgk_window_attention: bad shape q_len=%d kv_len=%d dk=%d dv=%d window=%d", q_len, kv_len, dk, dv, window);
    const WindowStrides sd{dk, (long long)hq * dk, dk, (long long)hkv * dk, dv, (long long)hkv * dv, dv, (long long)hq * dv};
    const OutGate og{gate, gate_stride, gate_elementwise ? dv : 1, gate_elementwise ? 1 : 0};
    return window_attention(q, k, v, out, hq, hkv, q_len, kv_len, dk, dv, scale, window, sd, og, slopes, dt, resolve_stream(s));
}

pgk_status pgk_xielu(const void* x, void* y, size_t n, float a, float b, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && y && aligned16(x) && aligned16(y), "pgk_xielu: null or unaligned pointer");
    if (!n) return PGK_OK;
    const size_t blocks = (n / 4 + 255) / 256 + 1;
    PGK_DISPATCH_FLOAT(dt, "pgk_xielu", (xielu_kernel<T><<<(int)(blocks > 8192 ? 8192 : blocks), 256, 0, resolve_stream(s)>>>((const T*)x, (T*)y, n, a, b)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_head_gate(void* x, const void* gate, int rows, int heads, int d, int64_t gate_stride, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && gate && rows >= 0 && heads > 0 && d > 0, "pgk_head_gate: bad arguments");
    const size_t total = (size_t)rows * heads * d;
    if (!total) return PGK_OK;
    const int grid = ceil_div((long long)total, 256) > 4096 ? 4096 : ceil_div((long long)total, 256);
    PGK_DISPATCH_FLOAT(dt, "pgk_head_gate", (head_gate_kernel<T><<<grid, 256, 0, resolve_stream(s)>>>((T*)x, (const T*)gate, total, heads, d, gate_stride)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_pad_2d(const void* src, void* dst, int rows, int cols, int dst_rows, int dst_cols, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(src && dst && rows >= 1 && cols >= 1 && dst_rows >= rows && dst_cols >= 1, "pgk_pad_2d: [%d, %d] into [%d, %d]", rows, cols, dst_rows, dst_cols);
    const size_t total = (size_t)dst_rows * dst_cols;
    const int grid = ceil_div((long long)total, 256) > 8192 ? 8192 : ceil_div((long long)total, 256);
    hipStream_t st = resolve_stream(s);
    if (dtype_size(dt) == 2) pad_2d_kernel<uint16_t><<<grid, 256, 0, st>>>((const uint16_t*)src, (uint16_t*)dst, rows, cols, dst_cols, total);
    else if (dtype_size(dt) == 4) pad_2d_kernel<uint32_t><<<grid, 256, 0, st>>>((const uint32_t*)src, (uint32_t*)dst, rows, cols, dst_cols, total);
    else return set_error(PGK_ERR_UNSUPPORTED, "pgk_pad_2d: dtype %d", (int)dt);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

}  // extern "C"
