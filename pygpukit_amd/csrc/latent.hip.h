// Shared by ops_latent.hip (operators) and engine_stack.hip (engine): fp32-stream norms and sliding-window attention.
#pragma once

#include "gemv_core.hip.h"
#include "pgk_device.hip.h"
#include "pgk_internal.h"

namespace pgk {

template <class T> __device__ __forceinline__ float4 load4(const T* p);
template <> __device__ __forceinline__ float4 load4<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <> __device__ __forceinline__ float4 load4<bf16>(const bf16* p) {
    const uint2 g = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(g.x << 16), __uint_as_float(g.x & 0xFFFF0000u), __uint_as_float(g.y << 16), __uint_as_float(g.y & 0xFFFF0000u));
}
template <class T> __device__ __forceinline__ void store4(T* p, const float4& v);
template <> __device__ __forceinline__ void store4<float>(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
template <> __device__ __forceinline__ void store4<bf16>(bf16* p, const float4& v) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
}

// One sandwich step on rows of the fp32 stream h [*][ld] (columns W..ld are zero padding):
//   y given:    h += mult * y / rms(y) * g_post       (y rows in the engine's element type, row stride ldy; store_h: write h back)
//   out given:  out[i] = h / rms(h) * gamma           (rows of stride ld in the engine's element type; gamma null: out[i] = h)
// Workgroup i works on row rows[i] (null: row i) and writes out row i.  The norm weights are fp32, offsets already applied.
struct RowsNormArgs {
    float* h;
    const void* y;
    int ldy;
    const float* g_post;
    float mult;
    const float* gamma;
    void* out;
    int W, ld;
    float eps;
    const int32_t* rows;
    int store_h;
    int nslabs;               // > 0: y is fp32 split-K slabs, slab i at y + i * slab_stride (elements); the sublayer output is their sum
    long long slab_stride;
    // plain: the sublayer output is added as it is, h = (base or h) + mult * (y + sum of e_top rows of e); y and e may be null
    int plain, layer_norm;    // layer_norm: gamma's norm subtracts the mean
    const float* base;        // [ld] or null
    const void* e;            // [*][e_top][ld], element type
    int e_top;
    const void* embed;        // given: no norm, out rows (2 ld wide) are [h | embed[tok[row]]] (table rows of W)
    const int32_t* tok;
};
pgk_status rows_norm(const RowsNormArgs& a, int n, pgk_dtype dt, hipStream_t st);

struct WindowStrides { long long qh, qs, kh, ks, vh, vs, oh, os; };   // elements: per head, per row
// Output gate: the result is multiplied by sigmoid(p[row * gs + head * gh + column * gc]).  One value per head: gh 1, gc 0; one per
// element: gh the head stride, gc 1.  p null: none.
struct OutGate { const void* p; long long gs; int gh, gc; };
// out[i] = gate * softmax over keys i' with 0 <= i - i' < window (queries are the last q_len of kv_len positions) of
// scale * q . k - slopes[head] * (i - i')   (slopes fp32, or null)
pgk_status window_attention(const void* q, const void* k, const void* v, void* out, int hq, int hkv, int q_len, int kv_len, int dk, int dv, float scale,
                            int window, const WindowStrides& sd, const OutGate& gate, const float* slopes, pgk_dtype dt, hipStream_t st);
pgk_status flash_window(const void* q, const void* k, const void* v, void* out, int hq, int hkv, int q_len, int kv_len, int d, float scale,
                        int window, const OutGate& gate, const float* slopes, long long qh, long long qs, long long kh, long long ks, long long oh,
                        long long os, hipStream_t st);   // ops_flash.hip

// ops_attention.hip: kv_len <= 128, head width 128, plain causal mask, bf16
pgk_status attn_short_gated(const void* q, const void* k, const void* v, void* out, int hq, int hkv, int q_len, int kv_len, float scale, const WindowStrides& sd,
                            const void* gate, long long gs, hipStream_t st);

}  // namespace pgk
