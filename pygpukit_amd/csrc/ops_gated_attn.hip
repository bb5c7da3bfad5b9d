// Short convolution + norms over projection rows, and single-query attention over a K/V ring with a distance bias per head, grouped
// heads and an elementwise output gate (mixers.hip.h); the prompt form of the attention is window_attention (ops_latent.hip).

#include <type_traits>

#include "mixers.hip.h"

namespace pgk {

constexpr float GA_LOG2E = 1.4426950408889634f;

// -------------------------------------------------------------------------------------------- short convolution, norms
// Where the channels c .. c + 3 (all of q, of k or of v) of one row go: normalised values to q_out, or to the scratch row and the cache.
template <class T, class QT>
__device__ __forceinline__ void conv_store(const ConvArgs& a, int row, int pos, int slot, int c, float4 y, float inv) {
    if (c < a.n_q) {
        const float s = a.q_norm ? inv * a.q_mult : a.q_mult;
        const float4 g = a.q_norm ? *reinterpret_cast<const float4*>(a.q_norm + c) : make_float4(1.f, 1.f, 1.f, 1.f);
        y.x *= s * g.x; y.y *= s * g.y; y.z *= s * g.z; y.w *= s * g.w;
        store4<QT>(reinterpret_cast<QT*>(a.q_out) + (size_t)row * a.ld_q + c, y);
        return;
    }
    const bool is_k = c < a.n_q + a.n_kv;
    const int kc = c - a.n_q - (is_k ? 0 : a.n_kv);
    if (is_k && a.k_norm) {
        const float4 g = *reinterpret_cast<const float4*>(a.k_norm + kc);
        y.x *= inv * g.x; y.y *= inv * g.y; y.z *= inv * g.z; y.w *= inv * g.w;
    }
    if (a.place) {
        const RowPlace p = a.place[row];
        store4<T>(reinterpret_cast<T*>(a.kv_rows) + (size_t)p.kv * a.ld_kv + (is_k ? 0 : a.n_kv) + kc, y);
        if (!p.store) return;
    }
    store4<T>(reinterpret_cast<T*>(a.cache) + ((((size_t)slot * 2 + (is_k ? 0 : 1)) * (a.n_kv / a.D) + kc / a.D) * a.R + pos % a.R) * a.D + kc % a.D, y);
}

// blockIdx.y: 0 works on q, 1 on k and v.  Per-row scale of the part's norm from per-thread sums of squares
__device__ __forceinline__ void conv_part(const ConvArgs& a, int& c0, int& c1) {
    c0 = blockIdx.y ? a.n_q : 0;
    c1 = blockIdx.y ? a.n_q + 2 * a.n_kv : a.n_q;
}
template <int RB>
__device__ __forceinline__ void conv_scales(const ConvArgs& a, float (&ss)[RB], float (&red)[16][RB], float (&inv)[RB]) {
#pragma unroll
    for (int i = 0; i < RB; ++i) {
        const float t = wave_sum(ss[i]);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6][i] = t;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < RB; ++i) {
        float t = 0.f;
        for (int w = 0; w < (int)(blockDim.x >> 6); ++w) t += red[w][i];
        inv[i] = 1.0f / sqrtf(t / (blockIdx.y ? a.k_true : a.q_true) + a.eps);
    }
}

__device__ __forceinline__ RowSrc conv_row(const ConvArgs& a, int r) {
    return a.rows ? a.rows[r] : RowSrc{max(a.positions[r], 0), r, r};
}

// four elements as they come from memory
template <class T> struct Raw4;
template <> struct Raw4<float> {
    float4 v;
    __device__ __forceinline__ void load(const float* p) { v = *reinterpret_cast<const float4*>(p); }
    __device__ __forceinline__ float4 get() const { return v; }
};
template <> struct Raw4<bf16> {
    uint2 v;
    __device__ __forceinline__ void load(const bf16* p) { v = *reinterpret_cast<const uint2*>(p); }
    __device__ __forceinline__ float4 get() const {
        return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xFFFF0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xFFFF0000u));
    }
};

// Up to four taps.  A workgroup walks `span` rows, RB at a time, QPT groups of four channels per thread: the taps' weights and the last
// three rows stay in registers, the next RB rows travel while these are normalised and stored.  At a portion's first row (and the
// workgroup's) the rows above come from the slot's ring or the rows above.
constexpr int CONV_MT = 4;
template <class T, class IT, class QT, int RB, int QPT>
__global__ __launch_bounds__(1024) void conv_rows_kernel(unsigned long long* tl, ConvArgs a, int span) {
    const TLStamp tls(tl);
    __shared__ float red[2][16][RB];
    const int taps = a.taps, nc = a.n_q + 2 * a.n_kv, nt = blockDim.x, begin = blockIdx.x * span, end = min(begin + span, a.n);
    int c0, c1;
    conv_part(a, c0, c1);
    const int normed = blockIdx.y ? a.n_q + a.n_kv : a.n_q;
    const T* conv = reinterpret_cast<const T*>(a.conv);
    const IT* in = reinterpret_cast<const IT*>(a.in);
    T* ring = reinterpret_cast<T*>(a.tap_ring);
    const float4 zero = {0.f, 0.f, 0.f, 0.f};
    int c[QPT], cc[QPT];
    float4 b[QPT], w[QPT][CONV_MT], h[QPT][CONV_MT - 1];          // h[k]: the row k + 1 above
    Raw4<IT> next[QPT][RB];
#pragma unroll
    for (int q = 0; q < QPT; ++q) {
        c[q] = c0 + 4 * (threadIdx.x + q * nt);
        cc[q] = min(c[q], c1 - 4);
#pragma unroll
        for (int m = 0; m < RB; ++m) next[q][m].load(in + (size_t)min(begin + m, end - 1) * a.ld_in + cc[q]);
        b[q] = a.bias ? *reinterpret_cast<const float4*>(a.bias + cc[q]) : zero;
#pragma unroll
        for (int k = 0; k < CONV_MT; ++k)
            w[q][k] = k >= taps ? zero : conv ? load4<T>(conv + (size_t)(taps - 1 - k) * nc + cc[q]) : make_float4(1.f, 1.f, 1.f, 1.f);
    }
    auto add = [](float4 u, const float4& v) { u.x += v.x; u.y += v.y; u.z += v.z; u.w += v.w; return u; };
    auto fma4 = [](const float4& x, const float4& u, float4 acc) {
        acc.x = fmaf(x.x, u.x, acc.x); acc.y = fmaf(x.y, u.y, acc.y); acc.z = fmaf(x.z, u.z, acc.z); acc.w = fmaf(x.w, u.w, acc.w);
        return acc;
    };
    for (int r0 = begin, pass = 0; r0 < end; r0 += RB, pass ^= 1) {
        Raw4<IT> raw[QPT][RB];
        RowSrc src[RB];
        float4 y[QPT][RB];
        float ss[RB], inv[RB];
#pragma unroll
        for (int m = 0; m < RB; ++m) { src[m] = conv_row(a, min(r0 + m, end - 1)); ss[m] = 0.f; }
#pragma unroll
        for (int q = 0; q < QPT; ++q)
#pragma unroll
            for (int m = 0; m < RB; ++m) raw[q][m] = next[q][m];
        if (r0 + RB < end) {
#pragma unroll
            for (int q = 0; q < QPT; ++q)
#pragma unroll
                for (int m = 0; m < RB; ++m) next[q][m].load(in + (size_t)min(r0 + RB + m, end - 1) * a.ld_in + cc[q]);
        }
#pragma unroll
        for (int m = 0; m < RB; ++m) {
            const int r = min(r0 + m, end - 1);
            if (r == begin || r == src[m].first) {                 // workgroup-uniform
#pragma unroll
                for (int k = 0; k < CONV_MT - 1; ++k) {
                    const int p = src[m].pos - 1 - k;
                    const bool live = p >= 0 && k + 1 < taps;      // before the sequence's start: zero, bias included
#pragma unroll
                    for (int q = 0; q < QPT; ++q) {
                        h[q][k] = zero;
                        if (live) h[q][k] = add(b[q], r - 1 - k >= src[m].first ? load4<IT>(in + (size_t)(r - 1 - k) * a.ld_in + cc[q])
                                                                                : load4<T>(ring + ((size_t)src[m].slot * taps + p % taps) * nc + cc[q]));
                    }
                }
            }
#pragma unroll
            for (int q = 0; q < QPT; ++q) {
                const float4 u = add(raw[q][m].get(), b[q]);
                float4 t = fma4(w[q][0], u, zero);
#pragma unroll
                for (int k = 0; k < CONV_MT - 1; ++k) t = fma4(w[q][k + 1], h[q][k], t);
                y[q][m] = t;
#pragma unroll
                for (int k = CONV_MT - 2; k > 0; --k) h[q][k] = h[q][k - 1];
                h[q][0] = u;
                ss[m] += c[q] < normed ? t.x * t.x + t.y * t.y + t.z * t.z + t.w * t.w : 0.f;
            }
        }
        conv_scales<RB>(a, ss, red[pass], inv);                    // (one barrier: the other half of `red` is the next pass's)
#pragma unroll
        for (int q = 0; q < QPT; ++q) {
            if (c[q] >= c1) break;
#pragma unroll
            for (int m = 0; m < RB; ++m) {
                if (r0 + m >= end) break;
                conv_store<T, QT>(a, r0 + m, src[m].pos, src[m].slot, c[q], y[q][m], inv[m]);
                if (!a.rows && a.conv) store4<T>(ring + ((size_t)src[m].slot * taps + src[m].pos % taps) * nc + c[q], raw[q][m].get());
            }
        }
    }
    tls.end();
}

// Any number of taps and channels, one row per workgroup: the taps are computed twice (sums of squares, then results)
template <class T, class IT, class QT>
__global__ __launch_bounds__(256) void conv_rows_any_kernel(unsigned long long* tl, ConvArgs a) {
    const TLStamp tls(tl);
    __shared__ float red[16][1];
    const int taps = a.taps, nc = a.n_q + 2 * a.n_kv, r = blockIdx.x;
    int c0, c1;
    conv_part(a, c0, c1);
    const T* conv = reinterpret_cast<const T*>(a.conv);
    const IT* in = reinterpret_cast<const IT*>(a.in);
    T* ring = reinterpret_cast<T*>(a.tap_ring);
    const RowSrc s = conv_row(a, r);
    auto conv4 = [&](int c) -> float4 {
        const float4 b = a.bias ? *reinterpret_cast<const float4*>(a.bias + c) : make_float4(0.f, 0.f, 0.f, 0.f);
        float4 y = {0.f, 0.f, 0.f, 0.f};
        for (int back = 0; back < taps && s.pos - back >= 0; ++back) {
            const float4 w = conv ? load4<T>(conv + (size_t)(taps - 1 - back) * nc + c) : make_float4(1.f, 1.f, 1.f, 1.f);
            const float4 u = r - back >= s.first ? load4<IT>(in + (size_t)(r - back) * a.ld_in + c) : load4<T>(ring + ((size_t)s.slot * taps + (s.pos - back) % taps) * nc + c);
            y.x = fmaf(w.x, u.x + b.x, y.x); y.y = fmaf(w.y, u.y + b.y, y.y); y.z = fmaf(w.z, u.z + b.z, y.z); y.w = fmaf(w.w, u.w + b.w, y.w);
        }
        return y;
    };
    float ss[1] = {0.f}, inv[1];
    for (int c = c0 + 4 * threadIdx.x; c < (blockIdx.y ? a.n_q + a.n_kv : a.n_q); c += 1024) {
        const float4 y = conv4(c);
        ss[0] += y.x * y.x + y.y * y.y + y.z * y.z + y.w * y.w;
    }
    conv_scales<1>(a, ss, red, inv);
    for (int c = c0 + 4 * threadIdx.x; c < c1; c += 1024) {
        conv_store<T, QT>(a, r, s.pos, s.slot, c, conv4(c), inv[0]);
        // (the row written is read by no tap of this step, and its channels by this thread only)
        if (!a.rows && a.conv) store4<T>(ring + ((size_t)s.slot * taps + s.pos % taps) * nc + c, load4<IT>(in + (size_t)r * a.ld_in + c));
    }
    tls.end();
}

template <class T, class IT, class QT, bool PROMPT>
static hipError_t conv_rows_launch(const ConvArgs& a, hipStream_t st) {
    const int quads = (a.n_q > 2 * a.n_kv ? a.n_q : 2 * a.n_kv) / 4, parts = a.n_kv ? 2 : 1;     // of the longer part
    auto waves = [](int t) { return (t + 63) / 64 * 64; };
    if (a.taps > CONV_MT || quads > 4096 || (PROMPT && quads > 2048)) return launch_k(&conv_rows_any_kernel<T, IT, QT>, dim3(a.n, parts), dim3(256), 0, st, a);
    // prompts: about a workgroup per CU and part, whole batches of rows each
    auto go = [&](auto kfn, int rb, int qpt) {
        const int span = PROMPT ? ceil_div(ceil_div(a.n, 256), rb) * rb : 1;
        return launch_k(kfn, dim3(ceil_div(a.n, span), parts), dim3(waves((quads + qpt - 1) / qpt)), 0, st, a, span);
    };
    if constexpr (PROMPT) {
        if (a.n <= 512) return quads <= 1024 ? go(&conv_rows_kernel<T, IT, QT, 1, 1>, 1, 1) : go(&conv_rows_kernel<T, IT, QT, 1, 2>, 1, 2);
        return quads <= 1024 ? go(&conv_rows_kernel<T, IT, QT, 4, 1>, 4, 1) : go(&conv_rows_kernel<T, IT, QT, 2, 2>, 2, 2);
    } else {
        if (quads <= 1024) return go(&conv_rows_kernel<T, IT, QT, 1, 1>, 1, 1);
        if (quads <= 2048) return go(&conv_rows_kernel<T, IT, QT, 1, 2>, 1, 2);
        return go(&conv_rows_kernel<T, IT, QT, 1, 4>, 1, 4);
    }
}

pgk_status conv_rows(const ConvArgs& a, pgk_dtype dt, bool in32, bool q32, hipStream_t st) {
    PGK_REQUIRE(a.n >= 1 && a.n_q % 4 == 0 && a.n_kv % 4 == 0 && a.D % 4 == 0 && (a.n_kv == 0 || a.n_kv % a.D == 0) && a.ld_in % 4 == 0 && a.ld_q % 4 == 0 && a.taps >= 1,
                "conv_rows: %d rows of %d + 2 x %d channels, heads of %d, %d taps", a.n, a.n_q, a.n_kv, a.D, a.taps);
    if (a.rows) {                                                  // prompt: rows and q in the element type
        if (dt == PGK_F32) PGK_CHECK_HIP((conv_rows_launch<float, float, float, true>(a, st)));
        else PGK_CHECK_HIP((conv_rows_launch<bf16, bf16, bf16, true>(a, st)));
        return PGK_OK;
    }
    if (dt == PGK_F32) PGK_CHECK_HIP((conv_rows_launch<float, float, float, false>(a, st)));
    else if (in32) PGK_CHECK_HIP((q32 ? conv_rows_launch<bf16, float, float, false>(a, st) : conv_rows_launch<bf16, float, bf16, false>(a, st)));
    else PGK_CHECK_HIP((q32 ? conv_rows_launch<bf16, bf16, float, false>(a, st) : conv_rows_launch<bf16, bf16, bf16, false>(a, st)));
    return PGK_OK;
}

template <class T>
__global__ __launch_bounds__(256) void conv_save_kernel(const T* in, int ld_in, const SeqSpan* seqs, T* ring, int taps, int channels) {
    const SeqSpan s = seqs[blockIdx.x];
    const int p = s.start + s.len - 1 - (int)blockIdx.y;
    if (p < s.start) return;
    const T* src = in + (size_t)(s.row0 + p - s.start) * ld_in;
    T* dst = ring + ((size_t)s.slot * taps + p % taps) * channels;
    for (int c = 4 * threadIdx.x; c < channels; c += 1024) store4<T>(dst + c, load4<T>(src + c));
}
pgk_status conv_save(const void* in, int ld_in, const SeqSpan* seqs, int n_seqs, void* tap_ring, int taps, int channels, pgk_dtype dt, hipStream_t st) {
    const dim3 grid(n_seqs, taps);
    if (dt == PGK_F32) conv_save_kernel<float><<<grid, 256, 0, st>>>((const float*)in, ld_in, seqs, (float*)tap_ring, taps, channels);
    else conv_save_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)in, ld_in, seqs, (bf16*)tap_ring, taps, channels);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

template <class T>
__global__ __launch_bounds__(256) void kv_gather_kernel(const RowPlace* place, const T* cache, T* rows, int ld, int n_kv, int D, int R) {
    const RowPlace p = place[blockIdx.x];
    for (int c = 4 * threadIdx.x; c < 2 * n_kv; c += 1024) {
        const int half = c >= n_kv ? 1 : 0, kc = c - half * n_kv;
        store4<T>(rows + (size_t)p.kv * ld + c, load4<T>(cache + ((((size_t)p.slot * 2 + half) * (n_kv / D) + kc / D) * R + p.pos % R) * D + kc % D));
    }
}
pgk_status kv_gather(const RowPlace* place, int n, const void* cache, void* kv_rows, int ld_kv, int n_kv, int D, int R, pgk_dtype dt, hipStream_t st) {
    if (!n) return PGK_OK;
    if (dt == PGK_F32) kv_gather_kernel<float><<<n, 256, 0, st>>>(place, (const float*)cache, (float*)kv_rows, ld_kv, n_kv, D, R);
    else kv_gather_kernel<bf16><<<n, 256, 0, st>>>(place, (const bf16*)cache, (bf16*)kv_rows, ld_kv, n_kv, D, R);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

// -------------------------------------------------------------------------------------------- single-query attention
template <class IT> __device__ __forceinline__ float gate_at(const KvAttnArgs& a, int b, int col) {
    return a.gate ? 1.0f / (1.0f + expf(-to_f(reinterpret_cast<const IT*>(a.gate)[(size_t)b * a.ld_gate + col]))) : 1.0f;
}

// bf16, D <= 64 RT: up to 16 query heads of one key head x 64 keys per step on the matrix pipe.  S[head][key] = q K^T (each wave 16
// keys), O[head][d] += P V (each wave its share of the columns; V^T comes out of the row-major image through ds_read_b64_tr_b16, whose
// k order is 16 (j >> 2) + 4 (lane >> 4) + (j & 3), and P is read back from LDS in that order).
typedef __bf16 bf16x8_ga __attribute__((ext_vector_type(8)));
typedef float f32x4_ga __attribute__((ext_vector_type(4)));
typedef short v4s_ga __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4_ga mfma16_ga(const uint4& a, const uint4& b, f32x4_ga c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_ga, a), __builtin_bit_cast(bf16x8_ga, b), c, 0, 0, 0);
}
constexpr int GA_PAD = 8;           // elements added to an LDS row: rows start 4 banks apart
static size_t kv_mfma_lds(int D) { return (size_t)(64 + 64 + 16) * (D + GA_PAD) * 2; }

template <class IT, int RT>
__global__ __launch_bounds__(256) void kv_attn_mfma_kernel(unsigned long long* tl, KvAttnArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) char ga_smem[];
    __shared__ __attribute__((aligned(16))) bf16 ps[16][72];
    __shared__ float red[4][16];
    const int D = a.D, ld = D + GA_PAD, nch = D / 8;
    bf16* ks = reinterpret_cast<bf16*>(ga_smem);                  // [64][ld]
    bf16* vs = ks + 64 * ld;                                      // [64][ld]
    bf16* qs = vs + 64 * ld;                                      // [16][ld]
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4;
    const int rep = a.H / a.G, nhb = (rep + 15) / 16;
    const int s = blockIdx.x, g = blockIdx.y / nhb, hb = blockIdx.y % nhb, b = blockIdx.z;
    const int h0 = g * rep + hb * 16, nh = min(16, rep - hb * 16);
    int n, lo, k0, k1;
    ring_window(max(a.positions[b], 0), a.window, a.R, n, lo);
    split_range(n, a.nsplit, s, k0, k1);
    if (k0 >= k1) {                                                // an empty split: its record says so, the sums are never read
        if (tid < nh) {
            float* ml = a.pml + (((size_t)b * a.H + h0 + tid) * a.nsplit + s) * 2;
            ml[0] = -INFINITY; ml[1] = 0.f;
        }
        tls.end();
        return;
    }
    float m_run[4], l_run[4], slope[4];
    f32x4_ga o[RT];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        m_run[i] = -INFINITY; l_run[i] = 0.f;
        slope[i] = a.slopes ? a.slopes[min(h0 + 4 * q4 + i, a.H - 1)] * GA_LOG2E : 0.f;
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) o[t] = f32x4_ga{0.f, 0.f, 0.f, 0.f};
    const bf16* kb = reinterpret_cast<const bf16*>(a.cache) + (((size_t)b * 2) * a.G + g) * a.R * D;
    const bf16* vb = kb + (size_t)a.G * a.R * D;
    const bf16* qb = reinterpret_cast<const bf16*>(a.q) + (size_t)b * a.H * D;
    // 16-byte pieces: LPR lanes per row (a power of two), lanes past a row's end repeat its last piece
    constexpr int LPR = 8 * RT, RPP = 256 / LPR, QN = RPP >= 16 ? 1 : 16 / RPP, CN = 64 / RPP;
    const int r_in = tid / LPR, col = min(tid % LPR, nch - 1) * 8;
    u32x4 qv[QN], kv[CN], vv[CN];
    auto fetch = [&](int kt) {
#pragma unroll
        for (int i = 0; i < CN; ++i) {
            const size_t off = (size_t)ring_row(lo, min(kt + i * RPP + r_in, k1 - 1), a.R) * D + col;
            kv[i] = *reinterpret_cast<const u32x4*>(kb + off);
            vv[i] = *reinterpret_cast<const u32x4*>(vb + off);
        }
    };
#pragma unroll
    for (int i = 0; i < QN; ++i) qv[i] = *reinterpret_cast<const u32x4*>(qb + (size_t)(h0 + min(i * RPP + r_in, nh - 1)) * D + col);
    fetch(k0);
#pragma unroll
    for (int i = 0; i < QN; ++i) *reinterpret_cast<u32x4*>(qs + min(i * RPP + r_in, 15) * ld + col) = qv[i];     // (rows past nh - 1 repeat the last head)
    for (int kt = k0; kt < k1; kt += 64) {
        const int rt = k1 - kt > 32 ? 64 : 32;                    // rows of this tile that take part (the rest repeat the last key)
        if (kt != k0) __syncthreads();                            // the last step's reads of the images are done
#pragma unroll
        for (int i = 0; i < CN; ++i) {
            *reinterpret_cast<u32x4*>(ks + (i * RPP + r_in) * ld + col) = kv[i];
            *reinterpret_cast<u32x4*>(vs + (i * RPP + r_in) * ld + col) = vv[i];
        }
        __syncthreads();
        fetch(kt + 64);                                           // the next tile travels under this one's products
        f32x4_ga sc = {-INFINITY, -INFINITY, -INFINITY, -INFINITY};
        const bool mine = 16 * wid < rt;                          // wave-uniform
        if (mine) {
            f32x4_ga t = {0.f, 0.f, 0.f, 0.f};
            const bf16* qr = qs + l15 * ld + 8 * q4;
            const bf16* kr = ks + (16 * wid + l15) * ld + 8 * q4;
            for (int c = 0; c < D; c += 32) t = mfma16_ga(*reinterpret_cast<const uint4*>(qr + c), *reinterpret_cast<const uint4*>(kr + c), t);
            const int key = kt + 16 * wid + l15;
            const float dist = (float)(n - 1 - key);
            if (key < k1) {                                       // lane: heads 4 q4 + i, key 16 wid + l15
#pragma unroll
                for (int i = 0; i < 4; ++i) sc[i] = fmaf(-slope[i], dist, t[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float t = group16_max(sc[i]);
            if (l15 == 0) red[wid][4 * q4 + i] = t;
        }
        __syncthreads();
        float al[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int hh = 4 * q4 + i;
            const float mn = fmaxf(m_run[i], fmaxf(fmaxf(red[0][hh], red[1][hh]), fmaxf(red[2][hh], red[3][hh])));   // finite: kt < k1
            al[i] = __builtin_amdgcn_exp2f(m_run[i] - mn);
            m_run[i] = mn;
            const float p = __builtin_amdgcn_exp2f(sc[i] - mn);
            l_run[i] = l_run[i] * al[i] + p;
            if (mine) ps[hh][16 * wid + l15] = from_f<bf16>(p);
        }
        __syncthreads();
#pragma unroll
        for (int t = 0; t < RT; ++t)
#pragma unroll
            for (int i = 0; i < 4; ++i) o[t][i] *= al[i];
        for (int c = 0; c < rt; c += 32) {
            const uint2 p0 = *reinterpret_cast<const uint2*>(&ps[l15][c + 4 * q4]), p1 = *reinterpret_cast<const uint2*>(&ps[l15][c + 16 + 4 * q4]);
            const uint4 pf = make_uint4(p0.x, p0.y, p1.x, p1.y);
            const bf16* row = vs + (c + 4 * q4 + (l15 >> 2)) * ld + 4 * (l15 & 3);
#pragma unroll
            for (int t = 0; t < RT; ++t) {
                const int dc = 16 * (wid + 4 * t);
                if (dc < D) {                                     // wave-uniform
                    const v4s_ga c0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_ga*)(row + dc));
                    const v4s_ga c1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_ga*)(row + 16 * ld + dc));
                    const uint2 u0 = __builtin_bit_cast(uint2, c0), u1 = __builtin_bit_cast(uint2, c1);
                    o[t] = mfma16_ga(pf, make_uint4(u0.x, u0.y, u1.x, u1.y), o[t]);
                }
            }
        }
    }
    // lane: heads 4 q4 + i, column l15 of each 16-column tile; the row sums are spread over the 16 lanes of a group and the waves
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float t = group16_sum(l_run[i]);
        if (l15 == 0) red[wid][4 * q4 + i] = t;
    }
    // (red was last read before the barrier that precedes the products)
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int hh = 4 * q4 + i;
        if (hh >= nh) continue;
        const float l = red[0][hh] + red[1][hh] + red[2][hh] + red[3][hh];
        const size_t rec = ((size_t)b * a.H + h0 + hh) * a.nsplit + s;
#pragma unroll
        for (int t = 0; t < RT; ++t) {
            const int dc = 16 * (wid + 4 * t) + l15, oc = (h0 + hh) * D + dc;
            if (dc >= D) continue;
            if (a.nsplit > 1) a.po[rec * D + dc] = o[t][i];
            else reinterpret_cast<IT*>(a.out)[(size_t)b * a.ld_out + oc] = from_f<IT>(o[t][i] / l * gate_at<IT>(a, b, oc));
        }
        if (a.nsplit > 1 && wid == 0 && l15 == 0) {
            a.pml[2 * rec] = m_run[i];
            a.pml[2 * rec + 1] = l;
        }
    }
    tls.end();
}

// Any element type, D <= 64 RC: HB query heads of one key head per workgroup, a wave walks every fourth key, 64 columns apart per lane.
template <class T, class IT, int RC, int HB>
__global__ __launch_bounds__(256) void kv_attn_kernel(unsigned long long* tl, KvAttnArgs a) {
    const TLStamp tls(tl);
    __shared__ float sm[4][HB][2];
    extern __shared__ float so[];                                  // [HB][D]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, D = a.D, rep = a.H / a.G, nhb = (rep + HB - 1) / HB;
    const int s = blockIdx.x, g = blockIdx.y / nhb, hb = blockIdx.y % nhb, b = blockIdx.z, h0 = g * rep + hb * HB, nh = min(HB, rep - hb * HB);
    int n, lo, k0, k1;
    ring_window(max(a.positions[b], 0), a.window, a.R, n, lo);
    split_range(n, a.nsplit, s, k0, k1);
    float q[HB][RC], o[HB][RC], m[HB], l[HB], slope[HB];
#pragma unroll
    for (int i = 0; i < HB; ++i) {
        const int h = h0 + min(i, nh - 1);
        m[i] = -INFINITY; l[i] = 0.f;
        slope[i] = a.slopes ? a.slopes[h] * GA_LOG2E : 0.f;
        const float* qp = reinterpret_cast<const float*>(a.q) + ((size_t)b * a.H + h) * D;
#pragma unroll
        for (int j = 0; j < RC; ++j) { const int d = 64 * j + lane; q[i][j] = d < D ? qp[d] : 0.f; o[i][j] = 0.f; }
    }
    const T* kb = reinterpret_cast<const T*>(a.cache) + (((size_t)b * 2) * a.G + g) * a.R * D;
    const T* vb = kb + (size_t)a.G * a.R * D;
    for (int k = k0 + wid; k < k1; k += 4) {
        const size_t off = (size_t)ring_row(lo, k, a.R) * D;
        float c[RC], v[RC];
#pragma unroll
        for (int j = 0; j < RC; ++j) {
            const int d = 64 * j + lane;
            c[j] = d < D ? to_f(kb[off + d]) : 0.f;
            v[j] = d < D ? to_f(vb[off + d]) : 0.f;
        }
        const float dist = (float)(n - 1 - k);
#pragma unroll
        for (int i = 0; i < HB; ++i) {
            float t = 0.f;
#pragma unroll
            for (int j = 0; j < RC; ++j) t = fmaf(q[i][j], c[j], t);
            t = fmaf(-slope[i], dist, wave_sum(t));
            const float mn = fmaxf(m[i], t), al = exp2f(m[i] - mn), p = exp2f(t - mn);
            m[i] = mn;
            l[i] = fmaf(l[i], al, p);
#pragma unroll
            for (int j = 0; j < RC; ++j) o[i][j] = fmaf(o[i][j], al, p * v[j]);
        }
    }
    if (lane == 0) {
#pragma unroll
        for (int i = 0; i < HB; ++i) { sm[wid][i][0] = m[i]; sm[wid][i][1] = l[i]; }
    }
    for (int i = threadIdx.x; i < HB * D; i += 256) so[i] = 0.f;
    __syncthreads();
    for (int w = 0; w < 4; ++w) {                                  // waves add their share in turn: a fixed order
        if (wid == w) {
#pragma unroll
            for (int i = 0; i < HB; ++i) {
                const float mm = fmaxf(fmaxf(sm[0][i][0], sm[1][i][0]), fmaxf(sm[2][i][0], sm[3][i][0]));
                const float f = l[i] > 0.f ? exp2f(m[i] - mm) : 0.f;
#pragma unroll
                for (int j = 0; j < RC; ++j) { const int d = 64 * j + lane; if (d < D) so[i * D + d] += f * o[i][j]; }
            }
        }
        __syncthreads();
    }
    auto total = [&](int i, float& mm) {
        float ll = 0.f;
        mm = -INFINITY;
        for (int w = 0; w < 4; ++w) mm = fmaxf(mm, sm[w][i][0]);
        for (int w = 0; w < 4; ++w) if (sm[w][i][1] > 0.f) ll += sm[w][i][1] * exp2f(sm[w][i][0] - mm);
        return ll;
    };
    for (int i = threadIdx.x; i < nh * D; i += 256) {
        const int hh = i / D, oc = (h0 + hh) * D + i % D;
        float mm;
        if (a.nsplit > 1) a.po[(((size_t)b * a.H + h0 + hh) * a.nsplit + s) * D + i % D] = so[i];
        else reinterpret_cast<IT*>(a.out)[(size_t)b * a.ld_out + oc] = from_f<IT>(so[i] / total(hh, mm) * gate_at<IT>(a, b, oc));
    }
    if (a.nsplit > 1 && (int)threadIdx.x < nh) {
        float mm, ll = total(threadIdx.x, mm);
        float* ml = a.pml + (((size_t)b * a.H + h0 + threadIdx.x) * a.nsplit + s) * 2;
        ml[0] = mm; ml[1] = ll;
    }
    tls.end();
}

// Combine the split records of (sequence, head) and apply the gate; nsplit <= 64.
template <class IT>
__global__ __launch_bounds__(128) void kv_merge_kernel(unsigned long long* tl, KvAttnArgs a) {
    const TLStamp tls(tl);
    const int h = blockIdx.x, b = blockIdx.y, lane = threadIdx.x & 63;
    __shared__ float sw[64];
    const size_t rec = ((size_t)b * a.H + h) * a.nsplit;
    const float mm = lane < a.nsplit ? a.pml[(rec + lane) * 2] : -INFINITY, ll = lane < a.nsplit ? a.pml[(rec + lane) * 2 + 1] : 0.f;
    const float top = wave_max(ll > 0.f ? mm : -INFINITY), f = ll > 0.f ? exp2f(mm - top) : 0.f;
    float den = wave_sum(f * ll), more = 1.0f;
    if (a.sink) {                                                  // (no value: it only takes its share)
        const float sk = a.sink[h] * GA_LOG2E, t2 = fmaxf(top, sk);
        more = exp2f(top - t2);
        den = fmaf(den, more, exp2f(sk - t2));
    }
    if (threadIdx.x < 64) sw[lane] = f * more / den;
    __syncthreads();
    int n, lo;
    ring_window(max(a.positions[b], 0), a.window, a.R, n, lo, a.chunked);
    const int per = split_rows(n, a.nsplit), used = (n + per - 1) / per;
    for (int c = 2 * threadIdx.x; c < a.D; c += 256) {
        float x = 0.f, y = 0.f;
#pragma unroll 8
        for (int s = 0; s < used; ++s) {
            const float2 p = *reinterpret_cast<const float2*>(a.po + (rec + s) * a.D + c);
            x = fmaf(sw[s], p.x, x);
            y = fmaf(sw[s], p.y, y);
        }
        const int oc = h * a.D + c;
        IT* out = reinterpret_cast<IT*>(a.out) + (size_t)b * a.ld_out + oc;
        out[0] = from_f<IT>(x * gate_at<IT>(a, b, oc));
        out[1] = from_f<IT>(y * gate_at<IT>(a, b, oc + 1));
    }
    tls.end();
}

pgk_status kv_merge(const KvAttnArgs& a, bool io32, hipStream_t st) {
    PGK_REQUIRE(a.D % 64 == 0 && a.nsplit >= 1 && a.nsplit <= 64, "kv_merge: head width %d, %d splits", a.D, a.nsplit);
    if (io32) PGK_CHECK_HIP(launch_k(&kv_merge_kernel<float>, dim3(a.H, a.B), dim3(128), 0, st, a));
    else PGK_CHECK_HIP(launch_k(&kv_merge_kernel<bf16>, dim3(a.H, a.B), dim3(128), 0, st, a));
    return PGK_OK;
}

bool kv_attn_q32(int D, pgk_dtype dt) { return dt == PGK_F32 || D > 256; }

int kv_attn_splits(int B, int H, int G, int keys, int cus) {
    const int groups = B * G * ceil_div(H / G, 16);
    int s = ceil_div(keys, 64);
    const int want = ceil_div(2 * cus, groups);
    if (s > want) s = want;
    return s > 64 ? 64 : (s < 1 ? 1 : s);
}

template <class T, class IT, int RC>
static hipError_t launch_kv_attn(const KvAttnArgs& a, hipStream_t st) {
    constexpr int HB = RC <= 4 ? 4 : 2;
    return launch_k(&kv_attn_kernel<T, IT, RC, HB>, dim3(a.nsplit, a.G * ceil_div(a.H / a.G, HB), a.B), dim3(256), (size_t)HB * a.D * 4, st, a);
}
template <class IT, int RT>
static hipError_t launch_kv_mfma(const KvAttnArgs& a, hipStream_t st) {
    const size_t lds = kv_mfma_lds(a.D);
    auto kfn = &kv_attn_mfma_kernel<IT, RT>;
    static bool done = false;
    if (lds > 48 * 1024 && !done) {
        if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024)) return e;
        done = true;
    }
    return launch_k(kfn, dim3(a.nsplit, a.G * ceil_div(a.H / a.G, 16), a.B), dim3(256), lds, st, a);
}

template <class T, class IT>
static pgk_status kv_attn_t(const KvAttnArgs& a, pgk_dtype dt, hipStream_t st, int* launches) {
    if (kv_attn_q32(a.D, dt)) {
        if (a.D <= 64) PGK_CHECK_HIP((launch_kv_attn<T, IT, 1>(a, st)));
        else if (a.D <= 128) PGK_CHECK_HIP((launch_kv_attn<T, IT, 2>(a, st)));
        else if (a.D <= 256) PGK_CHECK_HIP((launch_kv_attn<T, IT, 4>(a, st)));
        else PGK_CHECK_HIP((launch_kv_attn<T, IT, 16>(a, st)));
    }
    if constexpr (std::is_same<T, bf16>::value) {
        if (!kv_attn_q32(a.D, dt)) {
            if (a.D <= 64) PGK_CHECK_HIP((launch_kv_mfma<IT, 1>(a, st)));
            else if (a.D <= 128) PGK_CHECK_HIP((launch_kv_mfma<IT, 2>(a, st)));
            else PGK_CHECK_HIP((launch_kv_mfma<IT, 4>(a, st)));
        }
    }
    *launches += 1;
    if (a.nsplit > 1) {
        PGK_CHECK_HIP(launch_k(&kv_merge_kernel<IT>, dim3(a.H, a.B), dim3(128), 0, st, a));
        *launches += 1;
    }
    return PGK_OK;
}

pgk_status kv_attn_decode(const KvAttnArgs& a, pgk_dtype dt, bool io32, hipStream_t st, int* launches) {
    PGK_REQUIRE(a.D % 64 == 0 && a.D <= 1024 && a.H % a.G == 0 && a.nsplit >= 1 && a.nsplit <= 64 && a.window >= 1, "kv_attn: head width %d, %d / %d heads, %d splits", a.D, a.H, a.G, a.nsplit);
    if (dt == PGK_F32) return kv_attn_t<float, float>(a, dt, st, launches);
    return io32 ? kv_attn_t<bf16, float>(a, dt, st, launches) : kv_attn_t<bf16, bf16>(a, dt, st, launches);
}

// -------------------------------------------------------------------------------------------- operator form of the convolution
template <class T>
__global__ __launch_bounds__(256) void short_conv_kernel(const T* u, const T* past, const T* w, T* out, int n, int channels, int taps) {
    const size_t total = (size_t)n * channels;
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
        const int r = (int)(i / channels), c = (int)(i % channels);
        float y = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int s = r - (taps - 1) + j;
            const float x = s >= 0 ? to_f(u[(size_t)s * channels + c]) : past ? to_f(past[(size_t)(s + taps - 1) * channels + c]) : 0.f;
            y = fmaf(to_f(w[(size_t)c * taps + j]), x, y);
        }
        out[i] = from_f<T>(y);
    }
}

template <class T>
__global__ __launch_bounds__(256) void sigmoid_mul_kernel(T* x, const T* gate, size_t total) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < total; i += (size_t)gridDim.x * 256)
        x[i] = from_f<T>(to_f(x[i]) / (1.0f + expf(-to_f(gate[i]))));
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_short_conv(const void* u, const void* past, const void* w, void* out, int n, int channels, int taps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(u && w && out && n >= 0 && channels >= 1 && taps >= 1 && u != out, "pgk_short_conv: bad arguments [%d, %d], %d taps", n, channels, taps);
    if (!n) return PGK_OK;
    const long long blocks = ((long long)n * channels + 255) / 256;
    PGK_DISPATCH_FLOAT(dt, "pgk_short_conv", (short_conv_kernel<T><<<(int)(blocks > 8192 ? 8192 : blocks), 256, 0, resolve_stream(s)>>>((const T*)u, (const T*)past, (const T*)w, (T*)out, n, channels, taps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_sigmoid_mul(void* x, const void* gate, size_t n, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && gate, "pgk_sigmoid_mul: null pointer");
    if (!n) return PGK_OK;
    const size_t blocks = (n + 255) / 256;
    PGK_DISPATCH_FLOAT(dt, "pgk_sigmoid_mul", (sigmoid_mul_kernel<T><<<(int)(blocks > 8192 ? 8192 : blocks), 256, 0, resolve_stream(s)>>>((T*)x, (const T*)gate, n)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

}  // extern "C"
