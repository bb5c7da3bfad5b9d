// Attention whose heads mix their scores before the softmax, with a sink per head, over a K/V ring or prompt rows (mixers.hip.h), and the
// step before it: bias, norm per head and rotation of projection rows.

#include <type_traits>

#include "mixers.hip.h"

namespace pgk {

constexpr float TK_LOG2E = 1.4426950408889634f;

__device__ __forceinline__ void wave_sync() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// -------------------------------------------------------------------------------------------- bias, norm per head, rotation
// GL lanes per head, NI groups of four columns per lane.  Workgroup (row, y) works on heads y * hpw .. of the row; the angles of the row's
// position are computed once for all of them.
template <class T, class IT, int GL, int NI>
__global__ __launch_bounds__(256) void head_rows_kernel(unsigned long long* tl, HeadRowsArgs a, int hpw) {
    const TLStamp tls(tl);
    constexpr int NG = 256 / GL;
    extern __shared__ __attribute__((aligned(16))) float hr_smem[];
    const int D = a.D, half = a.rot / 2, row = blockIdx.x, total = a.H + 2 * a.G;
    const int lg = threadIdx.x % GL, grp = threadIdx.x / GL;
    float* cs = hr_smem;                                           // [half]
    float* sn = cs + half;                                         // [half]
    float* xb = hr_smem + ((2 * half + 3) & ~3) + grp * D;         // [D] of this head
    const RowSrc src = a.rows ? a.rows[row] : RowSrc{max(a.positions[row], 0), row, row};
    for (int i = threadIdx.x; i < half; i += 256) sincosf((float)src.pos * a.rot_freq[i], &sn[i], &cs[i]);
    __syncthreads();
    const IT* in = reinterpret_cast<const IT*>(a.in) + (size_t)row * a.ld_in;
    const int last = min(total, ((int)blockIdx.y + 1) * hpw);
    for (int u0 = blockIdx.y * hpw; u0 < last; u0 += NG) {         // uniform
        const int u = min(u0 + grp, last - 1);                     // (groups past the end repeat the last head)
        const bool is_q = u < a.H, is_k = !is_q && u < a.H + a.G;
        const float* gamma = is_q ? a.q_norm : is_k ? a.k_norm : nullptr;
        float4 x[NI];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int c = 4 * (lg + GL * i);
            x[i] = c < D ? load4<IT>(in + (size_t)u * D + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            if (a.bias && c < D) {
                const float4 b = *reinterpret_cast<const float4*>(a.bias + (size_t)u * D + c);
                x[i].x += b.x; x[i].y += b.y; x[i].z += b.z; x[i].w += b.w;
            }
            ss += x[i].x * x[i].x + x[i].y * x[i].y + x[i].z * x[i].z + x[i].w * x[i].w;
        }
        ss = group_sum<GL>(ss);
        const float inv = 1.0f / sqrtf(ss / a.dim + a.eps);
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int c = 4 * (lg + GL * i);
            if (c >= D) continue;
            if (gamma) {
                const float4 g = *reinterpret_cast<const float4*>(gamma + c);
                x[i].x *= inv * g.x; x[i].y *= inv * g.y; x[i].z *= inv * g.z; x[i].w *= inv * g.w;
            }
            *reinterpret_cast<float4*>(xb + c) = x[i];
        }
        wave_sync();
        if (is_q || is_k) {
#pragma unroll
            for (int i = 0; i < NI; ++i) {
                float* e = reinterpret_cast<float*>(&x[i]);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int c = 4 * (lg + GL * i) + j;
                    if (c >= a.rot) continue;
                    const bool first = c < half;
                    const int p = first ? c : c - half;
                    const float other = xb[first ? c + half : p];
                    e[j] = first ? fmaf(e[j], cs[p], -other * sn[p]) : fmaf(e[j], cs[p], other * sn[p]);
                }
            }
        }
        wave_sync();                                               // (the buffer is the next head's)
        if (u0 + grp >= last) continue;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int c = 4 * (lg + GL * i);
            if (c >= D) continue;
            if (is_q) { store4<T>(reinterpret_cast<T*>(a.q_out) + (size_t)row * a.ld_q + (size_t)u * D + c, x[i]); continue; }
            const int g = u - a.H - (is_k ? 0 : a.G);
            if (a.place) {
                const RowPlace p = a.place[row];
                store4<T>(reinterpret_cast<T*>(a.kv_rows) + (size_t)p.kv * a.ld_kv + (size_t)((is_k ? 0 : a.G) + g) * D + c, x[i]);
                if (!p.store) continue;
            }
            store4<T>(reinterpret_cast<T*>(a.cache) + ((((size_t)src.slot * 2 + (is_k ? 0 : 1)) * a.G + g) * a.R + src.pos % a.R) * D + c, x[i]);
        }
    }
    tls.end();
}

template <class T, class IT, int GL, int NI>
static hipError_t head_rows_launch(const HeadRowsArgs& a, hipStream_t st) {
    constexpr int NG = 256 / GL;
    const int total = a.H + 2 * a.G, rounds = a.n >= 512 ? ceil_div(total, NG) : 1;      // many rows: a workgroup takes a whole one
    const size_t lds = (size_t)(((a.rot + 3) & ~3) + NG * a.D) * 4;
    return launch_k(&head_rows_kernel<T, IT, GL, NI>, dim3(a.n, ceil_div(total, NG * rounds)), dim3(256), lds, st, a, NG * rounds);
}
template <class T, class IT>
static pgk_status head_rows_t(const HeadRowsArgs& a, hipStream_t st) {
    if (a.D == 64) PGK_CHECK_HIP((head_rows_launch<T, IT, 16, 1>(a, st)));
    else if (a.D == 128) PGK_CHECK_HIP((head_rows_launch<T, IT, 32, 1>(a, st)));
    else if (a.D <= 256) PGK_CHECK_HIP((head_rows_launch<T, IT, 64, 1>(a, st)));
    else PGK_CHECK_HIP((head_rows_launch<T, IT, 64, 4>(a, st)));
    return PGK_OK;
}
pgk_status head_rows(const HeadRowsArgs& a, pgk_dtype dt, bool in32, hipStream_t st) {
    PGK_REQUIRE(a.n >= 1 && a.H >= 1 && a.G >= 0 && a.D % 64 == 0 && a.D <= 1024 && a.dim >= 1 && a.dim <= a.D && a.rot >= 0 && a.rot % 2 == 0 && a.rot <= a.dim && (a.rot == 0 || a.rot_freq) &&
                    a.ld_in % 4 == 0 && a.ld_q % 4 == 0 && a.ld_kv % 4 == 0 && (a.G == 0 || a.R >= 1) && (!a.rows == !a.place || a.G == 0) && (a.rows || a.positions),
                "head_rows: %d rows of %d + 2 x %d heads of %d (%d true), %d turned", a.n, a.H, a.G, a.D, a.dim, a.rot);
    if (dt == PGK_F32) return head_rows_t<float, float>(a, st);
    return in32 ? head_rows_t<bf16, float>(a, st) : head_rows_t<bf16, bf16>(a, st);
}

// -------------------------------------------------------------------------------------------- where a query's keys are
// key t of a row: decode: ring rows of its slot, prompt: rows of the scratch
template <class T> struct KeySpan {
    const T *k, *v;
    long long gs, rs, vgs, vrs;           // elements between two heads, two rows
    int n, lo, R;
    __device__ __forceinline__ KeySpan(const TalkArgs& a, int row) {
        if (a.cache) {
            ring_window(max(a.positions[row], 0), a.window, a.R, n, lo, a.chunked);
            k = reinterpret_cast<const T*>(a.cache) + (size_t)row * 2 * a.G * a.R * a.D;
            v = k + (size_t)a.G * a.R * a.D;
            gs = vgs = (long long)a.R * a.D; rs = vrs = a.D; R = a.R;
        } else {
            const int last = a.kv_len - a.n + row;
            n = min(span_keys(a.pos0 + last, a.window, a.chunked), last + 1);
            lo = last - n + 1;
            k = reinterpret_cast<const T*>(a.k);
            v = reinterpret_cast<const T*>(a.v);
            gs = a.D; rs = a.ld_kv; R = 0x7FFFFFFF;
            vgs = a.Dv ? a.Dv : a.D; vrs = a.Dv ? a.ld_v : a.ld_kv;
        }
    }
    __device__ __forceinline__ int at(int t) const { return ring_row(lo, t, R); }
};

// out = o / (l + exp2(sink - m)): o, l relative to exp2(m)
__device__ __forceinline__ float sink_scale(const float* sink, int h, float m, float l) {
    if (!sink) return 1.0f / l;
    const float sk = sink[h] * TK_LOG2E, t = fmaxf(m, sk), f = exp2f(m - t);
    return f / fmaf(l, f, exp2f(sk - t));
}

// Any element type and widths: a workgroup per (split, row), all heads, 64 keys at a time.  A lane per key for the scores and their mix, a
// thread per (head, column) for the sum.
template <class T, class IT>
__global__ __launch_bounds__(256) void talk_any_kernel(unsigned long long* tl, TalkArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) float tk_smem[];
    const int H = a.H, D = a.D, DV = a.Dv ? a.Dv : D, HD = H * D, HV = H * DV, rep = H / a.G, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, s = blockIdx.x, row = blockIdx.y;
    float* qs = tk_smem;                                           // [H][D]
    float* acc = qs + ((HD + 3) & ~3);                             // [H][DV]
    float* raw = acc + HV;                                         // [H][64]
    float* mixed = raw + H * 64;                                   // [H][64]
    float *m = mixed + H * 64, *l = m + H, *al = l + H;            // [H]
    const KeySpan<T> ks(a, row);
    int k0, k1;
    split_range(ks.n, a.nsplit, s, k0, k1);
    const T* q = reinterpret_cast<const T*>(a.q) + (size_t)row * a.ld_q;
    const float mult = a.scale * TK_LOG2E;
    for (int i = threadIdx.x; i < HD; i += 256) qs[i] = to_f(q[i]);
    for (int i = threadIdx.x; i < HV; i += 256) acc[i] = 0.f;
    for (int i = threadIdx.x; i < H; i += 256) { m[i] = -INFINITY; l[i] = 0.f; }
    __syncthreads();
    for (int kt = k0; kt < k1; kt += 64) {
        const int kn = min(64, k1 - kt);
        const long long off = ks.at(kt + min(lane, kn - 1)) * ks.rs;
        for (int h = wid; h < H; h += 4) {
            const T* kr = ks.k + off + (h / rep) * ks.gs;
            const float* qh = qs + h * D;
            float t = 0.f;
            if (D & 3) for (int d = 0; d < D; ++d) t = fmaf(to_f(kr[d]), qh[d], t);
            else for (int d = 0; d < D; d += 4) {
                const float4 x = load4<T>(kr + d), y = *reinterpret_cast<const float4*>(qh + d);
                t = fmaf(x.x, y.x, t); t = fmaf(x.y, y.y, t); t = fmaf(x.z, y.z, t); t = fmaf(x.w, y.w, t);
            }
            raw[h * 64 + lane] = t * mult;
        }
        __syncthreads();
        for (int h = wid; h < H; h += 4) {
            float t = 0.f;
            if (a.talk) for (int g = 0; g < H; ++g) t = fmaf(a.talk[h * H + g], raw[g * 64 + lane], t);
            else t = raw[h * 64 + lane];
            if (lane >= kn) t = -INFINITY;
            const float mo = m[h], mn = fmaxf(mo, wave_max(t)), f = exp2f(mo - mn), p = exp2f(t - mn);      // mn is finite: kn >= 1
            const float sum = wave_sum(p);
            mixed[h * 64 + lane] = p;
            if (lane == 0) { al[h] = f; m[h] = mn; l[h] = fmaf(l[h], f, sum); }
        }
        __syncthreads();
        for (int i = threadIdx.x; i < HV; i += 256) {
            const int h = i / DV, d = i - h * DV;
            const T* vr = ks.v + (h / rep) * ks.vgs + d;
            float t = acc[i] * al[h];
            for (int j = 0; j < kn; ++j) t = fmaf(mixed[h * 64 + j], to_f(vr[ks.at(kt + j) * ks.vrs]), t);
            acc[i] = t;
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < HV; i += 256) {
        const int h = i / DV;
        if (a.nsplit > 1) a.po[(((size_t)row * H + h) * a.nsplit + s) * D + i - h * D] = acc[i];
        else reinterpret_cast<IT*>(a.out)[(size_t)row * a.ld_out + i] = from_f<IT>(acc[i] * sink_scale(a.sink, h, m[h], l[h]));
    }
    if (a.nsplit > 1)
        for (int h = threadIdx.x; h < H; h += 256) {
            float* ml = a.pml + (((size_t)row * H + h) * a.nsplit + s) * 2;
            ml[0] = m[h]; ml[1] = l[h];
        }
    tls.end();
}

constexpr int TALK_LDS_MAX = 150 * 1024;
template <class T, class IT>
static pgk_status talk_any(const TalkArgs& a, hipStream_t st) {
    const size_t lds = (size_t)(a.H * a.D + 3 + a.H * (a.Dv ? a.Dv : a.D) + 2 * a.H * 64 + 3 * a.H) * 4;
    PGK_REQUIRE(lds <= TALK_LDS_MAX, "talk_attention: %d heads of %d do not fit LDS", a.H, a.D);
    auto kfn = &talk_any_kernel<T, IT>;
    static bool done = false;
    if (lds > 48 * 1024 && !done) {
        PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, TALK_LDS_MAX));
        done = true;
    }
    PGK_CHECK_HIP(launch_k(kfn, dim3(a.nsplit, a.n), dim3(256), lds, st, a));
    return PGK_OK;
}

int talk_splits(int B, int H, int G, int keys, int cus) {
    int s = ceil_div(keys, 32);
    const int want = ceil_div(2 * cus, B);
    if (s > want) s = want;
    return s > 64 ? 64 : (s < 1 ? 1 : s);
}

pgk_status talk_attention(const TalkArgs& a, pgk_dtype dt, bool io32, hipStream_t st, int* launches) {
    PGK_REQUIRE(a.n >= 1 && a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.window >= 1 && a.nsplit >= 1 && a.nsplit <= 64 && ((a.D % 64 == 0 && a.ld_q % 8 == 0) || a.Dv) && (!a.Dv || !a.cache) &&
                    (a.cache ? a.positions && a.R >= 1 && (a.nsplit == 1 || (a.po && a.pml)) : a.k && a.v && a.kv_len >= a.n && a.nsplit == 1),
                "talk_attention: %d rows, %d / %d heads of %d, %d splits", a.n, a.H, a.G, a.D, a.nsplit);
    if (dt == PGK_F32) { if (pgk_status r = talk_any<float, float>(a, st)) return r; }
    else if (pgk_status r = io32 ? talk_any<bf16, float>(a, st) : talk_any<bf16, bf16>(a, st)) return r;
    *launches += 1;
    if (a.nsplit == 1) return PGK_OK;
    KvAttnArgs m{};
    m.positions = a.positions; m.B = a.n; m.H = a.H; m.G = a.G; m.D = a.D; m.R = a.R; m.window = a.window; m.chunked = a.chunked; m.nsplit = a.nsplit;
    m.po = a.po; m.pml = a.pml; m.out = a.out; m.ld_out = a.ld_out; m.sink = a.sink;
    *launches += 1;
    return kv_merge(m, io32 || dt == PGK_F32, st);
}

// -------------------------------------------------------------------------------------------- operators
// A wave per (row, head): norm over the head (norm null: none), columns i and i + rot / 2 turned by (first + row) * freq[i]
template <class T>
__global__ __launch_bounds__(256) void head_norm_rope_kernel(const T* x, const float* norm, const float* freq, T* out, int total, int heads, int dim, int rot, int first, float eps) {
    const int u = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, half = rot / 2;
    if (u >= total) return;
    const T* r = x + (size_t)u * dim;
    T* o = out + (size_t)u * dim;
    float ss = 0.f;
    for (int i = lane; i < dim; i += 64) { const float v = to_f(r[i]); ss = fmaf(v, v, ss); }
    const float inv = norm ? 1.0f / sqrtf(wave_sum(ss) / dim + eps) : 1.0f;
    auto at = [&](int i) { return to_f(r[i]) * inv * (norm ? norm[i] : 1.0f); };
    for (int i = lane; i < half; i += 64) {
        float s, c;
        sincosf((float)(first + u / heads) * freq[i], &s, &c);
        const float a = at(i), b = at(i + half);
        o[i] = from_f<T>(fmaf(a, c, -b * s));
        o[i + half] = from_f<T>(fmaf(b, c, a * s));
    }
    for (int i = rot + lane; i < dim; i += 64) o[i] = from_f<T>(at(i));
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_head_norm_rope(const void* x, const float* norm, const float* freq, void* out, int n, int heads, int dim, int rot, int first, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && out && x != out && n >= 1 && heads >= 1 && dim >= 1 && rot >= 0 && rot % 2 == 0 && rot <= dim && (!rot || freq) && first >= 0, "pgk_head_norm_rope: %d x %d x %d, %d turned", n, heads, dim, rot);
    PGK_DISPATCH_FLOAT(dt, "pgk_head_norm_rope", (head_norm_rope_kernel<T><<<ceil_div(n * heads, 4), 256, 0, resolve_stream(s)>>>((const T*)x, norm, freq, (T*)out, n * heads, heads, dim, rot, first, eps)));
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status pgk_talk_attention(const void* q, const void* k, const void* v, const float* talk, const float* sink, void* out, int hq, int hkv, int q_len, int kv_len, int first,
                              int dk, int dv, float scale, int window, int chunked, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(q && k && v && out && q_len >= 1 && dk >= 1 && dv >= 1 && first >= 0, "pgk_talk_attention: %d queries, head widths %d / %d", q_len, dk, dv);
    PGK_REQUIRE(hq >= 1 && hkv >= 1 && kv_len >= q_len, "pgk_talk_attention: %d / %d heads, %d keys", hq, hkv, kv_len);
    TalkArgs a{};
    a.q = q; a.ld_q = hq * dk; a.talk = talk; a.sink = sink; a.H = hq; a.G = hkv; a.D = dk; a.n = q_len; a.window = window; a.chunked = chunked; a.scale = scale; a.nsplit = 1;
    a.k = k; a.v = v; a.ld_kv = hkv * dk; a.kv_len = kv_len; a.pos0 = first; a.out = out; a.ld_out = hq * dv; a.Dv = dv; a.ld_v = hkv * dv;
    int launches = 0;
    return talk_attention(a, dt, dt == PGK_F32, resolve_stream(s), &launches);
}

}  // extern "C"
