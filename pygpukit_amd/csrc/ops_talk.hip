// Attention whose heads mix their scores before the softmax, with a sink per head, over a K/V ring or prompt rows (mixers.hip.h), and the
// step before it: bias, norm per head and rotation of projection rows.

#include <type_traits>
#include <vector>

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

// -------------------------------------------------------------------------------------------- bf16 on the matrix pipe
typedef __bf16 bf16x8_tk __attribute__((ext_vector_type(8)));
typedef float f32x4_tk __attribute__((ext_vector_type(4)));
typedef float f32x2_tk __attribute__((ext_vector_type(2)));
typedef short v4s_tk __attribute__((ext_vector_type(4)));
template <class A, class B>       // 16 bytes each
__device__ __forceinline__ f32x4_tk mfma_tk(const A& a, const B& b, f32x4_tk c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_tk, a), __builtin_bit_cast(bf16x8_tk, b), c, 0, 0, 0);
}
// four rows' worth of a 16-column block, transposed: two reads make an operand whose k order is 16 (j >> 2) + 4 (lane >> 4) + (j & 3)
__device__ __forceinline__ uint4 read_tr(const bf16* lo, const bf16* hi) {
    const v4s_tk a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_tk*)lo);
    const v4s_tk b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_tk*)hi);
    const uint2 x = __builtin_bit_cast(uint2, a), y = __builtin_bit_cast(uint2, b);
    return make_uint4(x.x, x.y, y.x, y.y);
}

// over the four quarters of a wave, lane by lane
__device__ __forceinline__ float max_of_quarters(float x) {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    x = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
    const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}

// ---- decode: one query per sequence ----
// A workgroup per (split, sequence), all heads, 32 keys at a time.  A wave has GW key heads, or WPG waves share one.  Raw scores K q go to
// LDS as S[head][key]; behind the barrier a wave mixes, in fp32 products S^T T^T of the matrix pipe, the heads of its key head, which
// leaves a lane with one head and an eighth of the keys: softmax in registers, then O^T[d][head] += V^T P^T, the waves of a key head each
// with their part of the columns.  Values pass through registers into a part of LDS of the wave's own; keys and values are fetched a step
// ahead (AHEAD: where they fit the registers).  S exists twice, so one barrier a step is enough.
constexpr int TD_S = 36;                                           // floats per head of S
static size_t talk_decode_lds(int nw, int H, int GW, int DW) {
    return (size_t)2 * ((H + 15) / 16 * 16) * TD_S * 4 + (size_t)nw * GW * 32 * (DW + 8) * 2;
}
template <class IT, int GW, int WPG, int RT>
__global__ __launch_bounds__(512) void talk_decode_kernel(unsigned long long* tl, TalkArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) char td_smem[];
    constexpr int D = 64 * RT, CH = D / 32, DW = D / WPG, DT = DW / 16, PC = DW / 8, NV = 32 * PC / 64, UN = WPG == 1 ? 2 : 1, LDV = DW + 8, KM = 4;
    constexpr bool AHEAD = GW * RT <= 2 * WPG;
    constexpr int GB = AHEAD ? GW : 1;                             // key heads in the registers
    const int H = a.H, G = a.G, rep = H / G, lane = threadIdx.x & 63, l15 = lane & 15, q4 = lane >> 4, s = blockIdx.x, b = blockIdx.y;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), nw = blockDim.x >> 6, sub = wid % WPG, gw = wid / WPG;     // the wave's key heads: gw + i nw / WPG
    const int kmt = (H + 15) / 16, SN = kmt * 16 * TD_S;
    float* S0 = reinterpret_cast<float*>(td_smem);                // [16 kmt][TD_S], twice
    bf16* kv = reinterpret_cast<bf16*>(S0 + 2 * SN) + wid * GW * 32 * LDV;     // [GW][32][LDV]
    int n, lo, k0, k1;
    ring_window(max(a.positions[b], 0), a.window, a.R, n, lo, a.chunked);
    split_range(n, a.nsplit, s, k0, k1);
    if (k0 >= k1) {                                                // an empty split: its record says so, the sums are never read
        for (int h = threadIdx.x; h < H; h += blockDim.x) {
            float* ml = a.pml + (((size_t)b * H + h) * a.nsplit + s) * 2;
            ml[0] = -INFINITY; ml[1] = 0.f;
        }
        tls.end();
        return;
    }
    const size_t gstep = (size_t)a.R * D;
    const bf16* kb = reinterpret_cast<const bf16*>(a.cache) + (size_t)b * 2 * G * gstep;
    const bf16* vb = kb + G * gstep;
    auto group = [&](int i) { return min(gw + i * (nw / WPG), G - 1); };       // (key heads past the last repeat it and store nothing)
    u32x4 qf[GW][CH], kf[GB][UN][CH], st[GB][NV];
    const int hl = min(l15, rep - 1), u0 = WPG == 1 ? 0 : sub & 1;
    auto fetch_k = [&](int kt, int i0) {                           // key heads i0 .. i0 + GB
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            const bf16* kr = kb + (size_t)ring_row(lo, min(kt + 16 * (u0 + u) + l15, k1 - 1), a.R) * D + 8 * q4;
#pragma unroll
            for (int i = 0; i < GB; ++i)
#pragma unroll
                for (int c = 0; c < CH; ++c) kf[i][u][c] = *reinterpret_cast<const u32x4*>(kr + group(i0 + i) * gstep + 32 * c);
        }
    };
    auto fetch_v = [&](int kt, int i0) {
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int p = v * 64 + lane;
            const bf16* vr = vb + (size_t)ring_row(lo, min(kt + p / PC, k1 - 1), a.R) * D + sub * DW + p % PC * 8;
#pragma unroll
            for (int i = 0; i < GB; ++i) st[i][v] = *reinterpret_cast<const u32x4*>(vr + group(i0 + i) * gstep);
        }
    };
    // T as operand: column l15 is the head's, steps go through the raw heads 16 k + 4 q4 + j; zero where there is none
    f32x4_tk tf[GW][KM];
#pragma unroll
    for (int i = 0; i < GW; ++i) {
        const int h = group(i) * rep + hl;
#pragma unroll
        for (int k = 0; k < KM; ++k) {
            tf[i][k] = f32x4_tk{0.f, 0.f, 0.f, 0.f};
            if (k >= kmt) continue;                                // uniform
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int g = 16 * k + 4 * q4 + j;
                tf[i][k][j] = a.talk ? a.talk[(size_t)h * H + min(g, H - 1)] : h == g ? 1.0f : 0.f;
            }
        }
    }
    if (AHEAD) fetch_k(k0, 0);
#pragma unroll
    for (int i = 0; i < GW; ++i) {
        const bf16* qr = reinterpret_cast<const bf16*>(a.q) + (size_t)b * a.ld_q + (size_t)(group(i) * rep + hl) * D + 8 * q4;
#pragma unroll
        for (int c = 0; c < CH; ++c) qf[i][c] = *reinterpret_cast<const u32x4*>(qr + 32 * c);
    }
    if (AHEAD) fetch_v(k0, 0);
    const float mult = a.scale * TK_LOG2E;
#pragma unroll
    for (int i = 0; i < GW; ++i)
#pragma unroll
        for (int k = 0; k < KM; ++k)
#pragma unroll
            for (int j = 0; j < 4; ++j) tf[i][k][j] = 16 * k + 4 * q4 + j < H ? tf[i][k][j] * mult : 0.f;
    for (int i = H * TD_S + threadIdx.x; i < SN; i += blockDim.x) { S0[i] = 0.f; S0[SN + i] = 0.f; }      // heads that do not exist
    f32x4_tk o[GW][DT];
    float m[GW], l[GW];
#pragma unroll
    for (int i = 0; i < GW; ++i) {
        m[i] = -INFINITY; l[i] = 0.f;
#pragma unroll
        for (int t = 0; t < DT; ++t) o[i][t] = f32x4_tk{0.f, 0.f, 0.f, 0.f};
    }
    float* S = S0;
    for (int kt = k0; kt < k1; kt += 32) {
        if (WPG <= 2 || sub < 2) {                                 // uniform: two waves have the two halves of the keys
#pragma unroll
            for (int i = 0; i < GW; ++i) {
                if (!AHEAD) fetch_k(kt, i);
#pragma unroll
                for (int u = 0; u < UN; ++u) {
                    f32x4_tk t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int c = 0; c < CH; ++c) t = mfma_tk(kf[AHEAD ? i : 0][u][c], qf[i][c], t);
                    if (l15 < rep) *reinterpret_cast<f32x4_tk*>(S + (group(i) * rep + l15) * TD_S + 16 * (u0 + u) + 4 * q4) = t;      // keys 16 u + 4 q4 .. of head l15
                }
                if (!AHEAD) __builtin_amdgcn_sched_barrier(0);
            }
        }
        if (AHEAD && kt + 32 < k1) fetch_k(kt + 32, 0);            // the next tile travels under the rest of this one
        wave_sync();                                               // (the last step's reads of the values)
#pragma unroll
        for (int i = 0; i < GW; ++i) {
            if (!AHEAD) fetch_v(kt, i);
#pragma unroll
            for (int v = 0; v < NV; ++v) {
                const int p = v * 64 + lane;
                *reinterpret_cast<u32x4*>(kv + (i * 32 + p / PC) * LDV + p % PC * 8) = st[AHEAD ? i : 0][v];
            }
            if (!AHEAD) __builtin_amdgcn_sched_barrier(0);
        }
        if (AHEAD && kt + 32 < k1) fetch_v(kt + 32, 0);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();                              // (loads stay in flight)
        asm volatile("" ::: "memory");
        const float* sk = S + 4 * q4 * TD_S + l15;
        f32x4_tk x[GW][2];
#pragma unroll
        for (int i = 0; i < GW; ++i) { x[i][0] = f32x4_tk{0.f, 0.f, 0.f, 0.f}; x[i][1] = x[i][0]; }
#pragma unroll
        for (int k = 0; k < KM; ++k) {
            if (k >= kmt) continue;                                // uniform
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int u = 0; u < 2; ++u) {
                    const float r = sk[(16 * k + j) * TD_S + 16 * u];
#pragma unroll
                    for (int i = 0; i < GW; ++i) x[i][u] = __builtin_amdgcn_mfma_f32_16x16x4f32(r, tf[i][k][j], x[i][u], 0, 0, 0);
                }
        }
        const int seen = k1 - kt - 4 * q4;
#pragma unroll
        for (int i = 0; i < GW; ++i) {
            f32x4_tk s0 = x[i][0], s1 = x[i][1];
            if (kt + 32 > k1) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (e >= seen) s0[e] = -INFINITY;
                    if (e + 16 >= seen) s1[e] = -INFINITY;
                }
            }
            const float top = max_of_quarters(fmaxf(fmaxf(fmaxf(s0[0], s0[1]), fmaxf(s0[2], s0[3])), fmaxf(fmaxf(s1[0], s1[1]), fmaxf(s1[2], s1[3]))));
            const float mn = fmaxf(m[i], top), f = __builtin_amdgcn_exp2f(m[i] - mn);        // mn is finite: kt < k1
            m[i] = mn;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s0[e] = __builtin_amdgcn_exp2f(s0[e] - mn);
                s1[e] = __builtin_amdgcn_exp2f(s1[e] - mn);
            }
            l[i] = fmaf(l[i], f, ((s0[0] + s0[1]) + (s0[2] + s0[3])) + ((s1[0] + s1[1]) + (s1[2] + s1[3])));
            const uint4 pf = make_uint4(pack_bf16x2(s0[0], s0[1]), pack_bf16x2(s0[2], s0[3]), pack_bf16x2(s1[0], s1[1]), pack_bf16x2(s1[2], s1[3]));
            const bf16* row = kv + (i * 32 + 4 * q4 + (l15 >> 2)) * LDV + 4 * (l15 & 3);
#pragma unroll
            for (int t = 0; t < DT; ++t) o[i][t] = mfma_tk(read_tr(row + 16 * t, row + 16 * LDV + 16 * t), pf, o[i][t] * f);
        }
        S = S == S0 ? S0 + SN : S0;
    }
#pragma unroll
    for (int i = 0; i < GW; ++i) {
        float sum = l[i];
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        const int g = gw + i * (nw / WPG), h = g * rep + l15, d0 = sub * DW + 4 * q4;
        if (g >= G || l15 >= rep) continue;
        if (a.nsplit > 1) {
            const size_t rec = ((size_t)b * H + h) * a.nsplit + s;
            if (sub == 0 && q4 == 0) *reinterpret_cast<float2*>(a.pml + rec * 2) = make_float2(m[i], sum);
            float* po = a.po + rec * D + d0;
#pragma unroll
            for (int t = 0; t < DT; ++t) *reinterpret_cast<f32x4_tk*>(po + 16 * t) = o[i][t];
        } else {
            const float f = sink_scale(a.sink, h, m[i], sum);
            IT* out = reinterpret_cast<IT*>(a.out) + (size_t)b * a.ld_out + h * D + d0;
#pragma unroll
            for (int t = 0; t < DT; ++t) store4<IT>(out + 16 * t, make_float4(o[i][t][0] * f, o[i][t][1] * f, o[i][t][2] * f, o[i][t][3] * f));
        }
    }
    tls.end();
}

static bool talk_decode_ok(const TalkArgs& a) {
    return a.cache && a.D % 64 == 0 && a.D <= (a.G > 8 ? 128 : 256) && a.H <= 64 && a.G <= 16 && a.H / a.G <= 16 && a.ld_q % 8 == 0 && a.ld_out % 4 == 0 && aligned16(a.q) && aligned16(a.out);
}
template <class IT>
static pgk_status talk_decode_mfma(const TalkArgs& a, hipStream_t st) {
    auto go = [&](auto gw, auto wpg, auto rt) -> pgk_status {
        constexpr int GW = decltype(gw)::value, WPG = decltype(wpg)::value, RT = decltype(rt)::value;
        auto kfn = &talk_decode_kernel<IT, GW, WPG, RT>;
        const int nw = GW > 1 ? 8 : min(8, a.G * WPG);
        const size_t lds = talk_decode_lds(nw, a.H, GW, 64 * RT / WPG);
        static bool done = false;
        if (lds > 48 * 1024 && !done) {
            PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, TALK_LDS_MAX + 8 * 1024));
            done = true;
        }
        PGK_CHECK_HIP(launch_k(kfn, dim3(a.nsplit, a.n), dim3(64 * nw), lds, st, a));
        return PGK_OK;
    };
    using std::integral_constant;
    integral_constant<int, 1> one;
    integral_constant<int, 2> two;
    integral_constant<int, 4> four;
    auto pick = [&](auto rt) -> pgk_status {
        if constexpr (decltype(rt)::value <= 2) { if (a.G > 8) return go(two, one, rt); }
        return a.G <= 2 ? go(one, four, rt) : a.G <= 4 ? go(one, two, rt) : go(one, one, rt);
    };
    switch (a.D / 64) {
        case 1: return pick(one);
        case 2: return pick(two);
        case 3: return pick(integral_constant<int, 3>{});
        default: return pick(four);
    }
}

// ---- prompts: 16 queries per workgroup, 32 keys at a time ----
// NW waves.  (1) The raw scores [32 keys][16 queries] of HW heads per wave go to LDS as S[head][query][key]; (2) a wave mixes the heads of its
// 16 / NW queries, fp32 products T S of the matrix pipe, into the NW HO output heads of this workgroup (blockIdx.y: which), in place;
// (3) HO output heads per wave: their rows come back, softmax in registers (a lane per query and eighth of the keys), O^T[d][query] +=
// V^T P^T.  Keys, then values, of a wave's key head come as whole rows through registers (fetched a step ahead) into a part of LDS of the
// wave's own, in 16-byte pieces that are XOR-ed by the row, so that operand reads of 16 rows spread over the banks.  DB: S exists twice, so
// that no wave waits for the others' step 3.  ONE: the heads of a wave share a key head.  Heads past the last repeat it and store nothing.
// blockIdx.z: which `part` tiles of 32 keys; queries with several such parts leave, per part, a normalised output and (m, l), which
// talk_join_kernel combines.
constexpr int TF_Q = 36, TF_H = 16 * TF_Q;                         // floats per query and head of S
static size_t talk_flash_lds(int NW, int HW, int HO, int D, bool db) {
    return (size_t)NW * HW * TF_H * 4 * (db ? 2 : 1) + (size_t)(NW * HO + 15) / 16 * 16 * (NW * HW + 4) * 4 + (size_t)NW * 32 * D * 2;
}

struct TalkParts { int part; bf16* o; float2* ml; };               // o [parts][n][H D], ml [parts][n][H]
__device__ __forceinline__ int talk_first_key(const TalkArgs& a, int q) {
    const int last = a.kv_len - a.n + q;
    return last + 1 - min(span_keys(a.pos0 + last, a.window, a.chunked), last + 1);
}

template <int NW, int HW, int HO, int RT, bool ONE, bool DB>
__global__ __launch_bounds__(64 * NW, 2) void talk_flash_kernel(unsigned long long* tl, TalkArgs a, int tiles, int per, TalkParts pt) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) char tf_smem[];
    constexpr int D = 64 * RT, CH = D / 32, DT = D / 16, HM = (NW * HO + 15) / 16, KS = NW * HW / 4, PC = D / 8, TL = NW * HW + 4, SN = NW * HW * TF_H;
    constexpr bool FULL = (HW * CH + HO * DT) * 4 >= 128;          // queries and sums take most of the registers
    float* S0 = reinterpret_cast<float*>(tf_smem);                // [NW HW][16][TF_Q]
    float* T = S0 + SN * (DB ? 2 : 1);                             // [16 HM][TL], times the score factor, zero where there is no head
    bf16* kv = reinterpret_cast<bf16*>(T + 16 * HM * TL) + (threadIdx.x >> 6) * 32 * D;       // [32][D] of this wave
    const int H = a.H, rep = H / a.G, lane = threadIdx.x & 63, l15 = lane & 15, q4 = lane >> 4;
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), ho0 = (int)blockIdx.y * NW * HO;
    // runs of `per` tiles (a chunk's), the last tiles of all runs first: they have the most keys
    const int runs = (tiles + per - 1) / per, tile = (int)(blockIdx.x % runs) * per + per - 1 - (int)(blockIdx.x / runs);
    if (tile >= tiles) { tls.end(); return; }
    const int q0 = tile * 16, nq = min(16, a.n - q0), past = a.kv_len - a.n;
    const int my_q = q0 + min(l15, nq - 1), my_lo = talk_first_key(a, my_q), my_last = past + my_q;
    const int k_first = talk_first_key(a, q0), k_last = past + q0 + nq, lo_max = talk_first_key(a, q0 + nq - 1), last_min = past + q0;
    const int k_begin = k_first + (int)blockIdx.z * pt.part * 32, k_end = min(k_last, k_begin + pt.part * 32);
    if (k_begin >= k_last) { tls.end(); return; }
    const bf16 *kbase = reinterpret_cast<const bf16*>(a.k), *vbase = reinterpret_cast<const bf16*>(a.v);
    auto head = [&](int i) { return min(wid * HW + i, H - 1); };
    auto out_head = [&](int i) { return min(ho0 + wid * HO + i, H - 1); };
    // 32 rows of a key head's keys or values pass through `st` into this wave's part of LDS: piece c of row r at c ^ swizzle(r)
    constexpr int NV = 32 * PC / 64;
    auto swz = [](int r) { return RT == 2 ? (r & 7) * 2 : ((r >> 1) & 3) * 2; };
    u32x4 qf[HW][CH], st[NV];
    uint32_t off[NV];                                              // of this lane's pieces in 32 whole rows
#pragma unroll
    for (int i = 0; i < NV; ++i) off[i] = (uint32_t)((i * 64 + lane) / PC) * (uint32_t)a.ld_kv + (lane % PC) * 8;
    auto fetch = [&](const bf16* base, int g, int kt) {
        const bf16* at = base + (size_t)kt * a.ld_kv + g * D;      // (uniform)
        if (kt + 32 <= k_end) {
#pragma unroll
            for (int i = 0; i < NV; ++i) st[i] = *reinterpret_cast<const u32x4*>(at + off[i]);
        } else if (kt < k_end) {                                   // rows past the end repeat the last
            const int back = k_end - 1 - kt;
#pragma unroll
            for (int i = 0; i < NV; ++i) st[i] = *reinterpret_cast<const u32x4*>(at + (size_t)min((i * 64 + lane) / PC, back) * a.ld_kv + (lane % PC) * 8);
        }
    };
    auto put = [&]() {                                             // (behind this wave's reads of what was there)
        wave_sync();
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int p = i * 64 + lane, r = p / PC;
            *reinterpret_cast<u32x4*>(kv + r * D + ((p % PC) ^ swz(r)) * 8) = st[i];
        }
        wave_sync();
    };
#pragma unroll
    for (int i = 0; i < HW; ++i) {
        const bf16* qr = reinterpret_cast<const bf16*>(a.q) + (size_t)my_q * a.ld_q + (size_t)head(i) * D + 8 * q4;
#pragma unroll
        for (int c = 0; c < CH; ++c) qf[i][c] = *reinterpret_cast<const u32x4*>(qr + 32 * c);
    }
    fetch(kbase, head(0) / rep, k_begin);
    const float mult = a.scale * TK_LOG2E;
    for (int i = threadIdx.x; i < 16 * HM * TL; i += 64 * NW) {
        const int h = ho0 + i / TL, g = i % TL;
        T[i] = h < H && g < H ? (a.talk ? a.talk[h * H + g] : h == g ? 1.0f : 0.f) * mult : 0.f;
    }
#pragma unroll
    for (int d = 0; d < (DB ? 2 : 1); ++d)
        for (int i = H * TF_H + threadIdx.x; i < SN; i += 64 * NW) S0[d * SN + i] = 0.f;      // heads that do not exist
    f32x4_tk o[HO][DT];
    float m[HO], l[HO];
#pragma unroll
    for (int i = 0; i < HO; ++i) {
        m[i] = -INFINITY; l[i] = 0.f;
#pragma unroll
        for (int t = 0; t < DT; ++t) o[i][t] = f32x4_tk{0.f, 0.f, 0.f, 0.f};
    }
    float* S = S0;
    for (int kt = k_begin; kt < k_end; kt += 32) {
        constexpr int KG = ONE ? 1 : HW, VG = ONE ? 1 : HO;        // key heads of the wave (those of the output heads: VG) and the heads of each
#pragma unroll
        for (int gi = 0; gi < KG; ++gi) {
            put();
            if (gi + 1 < KG) fetch(kbase, head(gi + 1) / rep, kt);
            else fetch(vbase, out_head(0) / rep, kt);
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                u32x4 kf[CH];
#pragma unroll
                for (int c = 0; c < CH; ++c) kf[c] = *reinterpret_cast<const u32x4*>(kv + (16 * u + l15) * D + (((4 * c + q4) ^ swz(l15)) << 3));
#pragma unroll
                for (int j = 0; j < HW / KG; ++j) {
                    const int i = gi * (HW / KG) + j;
                    f32x4_tk t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int c = 0; c < CH; ++c) t = mfma_tk(kf[c], qf[i][c], t);
                    *reinterpret_cast<f32x4_tk*>(S + head(i) * TF_H + l15 * TF_Q + 16 * u + 4 * q4) = t;        // keys 16 u + 4 q4 .. of query l15
                }
                if (FULL) __builtin_amdgcn_sched_barrier(0);       // (registers: one half's keys at a time)
            }
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();                              // (loads stay in flight)
        asm volatile("" ::: "memory");
#pragma unroll (FULL ? 1 : 2)
        for (int pass = 0; pass < 16 / NW; ++pass) {               // a query at a time: lane l15 has keys 2 l15 and 2 l15 + 1
            float* at = S + (wid * (16 / NW) + pass) * TF_Q + 2 * l15;
            f32x2_tk r[KS];
#pragma unroll
            for (int k = 0; k < KS; ++k) r[k] = *reinterpret_cast<const f32x2_tk*>(at + (4 * k + q4) * TF_H);
            f32x4_tk x[HM][2];
            const float* tp = T + l15 * TL + q4;                   // T as operand: row l15 of each 16 heads, columns 4 k + q4
#pragma unroll
            for (int mt = 0; mt < HM; ++mt)
#pragma unroll
                for (int j = 0; j < 2; ++j) {
                    x[mt][j] = f32x4_tk{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int k = 0; k < KS; ++k) x[mt][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(tp[mt * 16 * TL + 4 * k], r[k][j], x[mt][j], 0, 0, 0);
                }
            // (every lane's reads of this query fed the products: the wave may write it)
#pragma unroll
            for (int mt = 0; mt < HM; ++mt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int h = 16 * mt + 4 * q4 + e;
                    if (h < NW * HO) *reinterpret_cast<f32x2_tk*>(at + h * TF_H) = f32x2_tk{x[mt][0][e], x[mt][1][e]};
                }
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        const bool whole = kt >= lo_max && kt + 31 <= last_min;
#pragma unroll
        for (int gi = 0; gi < VG; ++gi) {
            put();
            if (gi + 1 < VG) fetch(vbase, out_head(gi + 1) / rep, kt);
            else fetch(kbase, head(0) / rep, kt + 32);
            constexpr int HG = HO / VG;
            uint4 pf[HG];
#pragma unroll
            for (int j = 0; j < HG; ++j) {
                const int i = gi * HG + j;
                const float* sr = S + min(wid * HO + i, NW * HW - 1) * TF_H + l15 * TF_Q + 4 * q4;
                f32x4_tk s0 = *reinterpret_cast<const f32x4_tk*>(sr), s1 = *reinterpret_cast<const f32x4_tk*>(sr + 16);      // keys 4 q4 .., 16 + 4 q4 ..
                if (!whole) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        const uint32_t k = kt + 4 * q4 + e - my_lo, seen = my_last - my_lo;      // (unsigned: before the first is past the last)
                        if (k > seen) s0[e] = -INFINITY;
                        if (k + 16 > seen) s1[e] = -INFINITY;
                    }
                }
                const float top = max_of_quarters(fmaxf(fmaxf(fmaxf(s0[0], s0[1]), fmaxf(s0[2], s0[3])), fmaxf(fmaxf(s1[0], s1[1]), fmaxf(s1[2], s1[3]))));
                // the reference follows the maximum only when it is left behind by 2^8: until then the weights are as exact
                if (__any(top > m[i] + 8.0f)) {
                    const float mn = fmaxf(m[i], top), f = mn == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m[i] - mn);
                    m[i] = mn;
                    l[i] *= f;
#pragma unroll
                    for (int t = 0; t < DT; ++t) o[i][t] *= f;
                }
                const float ref = m[i] == -INFINITY ? 0.f : m[i];              // (a query that has seen no key yet)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s0[e] = __builtin_amdgcn_exp2f(s0[e] - ref);
                    s1[e] = __builtin_amdgcn_exp2f(s1[e] - ref);
                }
                l[i] += ((s0[0] + s0[1]) + (s0[2] + s0[3])) + ((s1[0] + s1[1]) + (s1[2] + s1[3]));
                pf[j] = make_uint4(pack_bf16x2(s0[0], s0[1]), pack_bf16x2(s0[2], s0[3]), pack_bf16x2(s1[0], s1[1]), pack_bf16x2(s1[2], s1[3]));
            }
            const int r0 = 4 * q4 + (l15 >> 2), sz = swz(r0);                  // rows r0 and r0 + 16 have the same swizzle
#pragma unroll
            for (int t = 0; t < DT; ++t) {
                const bf16* row = kv + r0 * D + (((2 * t + ((l15 & 3) >> 1)) ^ sz) << 3) + 4 * (l15 & 1);
                const uint4 vt = read_tr(row, row + 16 * D);
#pragma unroll
                for (int j = 0; j < HG; ++j) o[gi * HG + j][t] = mfma_tk(vt, pf[j], o[gi * HG + j][t]);
                if (FULL && (t & 3) == 3) __builtin_amdgcn_sched_barrier(0);   // (... and no more reads in flight than four columns')
            }
        }
        if constexpr (DB) S = S == S0 ? S0 + SN : S0;
        else {
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
            __builtin_amdgcn_s_barrier();                          // the next tile's scores take S
        }
    }
#pragma unroll
    for (int i = 0; i < HO; ++i) {
        float sum = l[i];
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        const bool join = k_last - k_first > pt.part * 32;         // uniform
        const float f = join ? (sum > 0.f ? 1.0f / sum : 0.f) : sink_scale(a.sink, out_head(i), m[i], sum);
        const int h = ho0 + wid * HO + i;
        if (l15 >= nq || h >= H) continue;
        bf16* out = reinterpret_cast<bf16*>(a.out) + (size_t)(q0 + l15) * a.ld_out + (size_t)h * D + 4 * q4;
        if (join) {
            const size_t row = (size_t)blockIdx.z * a.n + q0 + l15;
            if (q4 == 0) pt.ml[row * H + h] = make_float2(m[i], sum);
            out = pt.o + (row * H + h) * D + 4 * q4;
        }
#pragma unroll
        for (int t = 0; t < DT; ++t) store4<bf16>(out + 16 * t, make_float4(o[i][t][0] * f, o[i][t][1] * f, o[i][t][2] * f, o[i][t][3] * f));
    }
    tls.end();
}

// A workgroup per query, eight columns per thread
__global__ __launch_bounds__(256) void talk_join_kernel(unsigned long long* tl, TalkArgs a, TalkParts pt) {
    const TLStamp tls(tl);
    const int q = blockIdx.x, q0 = q / 16 * 16, n = (a.kv_len - a.n + min(q0 + 16, a.n) - talk_first_key(a, q0) + pt.part * 32 - 1) / (pt.part * 32);
    if (n > 1)
        for (int i = threadIdx.x; i < a.H * a.D / 8; i += 256) {
            const int h = i * 8 / a.D;
            const float2* ml = pt.ml + (size_t)q * a.H + h;
            float m = -INFINITY;
            for (int p = 0; p < n; ++p) m = fmaxf(m, ml[(size_t)p * a.n * a.H].x);
            float l = 0.f, o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
            for (int p = 0; p < n; ++p) {
                const float2 r = ml[(size_t)p * a.n * a.H];
                const float w = r.y * __builtin_amdgcn_exp2f(r.x - m);         // (every query sees itself: m is finite)
                const uint4 v = *reinterpret_cast<const uint4*>(pt.o + ((size_t)p * a.n + q) * a.H * a.D + i * 8);
                const uint32_t* u = &v.x;
                l += w;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    o[2 * j] = fmaf(w, __uint_as_float(u[j] << 16), o[2 * j]);
                    o[2 * j + 1] = fmaf(w, __uint_as_float(u[j] & 0xffff0000u), o[2 * j + 1]);
                }
            }
            const float f = sink_scale(a.sink, h, m, l);
            bf16* out = reinterpret_cast<bf16*>(a.out) + (size_t)q * a.ld_out + i * 8;
            store4<bf16>(out, make_float4(o[0] * f, o[1] * f, o[2] * f, o[3] * f));
            store4<bf16>(out + 4, make_float4(o[4] * f, o[5] * f, o[6] * f, o[7] * f));
        }
    tls.end();
}

static bool talk_flash_ok(const TalkArgs& a) {
    return !a.cache && !a.Dv && (a.D == 64 || a.D == 128) && a.H <= 32 && a.ld_q % 8 == 0 && a.ld_kv % 8 == 0 && a.ld_out % 4 == 0 && aligned16(a.q) && aligned16(a.k) && aligned16(a.v) &&
           (reinterpret_cast<uintptr_t>(a.out) & 7u) == 0;
}
static int cu_count() {
    static const int n = [] {
        int dev = 0;
        hipDeviceProp_t prop;
        return hipGetDevice(&dev) == hipSuccess && hipGetDeviceProperties(&prop, dev) == hipSuccess && prop.multiProcessorCount > 0 ? prop.multiProcessorCount : 256;
    }();
    return n;
}
// Parts of the heaviest query tile's keys, and the 32-key tiles of one.  One workgroup fits a CU, so a launch ends with its longest
// workgroup: where CUs idle or the heaviest tiles outlast the mean, more parts pay, until their overhead and the joining do not.  Counted in
// times of a tile (about 3 us).
static int plan_parts(const TalkArgs& a, int tiles, int groups, int cus, int* part) {
    std::vector<int> keys(tiles);
    int most = 1;
    long long all = 0;
    for (int t = 0; t < tiles; ++t) {
        const int last = a.kv_len - a.n + 16 * t, seen = span_keys(a.pos0 + last, a.window, a.chunked), own = a.n - 16 * t < 16 ? a.n - 16 * t : 16;
        keys[t] = ceil_div((seen < last + 1 ? seen : last + 1) + own - 1, 32);
        all += keys[t];
        if (keys[t] > most) most = keys[t];
    }
    int best = 1;
    double best_cost = 0.0;
    for (int k = 1; k <= 16 && k <= most; ++k) {
        const int p = ceil_div(most, k);
        long long wgs = 0, joined = 0;
        for (int t : keys) { const int c = ceil_div(t, p); wgs += c; if (c > 1) joined += c; }
        const double lead = 3.0, alone = p + lead, shared = wgs * groups <= cus ? 0.0 : (double)(all + lead * wgs) * groups / cus + 2.0;
        const double join = k == 1 ? 0.0 : 1.7 + (double)joined * 16 * a.H * a.D * 4 / 12e6;
        const double cost = (alone > shared ? alone : shared) + join;
        if (k == 1 || cost < best_cost) { best = k; best_cost = cost; }
    }
    *part = ceil_div(most, best);
    return ceil_div(most, *part);
}
static pgk_status talk_flash(const TalkArgs& a, hipStream_t st, int* launches) {
    const int tiles = ceil_div(a.n, 16), rep = a.H / a.G;
    const int per = a.chunked && a.window / 16 >= 1 && a.window / 16 < tiles ? a.window / 16 : tiles, runs = ceil_div(tiles, per);
    auto go = [&](auto nw, auto hw, auto ho, auto rt, auto one, auto db) -> pgk_status {
        constexpr int NW = decltype(nw)::value, HW = decltype(hw)::value, HO = decltype(ho)::value, RT = decltype(rt)::value;
        auto kfn = &talk_flash_kernel<NW, HW, HO, RT, decltype(one)::value, decltype(db)::value>;
        const size_t lds = talk_flash_lds(NW, HW, HO, 64 * RT, decltype(db)::value);
        static bool done = false;
        if (lds > 48 * 1024 && !done) {
            PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
            done = true;
        }
        TalkParts pt{};
        const int groups = ceil_div(a.H, NW * HO), parts = plan_parts(a, tiles, groups, cu_count(), &pt.part);
        void* ws = nullptr;
        if (parts > 1) {
            const size_t rows = (size_t)parts * a.n * a.H, o_bytes = (rows * a.D * 2 + 255) & ~(size_t)255;
            if (pgk_status r = pgk_malloc(&ws, o_bytes + rows * sizeof(float2))) return r;
            pt.o = (bf16*)ws; pt.ml = (float2*)((char*)ws + o_bytes);
        }
        hipError_t err = launch_k(kfn, dim3(runs * per, groups, parts), dim3(64 * NW), lds, st, a, tiles, per, pt);
        if (ws) {
            if (err == hipSuccess) err = launch_k(&talk_join_kernel, dim3(a.n), dim3(256), 0, st, a, pt);
            *launches += 1;
            pgk_free(ws);                                          // (what takes it next runs behind these kernels)
        }
        PGK_CHECK_HIP(err);
        return PGK_OK;
    };
    using std::integral_constant;
    using std::true_type;
    using std::false_type;
    integral_constant<int, 1> one;
    integral_constant<int, 2> two;
    integral_constant<int, 4> four;
    integral_constant<int, 8> eight;
    auto pick = [&](auto rt) -> pgk_status {
        if (a.H <= 4) return go(four, one, one, rt, true_type{}, true_type{});
        if (a.H <= 8) return rep % 2 ? go(eight, one, one, rt, true_type{}, true_type{}) : go(four, two, two, rt, true_type{}, true_type{});
        if (a.H <= 16) return rep % 2 ? go(eight, two, two, rt, false_type{}, true_type{}) : go(eight, two, two, rt, true_type{}, true_type{});
        return rep % 4 ? go(eight, four, two, rt, false_type{}, false_type{}) : go(eight, four, two, rt, true_type{}, false_type{});
    };
    return a.D == 64 ? pick(one) : pick(two);
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
    pgk_status r;
    if (dt == PGK_F32) r = talk_any<float, float>(a, st);
    else if (talk_decode_ok(a)) r = io32 ? talk_decode_mfma<float>(a, st) : talk_decode_mfma<bf16>(a, st);
    else if (!io32 && talk_flash_ok(a)) r = talk_flash(a, st, launches);
    else r = io32 ? talk_any<bf16, float>(a, st) : talk_any<bf16, bf16>(a, st);
    if (r) return r;
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
    a.k = k; a.v = v; a.ld_kv = hkv * dk; a.kv_len = kv_len; a.pos0 = first; a.out = out; a.ld_out = hq * dv; a.Dv = dk == dv && dk % 64 == 0 ? 0 : dv; a.ld_v = hkv * dv;      // (0: as wide, in the same rows)
    int launches = 0;
    return talk_attention(a, dt, dt == PGK_F32, resolve_stream(s), &launches);
}

}  // extern "C"
