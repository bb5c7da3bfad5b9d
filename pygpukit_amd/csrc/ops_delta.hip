// Gated delta rule with a decay per key channel (mixers.hip.h): per head a state S [dim][vdim] in fp32,
//   S <- diag(g) S,  u = b (v - S^T k),  S <- S + k u^T,  o = S^T q.
// Decays, strengths, unit norms and the state are fp32 whatever the element type.
//
// Two forms.  Token by token (decode, short portions, head widths beyond 128): one workgroup per sequence and head, the state in
// registers.  Chunked (prompts), chunks of 64 rows; with G_ij = prod_{j < t <= i} g_t (per channel, G_i from the chunk's start):
//   1. every chunk on its own:  A_ij = b_i sum_d k_i k_j G_ij (j < i),  B_ij = sum_d q_i k_j G_ij (j <= i),
//      (I + A) X = b v  and  (I + A) W = b (k G):  with the state S before the chunk the written values are  u = X - W S
//   2. along the chunks, for 16 columns of the state at a time:  U = X - W S,  o = (q G) S + B U,  S <- diag(G_end) S + (k G_end,j)^T U
//   3. norm and gate of the output rows
// Decays are products of g over the rows they span, never quotients, so strong decays neither overflow nor cancel: A and B are built in
// blocks of 16 rows, off the diagonal from factors that reach to a block's edge, on the diagonal pair by pair.  (I + A) is solved by
// block substitution with the 16 x 16 inverses.  All products are fp32 (v_mfma_f32_16x16x4_f32).

#include <type_traits>
#include <vector>

#include "mixers.hip.h"

namespace pgk {

// decay exponent of one channel: g = exp(-decay softplus(z + bias))
__device__ __forceinline__ float delta_fade(float z, float bias, float decay) {
    const float t = z + bias;
    return expf(-decay * (t > 20.f ? t : log1pf(expf(t))));
}
constexpr float UNIT_EPS = 1e-6f;

// -------------------------------------------------------------------------------------------- token by token
// A thread owns four columns of every NG-th state row: RPT rows in registers, or (RPT 0) in memory.
template <class T, class IT, bool EXACT, int RPT>
__global__ __launch_bounds__(512) void delta_scan_kernel(unsigned long long* tl, DeltaArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float red[16];
    const int tid = threadIdx.x, NT = blockDim.x, lane = tid & 63, h = blockIdx.x, dim = a.dim, vdim = a.vdim, rep = a.H / a.G, kh = h / rep;
    const int NC = vdim / 4, NG = NT / NC, c = tid % NC, g = tid / NC;
    float *q = sm, *k = q + dim, *f = k + dim, *v = f + dim, *pk = v + vdim, *pq = pk + NG * vdim;      // pk, pq [NG][vdim]
    SeqSpan s;
    if (a.seqs) s = a.seqs[blockIdx.y];
    else { s.row0 = blockIdx.y; s.len = 1; s.start = max(a.positions[blockIdx.y], 0); s.slot = blockIdx.y; }
    float* S = a.state + ((size_t)s.slot * a.H + h) * dim * vdim;
    const bool act = g < NG;
    constexpr int R = RPT > 0 ? RPT : 1;
    float4 x[R];
    if constexpr (RPT > 0) {
#pragma unroll
        for (int i = 0; i < R; ++i)
            x[i] = s.start > 0 && act && g + i * NG < dim ? *reinterpret_cast<const float4*>(S + (size_t)(g + i * NG) * vdim + 4 * c) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const float qs = 1.0f / sqrtf((float)a.dim_true), decay = a.decay[h];
    for (int t = 0; t < s.len; ++t) {
        const IT* in = reinterpret_cast<const IT*>(a.in) + (size_t)(s.row0 + t) * a.ld_in;
        const T* row = reinterpret_cast<const T*>(a.rows) + (size_t)(s.row0 + t) * a.ld_rows;
        const int pos = s.start + t;
        auto channel = [&](int ch, bool own) { return a.seqs ? to_f(row[ch]) : conv_step<T, IT, EXACT>(a.conv, in, ch, s.slot, pos, own); };
        for (int i = tid; i < 3 * dim + vdim; i += NT) {
            if (i < dim) q[i] = channel(kh * dim + i, h % rep == 0);
            else if (i < 2 * dim) k[i - dim] = channel(a.G * dim + kh * dim + i - dim, h % rep == 0);
            else if (i < 3 * dim) f[i - 2 * dim] = delta_fade(a.z[(size_t)(s.row0 + t) * a.ld_z + h * dim + i - 2 * dim], a.dt_bias[h * dim + i - 2 * dim], decay);
            else v[i - 3 * dim] = channel(2 * a.G * dim + h * vdim + i - 3 * dim, true);
        }
        const float beta = 1.0f / (1.0f + expf(-to_f(in[a.b_off + h])));
        __syncthreads();
        float sq = 0.f, sk = 0.f, qk = 0.f;                        // every wave for itself: no barrier
        for (int d = lane; d < dim; d += 64) { sq = fmaf(q[d], q[d], sq); sk = fmaf(k[d], k[d], sk); qk = fmaf(q[d], k[d], qk); }
        const float iq = qs / sqrtf(wave_sum(sq) + UNIT_EPS), ik = 1.0f / sqrtf(wave_sum(sk) + UNIT_EPS), kq = wave_sum(qk) * iq * ik;
        float4 ak = {0.f, 0.f, 0.f, 0.f}, aq = {0.f, 0.f, 0.f, 0.f};
        auto fold = [&](float4& y, int d) {
            const float fd = f[d], kd = k[d], qd = q[d];
            y.x *= fd; y.y *= fd; y.z *= fd; y.w *= fd;
            ak.x = fmaf(kd, y.x, ak.x); ak.y = fmaf(kd, y.y, ak.y); ak.z = fmaf(kd, y.z, ak.z); ak.w = fmaf(kd, y.w, ak.w);
            aq.x = fmaf(qd, y.x, aq.x); aq.y = fmaf(qd, y.y, aq.y); aq.z = fmaf(qd, y.z, aq.z); aq.w = fmaf(qd, y.w, aq.w);
        };
        if (act) {
            if constexpr (RPT > 0) {
#pragma unroll
                for (int i = 0; i < R; ++i)
                    if (g + i * NG < dim) fold(x[i], g + i * NG);
            } else {
                for (int d = g; d < dim; d += NG) {
                    float4 y = pos > 0 ? *reinterpret_cast<const float4*>(S + (size_t)d * vdim + 4 * c) : make_float4(0.f, 0.f, 0.f, 0.f);
                    fold(y, d);
                    *reinterpret_cast<float4*>(S + (size_t)d * vdim + 4 * c) = y;
                }
            }
            *reinterpret_cast<float4*>(pk + g * vdim + 4 * c) = ak;
            *reinterpret_cast<float4*>(pq + g * vdim + 4 * c) = aq;
        }
        __syncthreads();
        float4 o = {0.f, 0.f, 0.f, 0.f};
        float ss = 0.f;
        if (act) {
            float4 r = {0.f, 0.f, 0.f, 0.f};
            for (int j = 0; j < NG; ++j) {
                const float4 p = *reinterpret_cast<const float4*>(pk + j * vdim + 4 * c);
                r.x += p.x; r.y += p.y; r.z += p.z; r.w += p.w;
            }
            const float4 vv = *reinterpret_cast<const float4*>(v + 4 * c);
            const float4 u = {beta * fmaf(-ik, r.x, vv.x), beta * fmaf(-ik, r.y, vv.y), beta * fmaf(-ik, r.z, vv.z), beta * fmaf(-ik, r.w, vv.w)};
            auto write = [&](float4& y, int d) {
                const float kd = ik * k[d];
                y.x = fmaf(kd, u.x, y.x); y.y = fmaf(kd, u.y, y.y); y.z = fmaf(kd, u.z, y.z); y.w = fmaf(kd, u.w, y.w);
            };
            if constexpr (RPT > 0) {
#pragma unroll
                for (int i = 0; i < R; ++i)
                    if (g + i * NG < dim) write(x[i], g + i * NG);
            } else {
                for (int d = g; d < dim; d += NG) {
                    float4 y = *reinterpret_cast<const float4*>(S + (size_t)d * vdim + 4 * c);
                    write(y, d);
                    *reinterpret_cast<float4*>(S + (size_t)d * vdim + 4 * c) = y;
                }
            }
            if (g == 0) {
                for (int j = 0; j < NG; ++j) {
                    const float4 p = *reinterpret_cast<const float4*>(pq + j * vdim + 4 * c);
                    o.x += p.x; o.y += p.y; o.z += p.z; o.w += p.w;
                }
                o.x = fmaf(kq, u.x, iq * o.x); o.y = fmaf(kq, u.y, iq * o.y); o.z = fmaf(kq, u.z, iq * o.z); o.w = fmaf(kq, u.w, iq * o.w);
                ss = o.x * o.x + o.y * o.y + o.z * o.z + o.w * o.w;
            }
        }
        const float inv = 1.0f / sqrtf(block_sum(ss, red) / a.vdim_true + a.eps);      // (its barriers end the reads of q .. pq)
        IT* out = reinterpret_cast<IT*>(a.out) + (size_t)(s.row0 + t) * a.ld_out;
        if (act && g == 0) {
            const float4 w = *reinterpret_cast<const float4*>(a.norm + 4 * c), z = load4<IT>(reinterpret_cast<const IT*>(a.gate) + (size_t)(s.row0 + t) * a.ld_gate + h * vdim + 4 * c);
            auto gated = [&](float y, float n, float e) { return y * inv * n / (1.0f + (EXACT ? expf(-e) : __expf(-e))); };
            store4<IT>(out + h * vdim + 4 * c, make_float4(gated(o.x, w.x, z.x), gated(o.y, w.y, z.y), gated(o.z, w.z, z.z), gated(o.w, w.w, z.w)));
        }
        if (h == a.H - 1)
            for (int i = a.H * vdim + tid; i < a.ld_out; i += NT) out[i] = from_f<IT>(0.f);
    }
    if constexpr (RPT > 0) {
#pragma unroll
        for (int i = 0; i < R; ++i)
            if (act && g + i * NG < dim) *reinterpret_cast<float4*>(S + (size_t)(g + i * NG) * vdim + 4 * c) = x[i];
    }
    tls.end();
}

template <class T, class IT, bool EXACT>
static pgk_status delta_scan(const DeltaArgs& a, hipStream_t st) {
    const int B = a.seqs ? a.n_seqs : a.n, threads = a.dim * a.vdim >= 8192 ? 512 : 256, cols = a.vdim / 4;
    PGK_REQUIRE(cols <= threads, "delta rule: head width %d", a.vdim);
    const int groups = threads / cols, rows = ceil_div(a.dim, groups);
    const size_t lds = (size_t)(3 * a.dim + a.vdim + 2 * groups * a.vdim) * 4;
    PGK_REQUIRE(lds <= 64 * 1024, "delta rule: head widths %d / %d do not fit LDS", a.dim, a.vdim);
    const dim3 grid(a.H, B);
#define PGK_DELTA(R) PGK_CHECK_HIP(launch_k(&delta_scan_kernel<T, IT, EXACT, R>, grid, dim3(threads), lds, st, a))
    if (rows <= 2) PGK_DELTA(2);
    else if (rows <= 4) PGK_DELTA(4);
    else if (rows <= 8) PGK_DELTA(8);
    else if (rows <= 16) PGK_DELTA(16);
    else PGK_DELTA(0);
#undef PGK_DELTA
    return PGK_OK;
}

pgk_status delta_rows(const DeltaArgs& a, pgk_dtype dt, bool io32, hipStream_t st) {
    PGK_REQUIRE(a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.dim >= 1 && a.vdim % 4 == 0 && a.ld_out >= a.H * a.vdim && a.ld_out % 4 == 0 && a.ld_gate % 4 == 0 &&
                    (a.seqs ? a.rows != nullptr : a.positions && a.conv.taps >= 1 && a.conv.ring), "delta rule: bad arguments");
    if (dt == PGK_F32) return delta_scan<float, float, true>(a, st);
    return io32 ? delta_scan<bf16, float, false>(a, st) : delta_scan<bf16, bf16, false>(a, st);
}

// -------------------------------------------------------------------------------------------- chunks
typedef float f32x4_dl __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4_dl mfma4d(float a, float b, f32x4_dl c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
// Four products in a row take k in the order 4 (lane >> 4) + step: a lane's four values of a row of the left operand are neighbours, and
// an accumulator tile (rows 4 (lane >> 4) + r, column lane & 15) is the right operand of the next product as it stands.
__device__ __forceinline__ f32x4_dl mfma16d(const float4& a, const f32x4_dl& b, f32x4_dl c) {
    c = mfma4d(a.x, b[0], c); c = mfma4d(a.y, b[1], c); c = mfma4d(a.z, b[2], c);
    return mfma4d(a.w, b[3], c);
}
__device__ __forceinline__ float4 ld4d(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 mul4d(const float4& a, const float4& b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }
__device__ __forceinline__ f32x4_dl vec4d(const float4& a) { return f32x4_dl{a.x, a.y, a.z, a.w}; }

constexpr int DC = DELTA_CHUNK, DNS = DC / 16, DAS = DC + 4, DTS = 20;
__host__ __device__ constexpr int dl_stride(int dim) { return dim + 4; }
static size_t delta_chunk_lds(int dim) { return ((size_t)3 * DC * dl_stride(dim) + 2 * DC * DAS + DNS * dim + DC) * 4; }
bool delta_chunk_ok(int dim, int vdim) { return (dim == 32 || dim == 64 || dim == 128) && vdim % 16 == 0; }

// workspace of one (chunk, head): -W [64][dim], q G [64][dim], (k G_end)^T [dim][64], X [64][vdim], B [64][64], G_end [dim]
struct DeltaRec {
    float *W, *Q, *KT, *X, *B, *D;
    __host__ __device__ static size_t size(int dim, int vdim) { return (size_t)DC * (3 * dim + vdim + DC) + dim; }
    __device__ DeltaRec(float* p, int dim, int vdim) : W(p), Q(W + DC * dim), KT(Q + DC * dim), X(KT + DC * dim), B(X + DC * vdim), D(B + DC * DC) {}
};
size_t delta_chunk_bytes(const DeltaArgs& a, int n_chunks) { return (size_t)n_chunks * a.H * DeltaRec::size(a.dim, a.vdim) * 4; }

// 1.  Eight waves.
template <class T, int DIM>
__global__ __launch_bounds__(512) void delta_chunk_kernel(DeltaArgs a, const RecurChunk* chunks, float* ws) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    constexpr int S = dl_stride(DIM), P = DIM / 32;                // pieces of four channels per thread and row
    const int vdim = a.vdim, h = blockIdx.x, kh = h / (a.H / a.G);
    float *q = sm, *f = q + DC * S, *k = f + DC * S, *Aq = k + DC * S, *Ak = Aq + DC * DAS, *F = Ak + DC * DAS, *beta = F + DNS * DIM;
    const RecurChunk ch = chunks[blockIdx.y];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4, last = ch.len - 1;
    const DeltaRec rec(ws + ((size_t)blockIdx.y * a.H + h) * DeltaRec::size(DIM, vdim), DIM, vdim);
    const T* rows = reinterpret_cast<const T*>(a.rows) + (size_t)ch.row0 * a.ld_rows;
    {   // eight lanes per row: unit q and k, decays; rows past the end are zero with decay one
        const int r = tid >> 3, l = tid & 7, rr = min(r, last);
        const bool live = r <= last;
        const T* row = rows + (size_t)rr * a.ld_rows + kh * DIM;
        const float* zr = a.z + (size_t)(ch.row0 + rr) * a.ld_z + h * DIM;
        const float* db = a.dt_bias + h * DIM;
        float4 vq[P], vk[P], vz[P], vb[P];
#pragma unroll
        for (int i = 0; i < P; ++i) {
            const int c = 4 * (l + 8 * i);
            vq[i] = load4<T>(row + c); vk[i] = load4<T>(row + a.G * DIM + c); vz[i] = ld4d(zr + c); vb[i] = ld4d(db + c);
        }
        float sq = 0.f, sk = 0.f;
#pragma unroll
        for (int i = 0; i < P; ++i) {
            sq += vq[i].x * vq[i].x + vq[i].y * vq[i].y + vq[i].z * vq[i].z + vq[i].w * vq[i].w;
            sk += vk[i].x * vk[i].x + vk[i].y * vk[i].y + vk[i].z * vk[i].z + vk[i].w * vk[i].w;
        }
        const float iq = live ? 1.0f / sqrtf((float)a.dim_true) / sqrtf(group8_sum(sq) + UNIT_EPS) : 0.f, ik = live ? 1.0f / sqrtf(group8_sum(sk) + UNIT_EPS) : 0.f, dec = live ? a.decay[h] : 0.f;
#pragma unroll
        for (int i = 0; i < P; ++i) {
            const int c = 4 * (l + 8 * i);
            *reinterpret_cast<float4*>(q + r * S + c) = make_float4(vq[i].x * iq, vq[i].y * iq, vq[i].z * iq, vq[i].w * iq);
            *reinterpret_cast<float4*>(k + r * S + c) = make_float4(vk[i].x * ik, vk[i].y * ik, vk[i].z * ik, vk[i].w * ik);
            *reinterpret_cast<float4*>(f + r * S + c) = make_float4(delta_fade(vz[i].x, vb[i].x, dec), delta_fade(vz[i].y, vb[i].y, dec), delta_fade(vz[i].z, vb[i].z, dec),
                                                                    delta_fade(vz[i].w, vb[i].w, dec));
        }
        if (l == 0) beta[r] = live ? 1.0f / (1.0f + expf(-to_f(reinterpret_cast<const T*>(a.in)[(size_t)(ch.row0 + rr) * a.ld_in + a.b_off + h]))) : 0.f;
    }
    __syncthreads();
    {   // diagonal blocks, pair by pair: two waves per block, rows 0..7 and 8..15.  Lane: column j = lane & 7 (and j + 8), every eighth group
        // of 4 channels; w = k_j times the decay from j to the row at hand.
        const int b = wid >> 1, r0 = 16 * b, half = (wid ^ (wid >> 2)) & 1, jl = lane & 7, dg = lane >> 3;
        float lo[8], hi[8], lk[8], hk[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) lo[i] = hi[i] = lk[i] = hk[i] = 0.f;
        for (int c = 4 * dg; c < DIM; c += 32) {
            auto row4 = [&](const float* p, float (&x)[4]) { const float4 u = ld4d(p); x[0] = u.x; x[1] = u.y; x[2] = u.z; x[3] = u.w; };
            float wl[4], wh[4];
            row4(k + (r0 + jl) * S + c, wl);
            if (half) {
                row4(k + (r0 + 8 + jl) * S + c, wh);
#pragma unroll
                for (int i = 1; i < 8; ++i) {
                    float g[4];
                    row4(f + (r0 + i) * S + c, g);
#pragma unroll
                    for (int e = 0; e < 4; ++e) wl[e] *= i > jl ? g[e] : 1.f;
                }
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                float g[4], x[4], y[4];
                const int row = r0 + 8 * half + i;
                row4(f + row * S + c, g);
                row4(q + row * S + c, x);
                row4(k + row * S + c, y);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (half) {
                        wl[e] *= g[e];
                        wh[e] *= i > jl ? g[e] : 1.f;
                        hi[i] = fmaf(x[e], wh[e], hi[i]);
                        hk[i] = fmaf(y[e], wh[e], hk[i]);
                    } else wl[e] *= i > jl ? g[e] : 1.f;
                    lo[i] = fmaf(x[e], wl[e], lo[i]);
                    lk[i] = fmaf(y[e], wl[e], lk[i]);
                }
            }
        }
        auto sum = [](float x) { x += dpp_f<DPP_ROR8>(x); x += __shfl_xor(x, 16, 64); return x + __shfl_xor(x, 32, 64); };
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float x = sum(lo[i]), y = sum(hi[i]), u = sum(lk[i]), w = sum(hk[i]);
            const int row = r0 + 8 * half + i;
            if (dg == 0) {
                Aq[row * DAS + r0 + jl] = half || i >= jl ? x : 0.f;
                Aq[row * DAS + r0 + 8 + jl] = half && i >= jl ? y : 0.f;
                Ak[row * DAS + r0 + jl] = half || i > jl ? beta[row] * u : 0.f;
                Ak[row * DAS + r0 + 8 + jl] = half && i > jl ? beta[row] * w : 0.f;
            }
        }
    }
    __syncthreads();
    // q and k times the decay from their block's start (their own row included; k's copy takes the place of the decays), k times the decay to its block's end
    for (int t = tid; t < DNS * DIM; t += 512) {
        const int b = t / DIM, d = t % DIM;
        float g[16], kk[16], run = 1.f;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int at = (16 * b + r) * S + d;
            g[r] = f[at];
            kk[r] = k[at];
            run *= g[r];
            q[at] *= run;
            f[at] = kk[r] * run;
        }
        F[b * DIM + d] = run;
        run = 1.f;
#pragma unroll
        for (int r = 15; r >= 0; --r) {
            k[(16 * b + r) * S + d] = kk[r] * run;
            run *= g[r];
        }
    }
    __syncthreads();
    // blocks below the diagonal: six of B, six of A
    for (int p = wid; p < 12; p += 8) {
        const bool isk = p >= 6;
        int bi = 1, bj = isk ? p - 6 : p;
        while (bj >= bi) { bj -= bi; ++bi; }
        const float* left = (isk ? f : q) + (16 * bi + l15) * S;
        f32x4_dl acc[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) acc[u] = f32x4_dl{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int d0 = 0; d0 < DIM; d0 += 16) {
            const int d = d0 + 4 * q4;
            float4 x = ld4d(left + d);
            const float4 y = ld4d(k + (16 * bj + l15) * S + d);
            if (bj + 1 < bi) x = mul4d(x, ld4d(F + (bj + 1) * DIM + d));
            if (bj + 2 < bi) x = mul4d(x, ld4d(F + (bj + 2) * DIM + d));      // (four blocks: at most two between)
            acc[0] = mfma4d(x.x, y.x, acc[0]); acc[1] = mfma4d(x.y, y.y, acc[1]);
            acc[2] = mfma4d(x.z, y.z, acc[2]); acc[3] = mfma4d(x.w, y.w, acc[3]);
        }
        float* dst = isk ? Ak : Aq;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * bi + 4 * q4 + r;
            dst[row * DAS + 16 * bj + l15] = ((acc[0][r] + acc[1][r]) + (acc[2][r] + acc[3][r])) * (isk ? beta[row] : 1.f);
        }
    }
    // 16 x 16 inverses of the diagonal blocks of I + A, a lane per column (they take the unused upper right corner of B: rows 16 b ..,
    // columns 48 .. of blocks 0..2, and for block 3 rows 0 .., columns 32 ..)
    float* Ti = Aq + (wid < 3 ? 16 * wid * DAS + 48 : 32);
    if (wid < DNS) {
        float x[16];
        const float* A = Ak + (16 * wid) * DAS + 16 * wid;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float t = i == l15 ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; ++j) t = fmaf(-A[i * DAS + j], x[j], t);
            x[i] = t;
        }
        if (q4 == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) Ti[i * DAS + l15] = x[i];
        }
    }
    __syncthreads();
    // substitution, 16 columns at a time: tiles of b v, then of b (k G)
    const int nv = vdim / 16, nt = nv + DIM / 16;
    for (int t = wid; t < nt; t += 8) {
        const bool isv = t < nv;
        const int col = 16 * (isv ? t : t - nv) + l15;
        f32x4_dl x[DNS];
        if (isv) {
            const T* vr = rows + 2 * a.G * DIM + h * vdim + col;
#pragma unroll
            for (int i = 0; i < DNS; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int row = 16 * i + 4 * q4 + r;
                    x[i][r] = beta[row] * to_f(vr[(size_t)min(row, last) * a.ld_rows]);
                }
        } else {
            float m = 1.f;
#pragma unroll
            for (int i = 0; i < DNS; ++i) {
#pragma unroll
                for (int r = 0; r < 4; ++r) { const int row = 16 * i + 4 * q4 + r; x[i][r] = beta[row] * f[row * S + col] * m; }
                m *= F[i * DIM + col];
            }
        }
#pragma unroll
        for (int i = 0; i < DNS; ++i) {
            f32x4_dl s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < i; ++j) s = mfma16d(ld4d(Ak + (16 * i + l15) * DAS + 16 * j + 4 * q4), x[j], s);
#pragma unroll
            for (int r = 0; r < 4; ++r) x[i][r] -= s[r];
            x[i] = mfma16d(ld4d(Aq + (i < 3 ? 16 * i * DAS + 48 : 32) + l15 * DAS + 4 * q4), x[i], f32x4_dl{0.f, 0.f, 0.f, 0.f});
        }
        float* dst = isv ? rec.X : rec.W;
        const int ld = isv ? vdim : DIM;
#pragma unroll
        for (int i = 0; i < DNS; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[(size_t)(16 * i + 4 * q4 + r) * ld + col] = isv ? x[i][r] : -x[i][r];
    }
    // q G, (k G_end)^T, G_end, B
    for (int t = tid; t < DC * DIM / 4; t += 512) {
        const int r = t / (DIM / 4), c = t % (DIM / 4) * 4;
        float4 y = ld4d(q + r * S + c);
        for (int b = 0; b < r / 16; ++b) y = mul4d(y, ld4d(F + b * DIM + c));
        *reinterpret_cast<float4*>(rec.Q + r * DIM + c) = y;
    }
    for (int t = tid; t < DIM * DC / 4; t += 512) {
        const int d = t / (DC / 4), r = t % (DC / 4) * 4;
        float m = 1.f;
        for (int b = r / 16 + 1; b < DNS; ++b) m *= F[b * DIM + d];
        *reinterpret_cast<float4*>(rec.KT + d * DC + r) = make_float4(k[r * S + d] * m, k[(r + 1) * S + d] * m, k[(r + 2) * S + d] * m, k[(r + 3) * S + d] * m);
    }
    for (int d = tid; d < DIM; d += 512) rec.D[d] = F[d] * F[DIM + d] * F[2 * DIM + d] * F[3 * DIM + d];
    for (int t = tid; t < DC * DC / 4; t += 512) {
        const int r = t / (DC / 4), c = t % (DC / 4) * 4;
        if (c / 16 <= r / 16) *reinterpret_cast<float4*>(rec.B + r * DC + c) = ld4d(Aq + r * DAS + c);      // (the rest is never read)
    }
}

// 2.  Four waves; a workgroup has 16 columns of one head's state.  A wave computes 16 rows of U and o and DIM / 64 row tiles of the state
// (or waves 0, 1 one each); U and the state go round through LDS, transposed.  A chunk's operands travel during the chunk before.
template <class T, int DIM>
__global__ __launch_bounds__(256) void delta_scan_chunks_kernel(DeltaArgs a, const RecurChunk* chunks, const int32_t* chunk_of_seq, float* ws) {
    constexpr int DT = DIM / 16, MY = DT >= 4 ? DT / 4 : 1;
    __shared__ __attribute__((aligned(16))) float Us[16][DC + 4], Ss[16][DIM + 4];
    const int vdim = a.vdim, h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4, col = 16 * blockIdx.y + l15;
    const SeqSpan s = a.seqs[blockIdx.z];
    const int c0 = chunk_of_seq[blockIdx.z], c1 = chunk_of_seq[blockIdx.z + 1];
    const bool own = wid * MY < DT;                                // wave-uniform
    const int dt0 = own ? wid * MY : 0;
    float* st = a.state + ((size_t)s.slot * a.H + h) * DIM * vdim;
    f32x4_dl S[DT], mine[MY];
#pragma unroll
    for (int t = 0; t < DT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] = s.start > 0 ? st[(size_t)(16 * t + 4 * q4 + r) * vdim + col] : 0.f;
#pragma unroll
    for (int i = 0; i < MY; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) mine[i][r] = s.start > 0 ? st[(size_t)(16 * (dt0 + i) + 4 * q4 + r) * vdim + col] : 0.f;
    float4 w[DT], qg[DT], bb[DNS], kt[MY][DNS], dd[MY];
    float x[4];
    auto fetch = [&](int c) {
        const DeltaRec rec(ws + ((size_t)c * a.H + h) * DeltaRec::size(DIM, vdim), DIM, vdim);
        const int row = 16 * wid + l15;
#pragma unroll
        for (int r = 0; r < 4; ++r) x[r] = rec.X[(size_t)(16 * wid + 4 * q4 + r) * vdim + col];
#pragma unroll
        for (int t = 0; t < DT; ++t) w[t] = ld4d(rec.W + row * DIM + 16 * t + 4 * q4);
#pragma unroll
        for (int t = 0; t < DT; ++t) qg[t] = ld4d(rec.Q + row * DIM + 16 * t + 4 * q4);
#pragma unroll
        for (int j = 0; j < DNS; ++j) bb[j] = ld4d(rec.B + row * DC + 16 * min(j, wid) + 4 * q4);
#pragma unroll
        for (int i = 0; i < MY; ++i) {
            dd[i] = ld4d(rec.D + 16 * (dt0 + i) + 4 * q4);
#pragma unroll
            for (int j = 0; j < DNS; ++j) kt[i][j] = ld4d(rec.KT + (16 * (dt0 + i) + l15) * DC + 16 * j + 4 * q4);
        }
    };
    T* out = reinterpret_cast<T*>(a.out) + h * vdim + col;
    if (c0 < c1) fetch(c0);
    for (int c = c0; c < c1; ++c) {
        const RecurChunk ch = chunks[c];
        f32x4_dl u = {x[0], x[1], x[2], x[3]}, u2 = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < DT; t += 2) {
            u = mfma16d(w[t], S[t], u);
            u2 = mfma16d(w[t + 1], S[t + 1], u2);
            o = mfma16d(qg[t], S[t], o);
            o2 = mfma16d(qg[t + 1], S[t + 1], o2);
        }
        *reinterpret_cast<float4*>(&Us[l15][16 * wid + 4 * q4]) = make_float4(u[0] + u2[0], u[1] + u2[1], u[2] + u2[2], u[3] + u2[3]);
        float4 bc[DNS], kc[MY][DNS];
#pragma unroll
        for (int j = 0; j < DNS; ++j) bc[j] = bb[j];
#pragma unroll
        for (int i = 0; i < MY; ++i) {
            mine[i][0] *= dd[i].x; mine[i][1] *= dd[i].y; mine[i][2] *= dd[i].z; mine[i][3] *= dd[i].w;
#pragma unroll
            for (int j = 0; j < DNS; ++j) kc[i][j] = kt[i][j];
        }
        fetch(min(c + 1, c1 - 1));
        __syncthreads();
        f32x4_dl ub[DNS];
#pragma unroll
        for (int j = 0; j < DNS; ++j) ub[j] = vec4d(*reinterpret_cast<const float4*>(&Us[l15][16 * j + 4 * q4]));
#pragma unroll
        for (int j = 0; j < DNS; ++j) {
            if (own) {
#pragma unroll
                for (int i = 0; i < MY; ++i) mine[i] = mfma16d(kc[i][j], ub[j], mine[i]);
            }
            if (j <= wid) o = mfma16d(bc[j], ub[j], o);            // wave-uniform
        }
        if (own) {
#pragma unroll
            for (int i = 0; i < MY; ++i) *reinterpret_cast<float4*>(&Ss[l15][16 * (dt0 + i) + 4 * q4]) = make_float4(mine[i][0], mine[i][1], mine[i][2], mine[i][3]);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * wid + 4 * q4 + r;
            if (row < ch.len) out[(size_t)(ch.row0 + row) * a.ld_out] = from_f<T>(o[r] + o2[r]);
        }
        __syncthreads();
#pragma unroll
        for (int t = 0; t < DT; ++t) S[t] = vec4d(*reinterpret_cast<const float4*>(&Ss[l15][16 * t + 4 * q4]));
    }
    if (own) {
#pragma unroll
        for (int i = 0; i < MY; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) st[(size_t)(16 * (dt0 + i) + 4 * q4 + r) * vdim + col] = mine[i][r];
    }
}

// 3.  A wave per (row, head)
template <class T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(DeltaArgs a) {
    constexpr bool EXACT = std::is_same<T, float>::value;
    const long long i = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63, h = (int)(i % a.H);
    const long long row = i / a.H;
    if (row >= a.n) return;
    T* o = reinterpret_cast<T*>(a.out) + row * a.ld_out + h * a.vdim;
    const T* gate = reinterpret_cast<const T*>(a.gate) + row * a.ld_gate + h * a.vdim;
    auto go = [&](auto keep) {
        constexpr int K = decltype(keep)::value;                   // pieces of four columns a lane keeps (0: read twice)
        float4 v[K > 0 ? K : 1], z[K > 0 ? K : 1];
        float ss = 0.f;
        if constexpr (K > 0) {
#pragma unroll
            for (int k = 0; k < K; ++k) { const int c = min(4 * (lane + 64 * k), a.vdim - 4); v[k] = load4<T>(o + c); z[k] = load4<T>(gate + c); }
#pragma unroll
            for (int k = 0; k < K; ++k) if (4 * (lane + 64 * k) < a.vdim) ss += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
        } else
            for (int c = 4 * lane; c < a.vdim; c += 256) { const float4 y = load4<T>(o + c); ss += y.x * y.x + y.y * y.y + y.z * y.z + y.w * y.w; }
        const float inv = 1.0f / sqrtf(wave_sum(ss) / a.vdim_true + a.eps);
        auto put = [&](int c, const float4& y, const float4& e) {
            const float4 w = *reinterpret_cast<const float4*>(a.norm + c);
            auto g = [](float t) { return 1.0f / (1.0f + (EXACT ? expf(-t) : __expf(-t))); };
            store4<T>(o + c, make_float4(y.x * inv * w.x * g(e.x), y.y * inv * w.y * g(e.y), y.z * inv * w.z * g(e.z), y.w * inv * w.w * g(e.w)));
        };
        if constexpr (K > 0) {
#pragma unroll
            for (int k = 0; k < K; ++k) if (4 * (lane + 64 * k) < a.vdim) put(4 * (lane + 64 * k), v[k], z[k]);
        } else
            for (int c = 4 * lane; c < a.vdim; c += 256) put(c, load4<T>(o + c), load4<T>(gate + c));
    };
    if (a.vdim <= 256) go(std::integral_constant<int, 1>{});
    else go(std::integral_constant<int, 0>{});
    if (h == a.H - 1)
        for (int c = a.H * a.vdim + lane; c < a.ld_out; c += 64) reinterpret_cast<T*>(a.out)[row * a.ld_out + c] = from_f<T>(0.f);
}

template <class T, int DIM>
static pgk_status delta_chunked_t(const DeltaArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, float* ws, hipStream_t st) {
    const size_t lds = delta_chunk_lds(DIM);
    static bool done = false;
    if (lds > 48 * 1024 && !done) {
        PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_chunk_kernel<T, DIM>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        done = true;
    }
    delta_chunk_kernel<T, DIM><<<dim3(a.H, n_chunks), 512, lds, st>>>(a, chunks, ws);
    PGK_LAUNCH_CHECK();
    delta_scan_chunks_kernel<T, DIM><<<dim3(a.H, a.vdim / 16, a.n_seqs), 256, 0, st>>>(a, chunks, chunk_of_seq, ws);
    PGK_LAUNCH_CHECK();
    head_norm_gate_kernel<T><<<ceil_div((long long)a.n * a.H, 4), 256, 0, st>>>(a);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

pgk_status delta_chunked(const DeltaArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, void* ws, pgk_dtype dt, hipStream_t st) {
    PGK_REQUIRE(delta_chunk_ok(a.dim, a.vdim) && a.G >= 1 && a.H % a.G == 0 && a.seqs && a.rows && n_chunks >= 1 && n_chunks <= 65535 && a.n_seqs <= 65535 && a.ld_out >= a.H * a.vdim && a.ld_out % 4 == 0 &&
                    a.ld_rows % 4 == 0 && a.ld_z % 4 == 0 && a.ld_gate % 4 == 0, "delta rule: %d chunks of head widths %d / %d", n_chunks, a.dim, a.vdim);
#define PGK_DELTA(T) (a.dim == 32 ? delta_chunked_t<T, 32>(a, chunks, n_chunks, chunk_of_seq, (float*)ws, st) : a.dim == 64 ? delta_chunked_t<T, 64>(a, chunks, n_chunks, chunk_of_seq, (float*)ws, st) \
                                                                                                     : delta_chunked_t<T, 128>(a, chunks, n_chunks, chunk_of_seq, (float*)ws, st))
    return dt == PGK_F32 ? PGK_DELTA(float) : PGK_DELTA(bf16);
#undef PGK_DELTA
}

// -------------------------------------------------------------------------------------------- low-rank projections of a few rows
// 16 lanes per output, every workgroup 16 x 4 outputs of one row; the outputs of A first, then those of G
template <class T, class IT>
__global__ __launch_bounds__(256) void lowrank_kernel(unsigned long long* tl, const IT* in, int ld_in, int a_off, int ka, const T* wa, float* z, int na, int g_off, int kg, const T* wg, IT* g, int ng) {
    const TLStamp tls(tl);
    constexpr int NW = WTraits<T>::NW;
    const int sub = threadIdx.x & 15, grp = threadIdx.x >> 4, row = blockIdx.y;
    const IT* x = in + (size_t)row * ld_in;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int o = blockIdx.x * 64 + i * 16 + grp;
        const bool isa = o < na;
        const int j = min(isa ? o : o - na, (isa ? na : ng) - 1), K = isa ? ka : kg;
        const T* w = (isa ? wa : wg) + (size_t)j * K;
        const IT* xr = x + (isa ? a_off : g_off);
        float acc = 0.f;
        for (int k = sub * NW; k < K; k += 16 * NW) {
            float f[NW];
            WTraits<T>::decode(*reinterpret_cast<const uint4*>(w + k), f);
#pragma unroll
            for (int e = 0; e < NW; e += 4) {
                const float4 v = load4<IT>(xr + k + e);
                acc = fmaf(f[e], v.x, acc); acc = fmaf(f[e + 1], v.y, acc); acc = fmaf(f[e + 2], v.z, acc); acc = fmaf(f[e + 3], v.w, acc);
            }
        }
        acc = group16_sum(acc);
        if (sub == 0 && o < na + ng) {
            if (isa) z[(size_t)row * na + o] = acc;
            else g[(size_t)row * ng + o - na] = from_f<IT>(acc);
        }
    }
    tls.end();
}

pgk_status lowrank_rows(const void* in, int ld_in, int n, int a_off, int ka, const void* wa, float* z, int na, int g_off, int kg, const void* wg, void* g, int ng,
                        pgk_dtype dt, bool io32, hipStream_t st) {
    PGK_REQUIRE(n >= 1 && ka % 8 == 0 && kg % 8 == 0 && ld_in % 4 == 0 && a_off % 4 == 0 && g_off % 4 == 0, "lowrank_rows: ranks %d / %d", ka, kg);
    const dim3 grid(ceil_div(na + ng, 64), n);
    if (dt == PGK_F32) PGK_CHECK_HIP(launch_k(&lowrank_kernel<float, float>, grid, dim3(256), 0, st, (const float*)in, ld_in, a_off, ka, (const float*)wa, z, na, g_off, kg, (const float*)wg, (float*)g, ng));
    else if (io32) PGK_CHECK_HIP(launch_k(&lowrank_kernel<bf16, float>, grid, dim3(256), 0, st, (const float*)in, ld_in, a_off, ka, (const bf16*)wa, z, na, g_off, kg, (const bf16*)wg, (float*)g, ng));
    else PGK_CHECK_HIP(launch_k(&lowrank_kernel<bf16, bf16>, grid, dim3(256), 0, st, (const bf16*)in, ld_in, a_off, ka, (const bf16*)wa, z, na, g_off, kg, (const bf16*)wg, (bf16*)g, ng));
    return PGK_OK;
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_delta_rule(const void* q, const void* k, const void* v, const float* z, const void* strength, const void* gate, const float* decay, const float* step_bias,
                          const float* norm, float* state, void* out, int n, int fresh, int heads, int kv_heads, int dim, int vdim, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(q && k && v && z && strength && gate && decay && step_bias && norm && state && out, "pgk_delta_rule: null pointer");
    PGK_REQUIRE(n >= 1 && heads >= 1 && kv_heads >= 1 && heads % kv_heads == 0 && dim >= 1 && vdim >= 1, "pgk_delta_rule: bad shape %d / %d x %d x %d, %d rows",
                heads, kv_heads, dim, vdim, n);
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_delta_rule: dtype %d (bf16 or f32)", (int)dt);
    hipStream_t st = resolve_stream(s);
    // one row buffer q | k | v, the tables and the chunked form's workspace behind it; head widths that are no multiple of 4 run as copies
    // with zeros behind every head
    const int dp = ceil_div(dim, 4) * 4, vp = ceil_div(vdim, 4) * 4;
    const bool pad = dp != dim || vp != vdim;
    const size_t E = dtype_size(dt), wq = (size_t)kv_heads * dp * E, wv = (size_t)heads * vp * E, row = 2 * wq + wv, wz = (size_t)heads * dp * 4;
    const size_t d = (size_t)dim * E, v1 = (size_t)vdim * E;
    auto up = [](size_t b) { return (b + 255) & ~(size_t)255; };
    DeltaArgs a{};
    a.in = strength; a.ld_in = heads; a.ld_rows = (int)(row / E); a.z = z; a.ld_z = heads * dp; a.gate = gate; a.ld_gate = heads * vp;
    a.decay = decay; a.dt_bias = step_bias; a.norm = norm; a.H = heads; a.G = kv_heads; a.dim = dp; a.dim_true = dim; a.vdim = vp; a.vdim_true = vdim; a.n = n; a.eps = eps;
    a.state = state; a.n_seqs = 1; a.out = out; a.ld_out = heads * vp;
    const int C = n >= RECUR_CHUNKED_FROM && delta_chunk_ok(dp, vp) ? DELTA_CHUNK : 0, nch = C ? ceil_div(n, C) : 0;
    std::vector<RecurChunk> chunks;
    for (int c = 0; c < nch; ++c) chunks.push_back(RecurChunk{c * C, n - c * C < C ? n - c * C : C});
    const int32_t of_seq[2] = {0, nch};
    const SeqSpan span{0, n, fresh ? 0 : 1, 0};
    size_t at = 0;
    auto take = [&](size_t b) { const size_t o = at; at += up(b); return o; };
    const size_t o_rows = take(n * row), o_z = take(pad ? n * wz : 0), o_gate = take(pad ? n * wv : 0), o_out = take(pad ? n * wv : 0), o_bias = take(pad ? wz : 0), o_norm = take(pad ? vp * 4 : 0),
                 o_state = take(pad ? wz * vp : 0), zeroed = at, o_span = take(sizeof(span)), o_of = take(sizeof(of_seq)), o_ch = take(nch * sizeof(RecurChunk)), o_ws = take(nch ? delta_chunk_bytes(a, nch) : 0);
    char* ws = nullptr;
    if (pgk_status r = pgk_malloc((void**)&ws, at + 256)) return r;
    hipError_t e = pad ? hipMemsetAsync(ws, 0, zeroed, st) : hipSuccess;
    const size_t fd = (size_t)dim * 4, fv = (size_t)vdim * 4, fdp = (size_t)dp * 4, fvp = (size_t)vp * 4;
    auto copy = [&](size_t dst, size_t ld_dst, size_t p_dst, const void* src, size_t p_src, size_t rows, int nh) {
        if (e == hipSuccess) e = copy_heads(ws + dst, ld_dst, p_dst, src, nh * p_src, p_src, rows, nh, st);
    };
    copy(o_rows, row, dp * E, q, d, n, kv_heads);
    copy(o_rows + wq, row, dp * E, k, d, n, kv_heads);
    copy(o_rows + 2 * wq, row, vp * E, v, v1, n, heads);
    if (pad) {
        copy(o_z, wz, fdp, z, fd, n, heads);
        copy(o_gate, wv, vp * E, gate, v1, n, heads);
        copy(o_bias, wz, fdp, step_bias, fd, 1, heads);
        copy(o_norm, fvp, fvp, norm, fv, 1, 1);
        for (int h = 0; h < heads; ++h) copy(o_state + h * dp * fvp, fvp, fvp, state + (size_t)h * dim * vdim, fv, dim, 1);
        a.z = (const float*)(ws + o_z); a.gate = ws + o_gate; a.dt_bias = (const float*)(ws + o_bias); a.norm = (const float*)(ws + o_norm);
        a.state = (float*)(ws + o_state); a.out = ws + o_out;
    }
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_span, &span, sizeof(span), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_of, of_seq, sizeof(of_seq), hipMemcpyHostToDevice, st);
    if (e == hipSuccess && nch) e = hipMemcpyAsync(ws + o_ch, chunks.data(), nch * sizeof(RecurChunk), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    a.rows = ws + o_rows; a.seqs = (const SeqSpan*)(ws + o_span);
    pgk_status r = PGK_OK;
    if (e == hipSuccess) r = nch ? delta_chunked(a, (const RecurChunk*)(ws + o_ch), nch, (const int32_t*)(ws + o_of), ws + o_ws, dt, st) : delta_rows(a, dt, dt == PGK_F32, st);
    if (pad && e == hipSuccess && r == PGK_OK) {
        e = copy_heads(out, heads * v1, v1, ws + o_out, wv, vp * E, n, heads, st);
        for (int h = 0; h < heads && e == hipSuccess; ++h) e = copy_heads(state + (size_t)h * dim * vdim, fv, fv, ws + o_state + h * dp * fvp, fvp, fvp, dim, 1, st);
    }
    if (e != hipSuccess) r = set_error(PGK_ERR_HIP, "pgk_delta_rule: %s", hipGetErrorString(e));
    pgk_free(ws);       // stream-ordered reuse
    return r;
}

}  // extern "C"
