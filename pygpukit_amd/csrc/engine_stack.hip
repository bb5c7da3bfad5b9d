// Native engine for layer-list decoders: an fp32 residual stream; every layer has its own mixer and its own sizes.  Elements are bf16
// (fp32 stream, norms, scores, softmax, routers, recurrent states) or fp32 throughout.
//
// Sandwich layers: RMSNorm rho after each sublayer and, where a layer has one, before it; a dense feed-forward (SwiGLU or xIELU) or none
//   x   <- x + m * rho(O mixer(h); n1b),            h = rho(x; n1) or x
//   x   <- x + m * rho(W_d act(W_u h); n2b),        h = rho(x; n2) or x
// Parallel layers: one norm (RMS or layer norm), a mixture of experts (moe.hip.h) or no feed-forward
//   x   <- x + m * (O mixer(h) + moe(h)),           h = nu(x; n1)
// Hyper-connected layers: s streams instead of one (hyper.hip.h), norms in groups; dense feed-forwards with a polynomial-norm activation
// (W_d p(W_u h)) or experts that a table of token ids chooses, beside a gated shared one
//   u = sum_a c_a x_a,   y = F(nu(u)),   x_b <- sum_a M_ab x_a + d_b y      for F the mixer, then the feed-forward
// A stretch of layers may run several times over with the same weights (`Run`: one pass of one layer, with a cache of its own); pass t
// starts with  x <- L [x; embedding] + s_t.
//
// Mixers (pgk_mixer):
//   latent attention  sigmoid(G h) * attention(Q h, c),  c = rms(D h) * w_c,  k = U_k c,  v = U_v c: over a sliding window; the cache holds
//                     one normalised latent row per token, not keys and values.  A latent row may end in columns that are turned by the
//                     position instead (the rotary part of the key, one for all heads).  The kernels are in this file.
//   attention         taps over time and norms on q, k, v, a K/V ring (which another layer may own), distance bias, elementwise gate:
//                     ops_gated_attn.hip
//   talk              norms per head and rotation, a K/V ring over a window or chunk, mixed scores, a sink: ops_talk.hip
//   hgrn2, ssd        linear recurrences with an fp32 state per sequence and head: ops_recurrence.hip
//   delta             gated delta rule with a decay per key channel: ops_delta.hip
// In a step a mixer takes the in-projection row(s) and leaves the rows that the out-projection multiplies.
//
// Latent cache: per layer [slot][R][rank] latents, R = min(window, max_seq_len); position p lives in row p mod R, so a full ring IS the
// window and a decode step needs no mask.  Keys and values are never stored: decode folds U_k into the query (q_lat = U_k^T q, scores
// q_lat . c) and applies U_v to the probability-weighted latent sum, prefill expands the latents it needs into a scratch K | V.
//
// Decode of a latent layer, one sequence (fp32 between kernels):
//   in_proj    [pending: x += m rho(y; n2b)] q | latent | gate = W_in . rho(x; n1)
//   absorb     q_lat = scale log2e U_k^T q per head;  the new latent row -> ring
//   attn       split over the ring: scores, softmax, sum p c  -> partial records
//   merge_uv   combine the records, U_v, head gate
//   oproj      y = O a
//   gateup     x += m rho(y; n1b);  act = silu(g) * u of rho(x; n2)
//   down       y = W_d act
// The reduction a post-norm needs over the whole sublayer output is done in the NEXT kernel's prologue, by every workgroup for itself
// (one row: a few KB from L2), so it costs no launch.
// A parallel layer, one sequence: in_proj (pending add, norm; router logits are rows of the same matrix), the mixer, moe_up (choice,
// SwiGLU of the chosen experts), out (W_o and the chosen experts' down projections as one product).
// A hyper-connected layer, one sequence: in_proj (pending update of the streams, their combination and norm in the prologue), head norms and
// rotation, attn, merge, oproj (+ bias), up, down (activation in the prologue; experts: the chosen ones and the shared one in one launch).
// Several sequences and prompts: the same kernels on rows, the norms as a launch of their own and the projections on the GEMM family
// (pgk_gemm_nt: GEMV up to 8 rows, weight-streaming MFMA up to 128, tiled MFMA beyond).
// All widths are padded with zeros by the caller: every K is a multiple of 64, head widths are 64, 128 or a larger multiple of 64.

#include <algorithm>
#include <cstring>

#include "engine_state.hip.h"
#include "gemm_epilogues.hip.h"
#include "hyper.hip.h"
#include "latent.hip.h"
#include "mixers.hip.h"
#include "moe.hip.h"
#include "pkgemm.hip.h"

namespace pgk {

pgk_status wsgemm_nt(const bf16* a, int lda, const void* w, const bf16* wscale, bool fp8, void* c, const bf16* bias, int mode,
                     int splits, int M, int N, int K, hipStream_t st);
bool engine_gemm_swiglu_ok(int M, int I, int K, bool fp8);     // ops_gemm.hip
pgk_status engine_gemm_swiglu_nt(const bf16* A, const void* W, const bf16* wscale, bool fp8, bf16* act, int M, int I, int K, hipStream_t st, bool packed = false);

bool engine_gemm_act_ok(int M, int N, int K);                  // ops_gemm.hip
pgk_status engine_gemm_act_nt(const bf16* A, const bf16* W, bf16* act, int M, int N, int K, const ActArgs& xa, hipStream_t st);

int wsgemm_pick_splits(int N, int K, bool allow_split);        // ops_wsgemm.hip
int engine_gemm_pick_splits(int M, int N, int K);              // ops_gemm.hip: split-K slabs for prompts whose tiles do not cover the chip
pgk_status engine_gemm_nt_slabs(const bf16* A, const void* W, float* slabs, int splits, int M, int N, int K, hipStream_t st, bool packed = false);

constexpr float LOG2E = 1.4426950408889634f;

// -------------------------------------------------------------------------------------------- one-row projection
enum { SP_NORM = 0, SP_PLAIN = 1, SP_ADD = 2, SP_CAT = 3, SP_HYPER = 4, SP_POLY = 5 };
enum { SE_STORE = 0, SE_SWIGLU = 1, SE_LOGITS = 2, SE_XIELU = 3, SE_TABLE = 4 };

struct StackGemvArgs {
    const void* w;            // [N][K] (SE_SWIGLU: [2 N][K], gate rows then up rows)
    int N, K, W;              // W: true width of the normalised row (columns W..K are zero padding)
    const float* x;           // SP_NORM: residual row; SP_PLAIN: input row  [K]
    const float* y;           // SP_NORM: pending sublayer output (null: none)
    const float* g_post;      // its post-norm weight
    float* x_out;             // where workgroup 0 writes the updated residual row (another buffer than x; null: nowhere)
    const float* gamma;       // null: the row is taken as it is
    // SP_ADD: v = (base or x) + mult * y, then the norm (layer_norm: the mean is taken off); h_out: where workgroup 0 writes the normed row.
    // SP_CAT: the input is [v | row *tok of the embedding table], K / 2 elements each
    const float* base;
    int layer_norm;
    float* h_out;
    const void* embed; const int32_t* tok;
    float eps, mult;
    float* out;               // [N]
    float* amax_val; int* amax_idx;
    float act_pos, act_neg;   // SE_XIELU
    const float* bias;        // SE_STORE: added to the result (null: none)
    float cap;                // SE_LOGITS: soft cap (0: none)
    // SP_HYPER: stream s at x + s * x_stream, y with `upd` the pending sublayer output, `in` the combination (null: sum), norm in groups;
    // x_out: [S][K].  SP_POLY: the input is the polynomial-norm activation of x, W true columns, act [4]
    int S, x_stream, groups;
    const float *upd, *in, *act;
    // SE_TABLE: rows of the shared expert (fs of them, w), then of the token's `top` experts (ff each, w2 [E][ff][K]), then the shared one's gate
    // (w3); gelu, gelu / top, sigmoid.  ids: where workgroup 0 writes the experts
    const void *w2, *w3;
    const int32_t* table;
    int fs, top, ff;
    int32_t* ids;
};

// s + 16 bytes of a weight row . the same piece of the LDS row
template <class WT>
__device__ __forceinline__ float dot_piece(const uint4& raw, const WT* xp, float s) {
    if constexpr (std::is_same<WT, bf16>::value) return dot8_bf16(raw, *reinterpret_cast<const uint4*>(xp), s);
    else {
        const float4 x4 = *reinterpret_cast<const float4*>(xp);
        s = fmaf(__uint_as_float(raw.x), x4.x, s); s = fmaf(__uint_as_float(raw.y), x4.y, s);
        s = fmaf(__uint_as_float(raw.z), x4.z, s); return fmaf(__uint_as_float(raw.w), x4.w, s);
    }
}

// 256 threads; a wave owns R weight rows per trip.  C > 0: the first trip's C chunks of every row are requested before the prologue
// touches the activations (which were requested before them: vector memory returns in order), K <= C * 64 * NW; C == 0: any K.
// Chunks beyond K are clamped in the weight row and zero in the LDS image.
template <class WT, int R, int PRO, int EPI, int C>
__global__ __launch_bounds__(256) void stack_gemv_kernel(unsigned long long* tl, StackGemvArgs a) {
    const TLStamp tls(tl);
    constexpr int NW = WTraits<WT>::NW, CH = 64 * NW;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    WT* xs = reinterpret_cast<WT*>(smem);                         // [round_up(K, CH)]
    __shared__ float red[16], s_bv[4];
    __shared__ int s_bi[4];
    const int K = a.K, N = a.N, lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    constexpr int OUT = EPI == SE_SWIGLU ? R / 2 : R;
    const int wave = blockIdx.x * 4 + wid, nwaves = gridDim.x * 4;
    const WT* w = reinterpret_cast<const WT*>(a.w);
    auto row_of = [&](int n0, int r) -> int {
        if constexpr (EPI == SE_SWIGLU) return r < R / 2 ? min(n0 + r, N - 1) : N + min(n0 + r - R / 2, N - 1);
        else return min(n0 + r, N - 1);
    };
    const int32_t* chosen = nullptr;
    if constexpr (EPI == SE_TABLE) {
        chosen = a.table + (size_t)*a.tok * a.top;
        if (blockIdx.x == 0) for (int i = threadIdx.x; i < a.top; i += 256) a.ids[i] = chosen[i];
    }
    auto row_at = [&](int n0, int r) -> const WT* {
        if constexpr (EPI == SE_TABLE) {
            const int n = min(n0 + r, N - 1), j = n - a.fs;
            if (j < 0) return w + (size_t)n * K;
            if (j >= a.top * a.ff) return reinterpret_cast<const WT*>(a.w3);
            const int k = j / a.ff;
            return reinterpret_cast<const WT*>(a.w2) + ((size_t)chosen[k] * a.ff + (j - k * a.ff)) * K;
        } else return w + (size_t)row_of(n0, r) * K;
    };
    uint4 pre[R][C > 0 ? C : 1];
    if constexpr (PRO == SP_HYPER) {
        float* xf = reinterpret_cast<float*>(smem + (size_t)((K + CH - 1) / CH * CH > C * CH ? (K + CH - 1) / CH * CH : C * CH) * sizeof(WT));   // [K], [groups]
        const int S = a.S;
        auto in_of = [&](int s) { return a.in ? a.in[s] : 1.0f; };
        auto coef_x = [&](int s) {
            if (!a.y) return in_of(s);
            float c = 0.f;
            for (int t = 0; t < S; ++t) c = fmaf(a.upd[2 * S + s * S + t], in_of(t), c);
            return c;
        };
        float cy = 0.f;
        if (a.y) for (int t = 0; t < S; ++t) cy = fmaf(a.upd[S + t], in_of(t), cy);
        if constexpr (C > 0) {                                     // S <= 4
            constexpr int NT = (C * CH + 1023) / 1024;
            const float4 zero = {0.f, 0.f, 0.f, 0.f};
            float4 x[NT][4], y[NT], gm[NT], v[NT];
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = min((int)(threadIdx.x + 256 * t) * 4, K - 4);
#pragma unroll
                for (int s = 0; s < 4; ++s) {
                    x[t][s] = zero;
                    if (s < S) x[t][s] = *reinterpret_cast<const float4*>(a.x + (size_t)s * a.x_stream + i);
                }
                y[t] = zero;
                if (a.y) y[t] = *reinterpret_cast<const float4*>(a.y + i);
                gm[t] = *reinterpret_cast<const float4*>(a.gamma + i);
            }
            __builtin_amdgcn_sched_barrier(0);
            const int nf = min(wave * OUT, N - 1);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const WT* wr = row_at(nf, r);
#pragma unroll
                for (int c = 0; c < C; ++c) pre[r][c] = load_nt16(wr + min(c * CH + lane * NW, K - NW));
            }
            __builtin_amdgcn_sched_barrier(0);
            float cx[4];
#pragma unroll
            for (int s = 0; s < 4; ++s) cx[s] = s < S ? coef_x(s) : 0.f;
            auto mul = [](float c, const float4& p, const float4& q) { return make_float4(fmaf(c, p.x, q.x), fmaf(c, p.y, q.y), fmaf(c, p.z, q.z), fmaf(c, p.w, q.w)); };
            float ss = 0.f;
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = (threadIdx.x + 256 * t) * 4;
                v[t] = mul(cy, y[t], zero);
#pragma unroll
                for (int s = 0; s < 4; ++s) v[t] = mul(cx[s], x[t][s], v[t]);
                if (i >= K) v[t] = zero;
                ss += v[t].x * v[t].x + v[t].y * v[t].y + v[t].z * v[t].z + v[t].w * v[t].w;
                if (a.y && a.x_out && blockIdx.x == t % gridDim.x && i < K)         // the new streams, a piece per workgroup
                    for (int o = 0; o < S; ++o) {
                        float4 z = mul(a.upd[S + o], y[t], zero);
#pragma unroll
                        for (int s = 0; s < 4; ++s) if (s < S) z = mul(a.upd[2 * S + s * S + o], x[t][s], z);
                        *reinterpret_cast<float4*>(a.x_out + (size_t)o * K + i) = z;
                    }
                if (a.groups > 1 && i < K) *reinterpret_cast<float4*>(xf + i) = v[t];
            }
            if (a.groups == 1) {
                const float inv = 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps);
#pragma unroll
                for (int t = 0; t < NT; ++t) { v[t].x *= inv; v[t].y *= inv; v[t].z *= inv; v[t].w *= inv; }
            } else {
                __syncthreads();
                group_rstd(xf, a.W, a.groups, a.eps, xf + K);
                const int gs = a.W / a.groups;
                const float* rs = xf + K;
#pragma unroll
                for (int t = 0; t < NT; ++t) {
                    const int i = min((int)(threadIdx.x + 256 * t) * 4, K - 4), top = a.groups - 1;
                    if ((gs & 3) == 0) { const float q = rs[min(i / gs, top)]; v[t].x *= q; v[t].y *= q; v[t].z *= q; v[t].w *= q; }
                    else { v[t].x *= rs[min(i / gs, top)]; v[t].y *= rs[min((i + 1) / gs, top)]; v[t].z *= rs[min((i + 2) / gs, top)]; v[t].w *= rs[min((i + 3) / gs, top)]; }
                }
            }
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = (threadIdx.x + 256 * t) * 4;
                if (i < C * CH) store4<WT>(xs + i, i < K ? make_float4(v[t].x * gm[t].x, v[t].y * gm[t].y, v[t].z * gm[t].z, v[t].w * gm[t].w) : zero);
            }
        } else {
            float* cx = xf + K + a.groups;                         // [S]
            for (int s = threadIdx.x; s < S; s += 256) cx[s] = coef_x(s);
            __syncthreads();
            const float4 zero = {0.f, 0.f, 0.f, 0.f};
            auto mul = [](float c, const float4& p, const float4& q) { return make_float4(fmaf(c, p.x, q.x), fmaf(c, p.y, q.y), fmaf(c, p.z, q.z), fmaf(c, p.w, q.w)); };
            for (int i = threadIdx.x * 4; i < K; i += 1024) {
                const float* xi = a.x + i;
                const float4 y = a.y ? *reinterpret_cast<const float4*>(a.y + i) : zero;
                float4 u = mul(cy, y, zero);
#pragma unroll 4
                for (int s = 0; s < S; ++s) u = mul(cx[s], *reinterpret_cast<const float4*>(xi + (size_t)s * a.x_stream), u);
                *reinterpret_cast<float4*>(xf + i) = u;
                if (a.y && a.x_out && blockIdx.x == (i >> 10) % gridDim.x)
                    for (int o = 0; o < S; ++o) {
                        float4 z = mul(a.upd[S + o], y, zero);
                        for (int s = 0; s < S; ++s) z = mul(a.upd[2 * S + s * S + o], *reinterpret_cast<const float4*>(xi + (size_t)s * a.x_stream), z);
                        *reinterpret_cast<float4*>(a.x_out + (size_t)o * K + i) = z;
                    }
            }
            __syncthreads();
            group_rstd(xf, a.W, a.groups, a.eps, xf + K);
            const int gs = a.W / a.groups;
            for (int i = threadIdx.x; i < K; i += 256) xs[i] = from_f<WT>(i < a.W ? xf[i] * xf[K + i / gs] * a.gamma[i] : 0.f);
        }
    } else if constexpr (PRO == SP_POLY) {
        float s2 = 0.f, s4 = 0.f, s6 = 0.f;
        auto add = [&](float z) { const float z2 = z * z, z4 = z2 * z2; s2 += z2; s4 += z4; s6 = fmaf(z4, z2, s6); };
        if constexpr (C > 0) {
            constexpr int NT = (C * CH + 1023) / 1024;
            float4 v[NT];
#pragma unroll
            for (int t = 0; t < NT; ++t) v[t] = *reinterpret_cast<const float4*>(a.x + min((int)(threadIdx.x + 256 * t) * 4, K - 4));
            __builtin_amdgcn_sched_barrier(0);
            const int nf = min(wave * OUT, N - 1);
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int c = 0; c < C; ++c) pre[r][c] = load_nt16(row_at(nf, r) + min(c * CH + lane * NW, K - NW));
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int t = 0; t < NT; ++t)
                if ((int)(threadIdx.x + 256 * t) * 4 < K) { add(v[t].x); add(v[t].y); add(v[t].z); add(v[t].w); }      // (columns W .. K are zero)
            s2 = block_sum(s2, red); s4 = block_sum(s4, red); s6 = block_sum(s6, red);
            const float3 cf = poly_coef(a.act, s2, s4, s6, a.W, a.eps);
            const float e = a.act[3];
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = (threadIdx.x + 256 * t) * 4;
                auto at = [&](int j, float z) { return j < a.W ? poly_at(cf, e, z) : 0.f; };
                if (i < C * CH) store4<WT>(xs + i, make_float4(at(i, v[t].x), at(i + 1, v[t].y), at(i + 2, v[t].z), at(i + 3, v[t].w)));
            }
        } else {
            for (int i = threadIdx.x * 4; i < K; i += 1024) { const float4 q = *reinterpret_cast<const float4*>(a.x + i); add(q.x); add(q.y); add(q.z); add(q.w); }
            s2 = block_sum(s2, red); s4 = block_sum(s4, red); s6 = block_sum(s6, red);
            const float3 cf = poly_coef(a.act, s2, s4, s6, a.W, a.eps);
            const float e = a.act[3];
            auto at = [&](int j, float z) { return j < a.W ? poly_at(cf, e, z) : 0.f; };
            for (int i = threadIdx.x * 4; i < K; i += 1024) {
                const float4 q = *reinterpret_cast<const float4*>(a.x + i);
                store4<WT>(xs + i, make_float4(at(i, q.x), at(i + 1, q.y), at(i + 2, q.z), at(i + 3, q.w)));
            }
        }
    } else if constexpr (PRO == SP_CAT) {
        const WT* er = reinterpret_cast<const WT*>(a.embed) + (size_t)*a.tok * a.W;
        const float* from = a.base ? a.base : a.x;
        const int half = K / 2, pad = (K + CH - 1) / CH * CH;
        for (int i = threadIdx.x; i < pad; i += 256)
            xs[i] = i < half ? from_f<WT>(a.y ? fmaf(a.mult, a.y[i], from[i]) : from[i]) : i - half < a.W ? er[i - half] : from_f<WT>(0.f);
        if constexpr (C > 0) {
            const int nf = min(wave * OUT, N - 1);
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int c = 0; c < C; ++c) pre[r][c] = load_nt16(w + (size_t)row_of(nf, r) * K + min(c * CH + lane * NW, K - NW));
            for (int i = pad + threadIdx.x; i < C * CH; i += 256) xs[i] = from_f<WT>(0.f);
        }
    } else if constexpr (C > 0) {
        constexpr int NT = (C * CH + 1023) / 1024;                // float4 per thread
        float4 v[NT], y[NT], gp[NT], gm[NT];
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = min((int)(threadIdx.x + 256 * t) * 4, K - 4);
            v[t] = *reinterpret_cast<const float4*>((PRO == SP_ADD && a.base ? a.base : a.x) + i);
            if constexpr (PRO == SP_ADD) {
                y[t] = *reinterpret_cast<const float4*>((a.y ? a.y : a.x) + i);
                gm[t] = *reinterpret_cast<const float4*>(a.gamma + i);
            }
            if constexpr (PRO == SP_NORM) {
                const float* yp = a.y ? a.y : a.x;                // unconditional loads; masked below
                const float* gm_p = a.gamma ? a.gamma : a.x;
                const float* pp = a.y ? a.g_post : gm_p;
                y[t] = *reinterpret_cast<const float4*>(yp + i);
                gp[t] = *reinterpret_cast<const float4*>(pp + i);
                gm[t] = *reinterpret_cast<const float4*>(gm_p + i);
            }
        }
        __builtin_amdgcn_sched_barrier(0);
        const int nf = min(wave * OUT, N - 1);
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
            for (int c = 0; c < C; ++c) pre[r][c] = load_nt16(w + (size_t)row_of(nf, r) * K + min(c * CH + lane * NW, K - NW));
        __builtin_amdgcn_sched_barrier(0);
        float ss = 0.f;
        if constexpr (PRO == SP_ADD) {
            if (a.y) {
#pragma unroll
                for (int t = 0; t < NT; ++t) {
                    const int i = (threadIdx.x + 256 * t) * 4;
                    v[t].x = fmaf(a.mult, y[t].x, v[t].x); v[t].y = fmaf(a.mult, y[t].y, v[t].y);
                    v[t].z = fmaf(a.mult, y[t].z, v[t].z); v[t].w = fmaf(a.mult, y[t].w, v[t].w);
                    if (a.x_out && blockIdx.x == 0 && i < K) *reinterpret_cast<float4*>(a.x_out + i) = v[t];
                }
            }
            float mean = 0.f;
            if (a.layer_norm) {                                    // (columns W .. K are zero)
                float s1 = 0.f;
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    if ((int)(threadIdx.x + 256 * t) * 4 < K) s1 += (v[t].x + v[t].y) + (v[t].z + v[t].w);
                mean = block_sum(s1, red) / a.W;
            }
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = (threadIdx.x + 256 * t) * 4;
                v[t].x -= mean; v[t].y -= mean; v[t].z -= mean; v[t].w -= mean;
                ss += (i < a.W ? v[t].x * v[t].x : 0.f) + (i + 1 < a.W ? v[t].y * v[t].y : 0.f) + (i + 2 < a.W ? v[t].z * v[t].z : 0.f) + (i + 3 < a.W ? v[t].w * v[t].w : 0.f);
            }
            const float inv = 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps);
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int i = (threadIdx.x + 256 * t) * 4;
                v[t].x *= inv * gm[t].x; v[t].y *= inv * gm[t].y; v[t].z *= inv * gm[t].z; v[t].w *= inv * gm[t].w;
                if (a.h_out && blockIdx.x == 0 && i < K) *reinterpret_cast<float4*>(a.h_out + i) = v[t];
            }
        }
        if constexpr (PRO == SP_NORM) {
            if (a.y) {
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    if ((int)(threadIdx.x + 256 * t) * 4 < K) ss += y[t].x * y[t].x + y[t].y * y[t].y + y[t].z * y[t].z + y[t].w * y[t].w;
                ss = block_sum(ss, red);
                const float inv = a.mult / sqrtf(ss / a.W + a.eps);
#pragma unroll
                for (int t = 0; t < NT; ++t) {
                    const int i = (threadIdx.x + 256 * t) * 4;
                    v[t].x = fmaf(y[t].x * inv, gp[t].x, v[t].x); v[t].y = fmaf(y[t].y * inv, gp[t].y, v[t].y);
                    v[t].z = fmaf(y[t].z * inv, gp[t].z, v[t].z); v[t].w = fmaf(y[t].w * inv, gp[t].w, v[t].w);
                    if (a.x_out && blockIdx.x == 0 && i < K) *reinterpret_cast<float4*>(a.x_out + i) = v[t];
                }
            }
            if (a.gamma) {
                ss = 0.f;
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    if ((int)(threadIdx.x + 256 * t) * 4 < K) ss += v[t].x * v[t].x + v[t].y * v[t].y + v[t].z * v[t].z + v[t].w * v[t].w;
                ss = block_sum(ss, red);
                const float inv = 1.0f / sqrtf(ss / a.W + a.eps);
#pragma unroll
                for (int t = 0; t < NT; ++t) {
                    v[t].x *= inv * gm[t].x; v[t].y *= inv * gm[t].y; v[t].z *= inv * gm[t].z; v[t].w *= inv * gm[t].w;
                }
            }
        }
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int i = (threadIdx.x + 256 * t) * 4;
            if (i < C * CH) store4<WT>(xs + i, i < K ? v[t] : make_float4(0.f, 0.f, 0.f, 0.f));
        }
    } else {
        if constexpr (PRO == SP_NORM) {
            float inv_y = 0.f;
            if (a.y) {
                float ss = 0.f;
                for (int i = threadIdx.x; i < K; i += 256) ss = fmaf(a.y[i], a.y[i], ss);
                inv_y = a.mult / sqrtf(block_sum(ss, red) / a.W + a.eps);
            }
            auto xin = [&](int i) -> float { return a.y ? fmaf(a.y[i] * inv_y, a.g_post[i], a.x[i]) : a.x[i]; };
            float ss = 0.f;
            for (int i = threadIdx.x; i < K; i += 256) {
                const float v = xin(i);
                if (a.y && a.x_out && blockIdx.x == 0) a.x_out[i] = v;
                ss = fmaf(v, v, ss);
            }
            const float inv = a.gamma ? 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps) : 1.0f;
            for (int i = threadIdx.x; i < K; i += 256) xs[i] = from_f<WT>(a.gamma ? xin(i) * inv * a.gamma[i] : xin(i));
        } else if constexpr (PRO == SP_ADD) {
            const float* from = a.base ? a.base : a.x;
            auto xin = [&](int i) -> float { return a.y ? fmaf(a.mult, a.y[i], from[i]) : from[i]; };
            float s1 = 0.f, ss = 0.f;
            for (int i = threadIdx.x; i < K; i += 256) {
                const float v = xin(i);
                if (a.y && a.x_out && blockIdx.x == 0) a.x_out[i] = v;
                s1 += v;
            }
            const float mean = a.layer_norm ? block_sum(s1, red) / a.W : 0.f;
            for (int i = threadIdx.x; i < a.W; i += 256) { const float v = xin(i) - mean; ss = fmaf(v, v, ss); }
            const float inv = 1.0f / sqrtf(block_sum(ss, red) / a.W + a.eps);
            for (int i = threadIdx.x; i < K; i += 256) {
                const float v = (xin(i) - mean) * inv * a.gamma[i];
                xs[i] = from_f<WT>(v);
                if (a.h_out && blockIdx.x == 0) a.h_out[i] = v;
            }
        } else {
            for (int i = threadIdx.x; i < K; i += 256) xs[i] = from_f<WT>(a.x[i]);
        }
    }
    __syncthreads();
    float best_v = -INFINITY;
    int best_i = 0x7FFFFFFF;
    for (int g = wave; g * OUT < N; g += nwaves) {
        const int n0 = g * OUT;
        float acc[R][1];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r][0] = 0.f;
        if (C > 0) {
            if (g != wave) {
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    const WT* wr = row_at(n0, r);
#pragma unroll
                    for (int c = 0; c < C; ++c) pre[r][c] = load_nt16(wr + min(c * CH + lane * NW, K - NW));
                }
            }
#pragma unroll
            for (int c = 0; c < (C > 0 ? C : 1); ++c)
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r][0] = dot_piece<WT>(pre[r][c], xs + c * CH + lane * NW, acc[r][0]);
        } else {
            const WT* wrow[R];
#pragma unroll
            for (int r = 0; r < R; ++r) wrow[r] = row_at(n0, r);
            gemv_rows<WT, WT, 1, R>(wrow, xs, K, K, lane, acc);
        }
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r][0] = wave_sum(acc[r][0]);
        if constexpr (EPI == SE_LOGITS) {
            if (a.cap > 0.f) {                                     // every lane has the sums: lane r caps row r's
                float v = acc[0][0];
#pragma unroll
                for (int r = 1; r < R; ++r) if (lane == r) v = acc[r][0];
                v = soft_cap(v, a.cap);
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r][0] = __shfl(v, r, 64);
            }
        }
        if (lane == 0) {
#pragma unroll
            for (int r = 0; r < OUT; ++r)
                if (n0 + r < N) {
                    float o = acc[r][0];
                    if constexpr (EPI == SE_SWIGLU) o = o / (1.0f + (std::is_same<WT, float>::value ? expf(-o) : __expf(-o))) * acc[r + R / 2][0];
                    if constexpr (EPI == SE_XIELU) o = xielu<std::is_same<WT, float>::value>(o, a.act_pos, a.act_neg);
                    if constexpr (EPI == SE_STORE) { if (a.bias) o += a.bias[n0 + r]; }
                    if constexpr (EPI == SE_TABLE) {
                        const int j = n0 + r - a.fs;
                        o = j >= a.top * a.ff ? 1.0f / (1.0f + expf(-o)) : j < 0 ? gelu_erf(o) : gelu_erf(o) / a.top;
                    }
                    a.out[n0 + r] = o;
                    if constexpr (EPI == SE_LOGITS) { if (o > best_v) { best_v = o; best_i = n0 + r; } }
                }
        }
    }
    if constexpr (EPI == SE_LOGITS) {
        if (lane == 0) { s_bv[wid] = best_v; s_bi[wid] = best_i; }
        __syncthreads();
        if (threadIdx.x == 0) {
            float bv = s_bv[0];
            int bi = s_bi[0];
            for (int i = 1; i < 4; ++i)
                if (s_bv[i] > bv || (s_bv[i] == bv && s_bi[i] < bi)) { bv = s_bv[i]; bi = s_bi[i]; }
            a.amax_val[blockIdx.x] = bv;
            a.amax_idx[blockIdx.x] = bi;
        }
    }
    tls.end();
}

template <class WT, int R, int PRO, int EPI, int C>
static pgk_status stack_gemv_c(const StackGemvArgs& a, int grid, hipStream_t st) {
    constexpr int CH = 64 * WTraits<WT>::NW;
    size_t lds = (size_t)ceil_div(a.K, CH) * CH * sizeof(WT) > (size_t)C * CH * sizeof(WT) ? (size_t)ceil_div(a.K, CH) * CH * sizeof(WT) : (size_t)C * CH * sizeof(WT);
    if (PRO == SP_HYPER && (C == 0 || a.groups > 1)) lds += (size_t)(a.K + a.groups + a.S) * 4;
    auto kfn = &stack_gemv_kernel<WT, R, PRO, EPI, C>;
    PGK_REQUIRE(lds <= 156 * 1024, "engine: a row of %d does not fit LDS", a.K);
    static bool attr_done = false;
    if (lds > 48 * 1024 && !attr_done) {
        PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, 156 * 1024));
        attr_done = true;
    }
    PGK_CHECK_HIP(launch_k(kfn, dim3(grid), dim3(256), lds, st, a));
    return PGK_OK;
}

template <class WT, int R, int PRO, int EPI>
static pgk_status stack_gemv_r(const StackGemvArgs& a, hipStream_t st, int force_grid = 0) {
    constexpr int OUT = EPI == SE_SWIGLU ? R / 2 : R;
    int grid = force_grid ? force_grid : ceil_div(a.N, OUT * 4);
    if (grid > 1024) grid = 1024;
    if constexpr (std::is_same<WT, bf16>::value) {
        const int c = PRO == SP_HYPER && a.S > 4 ? 99 : ceil_div(a.K, 512);
        if constexpr (R * 2 <= 16) { if (c <= 2) return stack_gemv_c<WT, R, PRO, EPI, 2>(a, grid, st); }
        if constexpr (R * 4 <= 16) { if (c <= 4) return stack_gemv_c<WT, R, PRO, EPI, 4>(a, grid, st); }
        if constexpr (R * 8 <= 16) { if (c <= 8) return stack_gemv_c<WT, R, PRO, EPI, 8>(a, grid, st); }
    }
    return stack_gemv_c<WT, R, PRO, EPI, 0>(a, grid, st);
}

// A wide row of several streams: two rows a wave, so that the streams stay in registers, and no more workgroups than are resident, since
// every one reads all streams
constexpr int HYPER_WIDE_GRID = 512;
static bool hyper_wide(int K) { return K > 2048 && K <= 4096; }

template <class WT, int PRO, int EPI>
static pgk_status stack_gemv(const StackGemvArgs& a, hipStream_t st, int force_grid = 0) {
    if constexpr (std::is_same<WT, float>::value) return stack_gemv_r<WT, EPI == SE_STORE || EPI == SE_XIELU ? 1 : 2, PRO, EPI>(a, st, force_grid);
    else if constexpr (EPI == SE_SWIGLU) {
        if (a.N >= 4096) return stack_gemv_r<WT, 4, PRO, EPI>(a, st);
        return stack_gemv_r<WT, 2, PRO, EPI>(a, st);
    } else if constexpr (EPI == SE_LOGITS) {
        if constexpr (PRO == SP_HYPER) { if (hyper_wide(a.K)) return stack_gemv_r<WT, 2, PRO, EPI>(a, st, force_grid); }
        return stack_gemv_r<WT, 4, PRO, EPI>(a, st, force_grid);
    } else {
        if (PRO == SP_HYPER && hyper_wide(a.K)) return stack_gemv_r<WT, 2, PRO, EPI>(a, st, min(ceil_div(a.N, 8), HYPER_WIDE_GRID));
        if (a.N >= 8192) return stack_gemv_r<WT, 4, PRO, EPI>(a, st);
        if (a.N >= 2048) return stack_gemv_r<WT, 2, PRO, EPI>(a, st);
        return stack_gemv_r<WT, 1, PRO, EPI>(a, st);
    }
}

// -------------------------------------------------------------------------------------------- latent attention, decode
struct LatentArgs {
    const void* in;           // [B][ld_in] (IT): q at h * D, latent at qn, head gates at qn + rank
    int ld_in, qn, g_off;     // g_off < 0: no gates
    const void *w_uk, *w_uv;  // [H * D][rank] (T)
    const float* c_norm;      // [rank]
    void* cache;              // [slots][R][rank] (T)
    const int32_t* positions; // [B]
    int B, H, D, dim, vdim, rank, rank_true, R, nsplit, vc;
    float eps, scale;         // scale already times log2e
    int rot;                  // the last rot of a head's dim query columns and the rot latent columns behind rank_true are turned by the position
    const float* rot_freq;    // [rot / 2]
    void* qlat;               // [B][H][rank], float or bf16
    float* po;                // [B][H][nsplit][rank]
    float* pml;               // [B][H][nsplit][2]
    void* out;                // [B][ld_out] (IT): head h at h * D
    int ld_out;
};

// Column i of n rotated ones (neighbours 2j, 2j + 1 are a pair): x points at column 0
template <class T>
__device__ __forceinline__ float rotated(const T* x, int i, int pos, const float* freq) {
    float s, c;
    sincosf((float)pos * freq[i >> 1], &s, &c);
    const float u = to_f(x[i & ~1]), v = to_f(x[i | 1]);
    return i & 1 ? fmaf(v, c, u * s) : fmaf(u, c, -v * s);
}

// q_lat[b][h][r] = scale * sum_d U_k[h D + d][r] q[b][h][d]: workgroup = (head, 128 columns) x MB sequences, the four waves split d
// in runs of four; 128 rows of U_k are requested before the queries are staged.  QT: element type of q_lat (bf16 for the MFMA kernel).
// The last workgroup column normalises the MB new latent rows into the ring instead.
template <class T, class IT, class QT, int MB>
__global__ __launch_bounds__(256) void latent_absorb_kernel(unsigned long long* tl, LatentArgs a) {
    const TLStamp tls(tl);
    const int nt = (a.rank + 127) / 128, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, b0 = blockIdx.y * MB;
    const IT* in = reinterpret_cast<const IT*>(a.in);
    if ((int)blockIdx.x == a.H * nt) {
        for (int m = wid; m < MB && b0 + m < a.B; m += 4) {        // a wave per sequence
            const int b = b0 + m;
            const IT* c = in + (size_t)b * a.ld_in + a.qn;
            float ss = 0.f;
            for (int r = lane; r < a.rank_true; r += 64) { const float v = to_f(c[r]); ss = fmaf(v, v, ss); }
            const float inv = 1.0f / sqrtf(wave_sum(ss) / a.rank_true + a.eps);
            const int pos = max(a.positions[b], 0);
            T* row = reinterpret_cast<T*>(a.cache) + ((size_t)b * a.R + pos % a.R) * a.rank;
            for (int r = lane; r < a.rank; r += 64)
                row[r] = from_f<T>(r >= a.rank_true && r < a.rank_true + a.rot ? rotated(c + a.rank_true, r - a.rank_true, pos, a.rot_freq) : to_f(c[r]) * inv * a.c_norm[r]);
        }
        tls.end();
        return;
    }
    __shared__ __attribute__((aligned(16))) float qs[MB][128];
    __shared__ float part[4][MB][128];
    const int h = blockIdx.x / nt, r0 = (blockIdx.x % nt) * 128 + 2 * lane;
    const bool live = r0 < a.rank;                                 // rank is a multiple of 64: both columns or none
    float acc[MB][2];
#pragma unroll
    for (int m = 0; m < MB; ++m) acc[m][0] = acc[m][1] = 0.f;
    for (int d0 = 0; d0 < a.dim; d0 += 128) {
        const int dn = min(128, a.dim - d0);
        const T* u = reinterpret_cast<const T*>(a.w_uk) + (size_t)(h * a.D + d0) * a.rank + (live ? r0 : 0);
        using W2 = typename std::conditional<std::is_same<T, bf16>::value, uint32_t, float2>::type;     // two columns
        W2 wr[32];
#pragma unroll
        for (int i = 0; i < 32; ++i) {
            const int d = min(4 * (4 * (i >> 2) + wid) + (i & 3), dn - 1);
            wr[i] = *reinterpret_cast<const W2*>(u + (size_t)d * a.rank);
        }
        __syncthreads();
        for (int i = threadIdx.x; i < MB * 128; i += 256) {
            const int m = i >> 7, d = i & 127;
            const int b = min(b0 + m, a.B - 1), at = d0 + d - (a.dim - a.rot);
            const IT* q = in + (size_t)b * a.ld_in + h * a.D;
            qs[m][d] = d >= dn ? 0.f : at < 0 ? to_f(q[d0 + d]) : rotated(q + a.dim - a.rot, at, max(a.positions[b], 0), a.rot_freq);
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            float w[4][2];
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                if constexpr (std::is_same<T, bf16>::value) { w[k][0] = __uint_as_float(wr[4 * i + k] << 16); w[k][1] = __uint_as_float(wr[4 * i + k] & 0xFFFF0000u); }
                else { w[k][0] = wr[4 * i + k].x; w[k][1] = wr[4 * i + k].y; }
            }
#pragma unroll
            for (int m = 0; m < MB; ++m) {
                const float4 q = *reinterpret_cast<const float4*>(&qs[m][4 * (4 * i + wid)]);
#pragma unroll
                for (int e = 0; e < 2; ++e) acc[m][e] = fmaf(w[3][e], q.w, fmaf(w[2][e], q.z, fmaf(w[1][e], q.y, fmaf(w[0][e], q.x, acc[m][e]))));
            }
        }
    }
#pragma unroll
    for (int m = 0; m < MB; ++m) { part[wid][m][2 * lane] = acc[m][0]; part[wid][m][2 * lane + 1] = acc[m][1]; }
    __syncthreads();
    for (int i = threadIdx.x; i < MB * 128; i += 256) {
        const int m = i >> 7, c = i & 127, r = (blockIdx.x % nt) * 128 + c;
        if (b0 + m < a.B && r < a.rank)
            reinterpret_cast<QT*>(a.qlat)[((size_t)(b0 + m) * a.H + h) * a.rank + r] = from_f<QT>(a.scale * (part[0][m][c] + part[1][m][c] + part[2][m][c] + part[3][m][c]));
    }
    tls.end();
}

// Any rank up to 2048, any element type: a wave walks every fourth key, one strided element per lane and 64 columns.
template <class T, int RC, int HB>
__global__ __launch_bounds__(256) void latent_attn_kernel(unsigned long long* tl, LatentArgs a) {
    const TLStamp tls(tl);
    __shared__ float sm[4][HB][2];
    extern __shared__ float so[];                                  // [HB][rank]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, s = blockIdx.x, h0 = blockIdx.y * HB, b = blockIdx.z;
    const int n = min(max(a.positions[b], 0) + 1, a.R);
    int k0, k1;
    split_range(n, a.nsplit, s, k0, k1);
    float q[HB][RC], o[HB][RC], m[HB], l[HB];
#pragma unroll
    for (int i = 0; i < HB; ++i) {
        m[i] = -INFINITY; l[i] = 0.f;
        const float* qp = reinterpret_cast<const float*>(a.qlat) + ((size_t)b * a.H + min(h0 + i, a.H - 1)) * a.rank;
#pragma unroll
        for (int j = 0; j < RC; ++j) { const int r = 64 * j + lane; q[i][j] = r < a.rank ? qp[r] : 0.f; o[i][j] = 0.f; }
    }
    const T* cb = reinterpret_cast<const T*>(a.cache) + (size_t)b * a.R * a.rank;
    for (int k = k0 + wid; k < k1; k += 4) {
        float c[RC];
#pragma unroll
        for (int j = 0; j < RC; ++j) { const int r = 64 * j + lane; c[j] = r < a.rank ? to_f(cb[(size_t)k * a.rank + r]) : 0.f; }
#pragma unroll
        for (int i = 0; i < HB; ++i) {
            float t = 0.f;
#pragma unroll
            for (int j = 0; j < RC; ++j) t = fmaf(q[i][j], c[j], t);
            t = wave_sum(t);
            const float mn = fmaxf(m[i], t), al = exp2f(m[i] - mn), p = exp2f(t - mn);
            m[i] = mn;
            l[i] = fmaf(l[i], al, p);
#pragma unroll
            for (int j = 0; j < RC; ++j) o[i][j] = fmaf(o[i][j], al, p * c[j]);
        }
    }
    if (lane == 0) {
#pragma unroll
        for (int i = 0; i < HB; ++i) { sm[wid][i][0] = m[i]; sm[wid][i][1] = l[i]; }
    }
    for (int i = threadIdx.x; i < HB * a.rank; i += 256) so[i] = 0.f;
    __syncthreads();
    for (int w = 0; w < 4; ++w) {                                  // waves add their share in turn: a fixed order
        if (wid == w) {
#pragma unroll
            for (int i = 0; i < HB; ++i) {
                const float mm = fmaxf(fmaxf(sm[0][i][0], sm[1][i][0]), fmaxf(sm[2][i][0], sm[3][i][0]));
                const float f = l[i] > 0.f ? exp2f(m[i] - mm) : 0.f;
#pragma unroll
                for (int j = 0; j < RC; ++j) { const int r = 64 * j + lane; if (r < a.rank) so[i * a.rank + r] += f * o[i][j]; }
            }
        }
        __syncthreads();
    }
    for (int i = threadIdx.x; i < HB * a.rank; i += 256) {
        const int hh = h0 + i / a.rank;
        if (hh < a.H) a.po[(((size_t)b * a.H + hh) * a.nsplit + s) * a.rank + i % a.rank] = so[i];
    }
    if (threadIdx.x < HB && h0 + (int)threadIdx.x < a.H) {
        const int i = threadIdx.x;
        float mm = -INFINITY, ll = 0.f;
        for (int w = 0; w < 4; ++w) mm = fmaxf(mm, sm[w][i][0]);
        for (int w = 0; w < 4; ++w) if (sm[w][i][1] > 0.f) ll += sm[w][i][1] * exp2f(sm[w][i][0] - mm);
        float* ml = a.pml + (((size_t)b * a.H + h0 + i) * a.nsplit + s) * 2;
        ml[0] = mm; ml[1] = ll;
    }
    tls.end();
}

// bf16, rank <= 64 RT <= 896: 16 heads x 64 keys per step on the matrix pipe.  Every head scores against the SAME latent rows, so one
// LDS image of a key tile is both operands: S[head][key] = q_lat . C^T (each wave 16 keys), then O[head][r] += P . C (each wave its
// share of the columns; C^T comes out of the row-major image through ds_read_b64_tr_b16, whose k order is 16 (j >> 2) + 4 (lane >> 4)
// + (j & 3), and P is read back from LDS in that order).
typedef __bf16 bf16x8_st __attribute__((ext_vector_type(8)));
typedef float f32x4_st __attribute__((ext_vector_type(4)));
typedef short v4s_st __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4_st mfma16_st(const uint4& a, const uint4& b, f32x4_st c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_st, a), __builtin_bit_cast(bf16x8_st, b), c, 0, 0, 0);
}

constexpr int LA_PAD = 8;           // elements added to an LDS row: rows start 4 banks apart
static size_t latent_mfma_lds(int rank) { return (size_t)(64 + 16) * (rank + LA_PAD) * 2; }

template <int RT>
__global__ __launch_bounds__(256) void latent_attn_mfma_kernel(unsigned long long* tl, LatentArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) char la_smem[];
    __shared__ __attribute__((aligned(16))) bf16 ps[16][72];
    __shared__ float red[4][16];
    const int ld = a.rank + LA_PAD, nch = a.rank / 8;
    bf16* cs = reinterpret_cast<bf16*>(la_smem);                  // [64][ld]
    bf16* qs = cs + 64 * ld;                                      // [16][ld]
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4;
    const int s = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z;
    const int n = min(max(a.positions[b], 0) + 1, a.R);
    int k0, k1;
    split_range(n, a.nsplit, s, k0, k1);
    float m_run[4], l_run[4];
    f32x4_st o[RT];
#pragma unroll
    for (int i = 0; i < 4; ++i) { m_run[i] = -INFINITY; l_run[i] = 0.f; }
#pragma unroll
    for (int t = 0; t < RT; ++t) o[t] = f32x4_st{0.f, 0.f, 0.f, 0.f};
    if (k0 >= k1) {                                                // an empty split: its record says so, the sums are never read
        if (tid < 16 && h0 + tid < a.H) {
            float* ml = a.pml + (((size_t)b * a.H + h0 + tid) * a.nsplit + s) * 2;
            ml[0] = -INFINITY; ml[1] = 0.f;
        }
        tls.end();
        return;
    }
    const bf16* cb = reinterpret_cast<const bf16*>(a.cache) + (size_t)b * a.R * a.rank;
    const bf16* qb = reinterpret_cast<const bf16*>(a.qlat) + (size_t)b * a.H * a.rank;
    // 16-byte pieces of the query block and of a key tile, all requested before the first is stored.  LPR lanes per row (a power of
    // two: no division), lanes past a row's end repeat its last piece.
    constexpr int LPR = RT >= 8 ? 64 : 8 * RT, HALF = RT > 8 ? 2 : 1, RPP = 256 / LPR, QN = (RPP >= 16 ? 1 : 16 / RPP) * HALF, CN = 64 / RPP * HALF;
    const int r_in = tid / LPR, k_in = tid % LPR;
    auto q_row = [&](int i) { return min(i / HALF * RPP + r_in, 15); };
    auto col = [&](int i) { return min(k_in + (i % HALF) * LPR, nch - 1) * 8; };
    u32x4 qv[QN], cv[CN];                                         // (vector type: a uint4 array carried around the loop is left in scratch memory)
#pragma unroll
    for (int i = 0; i < QN; ++i) qv[i] = *reinterpret_cast<const u32x4*>(qb + (size_t)(min(h0 + q_row(i), a.H - 1) * a.rank + col(i)));
#pragma unroll
    for (int i = 0; i < CN; ++i) cv[i] = *reinterpret_cast<const u32x4*>(cb + (size_t)(min(k0 + i / HALF * RPP + r_in, k1 - 1) * a.rank + col(i)));
#pragma unroll
    for (int i = 0; i < QN; ++i) *reinterpret_cast<u32x4*>(qs + q_row(i) * ld + col(i)) = qv[i];
    for (int kt = k0; kt < k1; kt += 64) {
        const int rt = k1 - kt > 32 ? 64 : 32;                    // rows of this tile that take part (the rest repeat the last key)
        if (kt != k0) __syncthreads();                            // the last step's reads of cs are done
#pragma unroll
        for (int i = 0; i < CN; ++i) *reinterpret_cast<u32x4*>(cs + (i / HALF * RPP + r_in) * ld + col(i)) = cv[i];
        __syncthreads();
#pragma unroll
        for (int i = 0; i < CN; ++i) cv[i] = *reinterpret_cast<const u32x4*>(cb + (size_t)(min(kt + 64 + i / HALF * RPP + r_in, k1 - 1) * a.rank + col(i)));     // the next tile travels under this one's products
        f32x4_st sc = {-INFINITY, -INFINITY, -INFINITY, -INFINITY};
        const bool mine = 16 * wid < rt;                          // wave-uniform
        if (mine) {
            f32x4_st t = {0.f, 0.f, 0.f, 0.f};
            const bf16* qr = qs + l15 * ld + 8 * q4;
            const bf16* cr = cs + (16 * wid + l15) * ld + 8 * q4;
            for (int ks = 0; ks < a.rank; ks += 32) t = mfma16_st(*reinterpret_cast<const uint4*>(qr + ks), *reinterpret_cast<const uint4*>(cr + ks), t);
            if (kt + 16 * wid + l15 < k1) sc = t;                 // lane: heads 4 q4 + i, key 16 wid + l15
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
        for (int ks = 0; ks < rt; ks += 32) {
            const uint2 p0 = *reinterpret_cast<const uint2*>(&ps[l15][ks + 4 * q4]), p1 = *reinterpret_cast<const uint2*>(&ps[l15][ks + 16 + 4 * q4]);
            const uint4 pf = make_uint4(p0.x, p0.y, p1.x, p1.y);
            const bf16* row = cs + (ks + 4 * q4 + (l15 >> 2)) * ld + 4 * (l15 & 3);
#pragma unroll
            for (int t = 0; t < RT; ++t) {
                const int col = 16 * (wid + 4 * t);
                if (col < a.rank) {                               // wave-uniform
                    const v4s_st c0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_st*)(row + col));
                    const v4s_st c1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_st*)(row + 16 * ld + col));
                    const uint2 u0 = __builtin_bit_cast(uint2, c0), u1 = __builtin_bit_cast(uint2, c1);
                    o[t] = mfma16_st(pf, make_uint4(u0.x, u0.y, u1.x, u1.y), o[t]);
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
        const int hh = h0 + 4 * q4 + i;
        if (hh >= a.H) continue;
        const size_t rec = ((size_t)b * a.H + hh) * a.nsplit + s;
#pragma unroll
        for (int t = 0; t < RT; ++t) {
            const int col = 16 * (wid + 4 * t) + l15;
            if (col < a.rank) a.po[rec * a.rank + col] = o[t][i];
        }
        if (wid == 0 && l15 == 0) {
            a.pml[2 * rec] = m_run[i];
            a.pml[2 * rec + 1] = red[0][4 * q4 + i] + red[1][4 * q4 + i] + red[2][4 * q4 + i] + red[3][4 * q4 + i];
        }
    }
    tls.end();
}

// Combine the split records of (sequence, head), apply U_v (the workgroup's vc runs of 32 rows) and the head's gate.  The waves share the splits,
// then meet in LDS; a row of U_v is 16 lanes wide, requested before the records when the rank allows (PF 128-column pieces per row).
template <class T, class IT, int MB, int PF>
__global__ __launch_bounds__(256) void latent_merge_uv_kernel(unsigned long long* tl, LatentArgs a) {
    const TLStamp tls(tl);
    extern __shared__ __attribute__((aligned(16))) float ol[];     // [4][MB][rank]; afterwards [MB][rank]
    __shared__ float sw[MB][64];
    constexpr int NW = WTraits<T>::NW;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, h = blockIdx.x, b0 = blockIdx.z * MB, sub = lane & 15, grp = lane >> 4;
    int v0 = blockIdx.y * 32 * a.vc;
    const T* u = reinterpret_cast<const T*>(a.w_uv) + (size_t)h * a.D * a.rank;
    uint4 w[2][PF > 0 ? PF : 1];
    if constexpr (PF > 0) {
#pragma unroll
        for (int p = 0; p < 2; ++p)
#pragma unroll
            for (int k = 0; k < PF; ++k)
                w[p][k] = *reinterpret_cast<const uint4*>(u + (size_t)min(v0 + 8 * wid + 4 * p + grp, a.vdim - 1) * a.rank + min(16 * NW * k + sub * NW, a.rank - NW));
    }
    for (int m = wid; m < MB; m += 4) {
        const size_t rec = ((size_t)min(b0 + m, a.B - 1) * a.H + h) * a.nsplit;
        const float mm = lane < a.nsplit ? a.pml[(rec + lane) * 2] : -INFINITY, ll = lane < a.nsplit ? a.pml[(rec + lane) * 2 + 1] : 0.f;
        const float top = wave_max(ll > 0.f ? mm : -INFINITY), f = ll > 0.f ? exp2f(mm - top) : 0.f;
        const float den = wave_sum(f * ll);
        sw[m][lane] = f / den;
    }
    __syncthreads();
    int nact[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) {
        const int n = min(max(a.positions[min(b0 + m, a.B - 1)], 0) + 1, a.R), per = split_rows(n, a.nsplit);
        nact[m] = (n + per - 1) / per;
    }
    for (int r0 = 0; r0 < a.rank; r0 += 256) {
        const int r = r0 + 4 * lane, rc = min(r, a.rank - 4);
        float4 t[MB];
        constexpr int SU = MB == 1 ? 8 : 4;                        // records in flight per sequence: clamped loads, weight 0 beyond the last
        int most = 0;
#pragma unroll
        for (int m = 0; m < MB; ++m) { t[m] = make_float4(0.f, 0.f, 0.f, 0.f); most = max(most, nact[m]); }
        for (int s0 = wid; s0 < most; s0 += 4 * SU) {
            float4 p[MB][SU];
#pragma unroll
            for (int m = 0; m < MB; ++m)
#pragma unroll
                for (int k = 0; k < SU; ++k)
                    p[m][k] = *reinterpret_cast<const float4*>(a.po + (((size_t)min(b0 + m, a.B - 1) * a.H + h) * a.nsplit + min(s0 + 4 * k, nact[m] - 1)) * a.rank + rc);
#pragma unroll
            for (int m = 0; m < MB; ++m)
#pragma unroll
                for (int k = 0; k < SU; ++k) {
                    const float f = s0 + 4 * k < nact[m] ? sw[m][s0 + 4 * k] : 0.f;
                    t[m].x = fmaf(f, p[m][k].x, t[m].x); t[m].y = fmaf(f, p[m][k].y, t[m].y); t[m].z = fmaf(f, p[m][k].z, t[m].z); t[m].w = fmaf(f, p[m][k].w, t[m].w);
                }
        }
        if (r < a.rank) {
#pragma unroll
            for (int m = 0; m < MB; ++m) *reinterpret_cast<float4*>(ol + ((size_t)wid * MB + m) * a.rank + r) = t[m];
        }
    }
    __syncthreads();
    const int span = MB * a.rank;
    for (int i = 4 * threadIdx.x; i < span; i += 1024) {
        float4 t = *reinterpret_cast<const float4*>(ol + i);
#pragma unroll
        for (int q = 1; q < 4; ++q) {
            const float4 p = *reinterpret_cast<const float4*>(ol + q * span + i);
            t.x += p.x; t.y += p.y; t.z += p.z; t.w += p.w;
        }
        *reinterpret_cast<float4*>(ol + i) = t;
    }
    __syncthreads();
    for (int c = 0; c < a.vc; ++c, v0 += 32) {
        if (v0 >= a.vdim) break;                                   // block-uniform
        if constexpr (PF > 0) {
            if (c > 0) {
#pragma unroll
                for (int p = 0; p < 2; ++p)
#pragma unroll
                    for (int k = 0; k < PF; ++k)
                        w[p][k] = *reinterpret_cast<const uint4*>(u + (size_t)min(v0 + 8 * wid + 4 * p + grp, a.vdim - 1) * a.rank + min(16 * NW * k + sub * NW, a.rank - NW));
            }
        }
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const int v = v0 + 8 * wid + 4 * p + grp;
            float acc[MB];
#pragma unroll
            for (int m = 0; m < MB; ++m) acc[m] = 0.f;
            auto piece = [&](const uint4& raw, int r) {
                float f[NW];
                WTraits<T>::decode(raw, f);
#pragma unroll
                for (int m = 0; m < MB; ++m)
#pragma unroll
                    for (int j = 0; j < NW; j += 4) {
                        const float4 x = *reinterpret_cast<const float4*>(ol + m * a.rank + r + j);
                        acc[m] = fmaf(f[j + 3], x.w, fmaf(f[j + 2], x.z, fmaf(f[j + 1], x.y, fmaf(f[j], x.x, acc[m]))));
                    }
            };
            if constexpr (PF > 0) {
#pragma unroll
                for (int k = 0; k < PF; ++k) { const int r = 16 * NW * k + sub * NW; if (r < a.rank) piece(w[p][k], r); }
            } else {
                const T* row = u + (size_t)min(v, a.vdim - 1) * a.rank;
                for (int r = sub * NW; r < a.rank; r += 16 * NW) piece(*reinterpret_cast<const uint4*>(row + r), r);
            }
#pragma unroll
            for (int m = 0; m < MB; ++m) {
                const float y = group16_sum(acc[m]);
                if (sub == 0 && v < a.vdim && b0 + m < a.B) {
                    const float g = a.g_off < 0 ? 1.f : 1.0f / (1.0f + expf(-to_f(reinterpret_cast<const IT*>(a.in)[(size_t)(b0 + m) * a.ld_in + a.g_off + h])));
                    reinterpret_cast<IT*>(a.out)[(size_t)(b0 + m) * a.ld_out + h * a.D + v] = from_f<IT>(y * g);
                }
            }
        }
    }
    tls.end();
}

// -------------------------------------------------------------------------------------------- experts of one row
struct MoeOneArgs {
    RouterCfg r;
    const float *logits, *h;              // [E], [W] (normed row)
    const void *w_up, *w_down;            // [E][2 ff][W], [E][N][ff]
    int W, ff;
    float* act;                           // [top][ff], times the choice's weight
    int32_t* ids;                         // [top]
    const void* w_o; const float* a; int n_att;
    const float* gate;                    // moe_out_one: a is multiplied by *gate (null: not)
    float* y; int N;
};

// Every workgroup chooses for itself (a few hundred operations); a wave owns R / 2 outputs of one expert per trip.
template <class WT, int R>
__global__ __launch_bounds__(256) void moe_up_one_kernel(unsigned long long* tl, MoeOneArgs a) {
    const TLStamp tls(tl);
    constexpr int NW = WTraits<WT>::NW, CH = 64 * NW, OUT = R / 2, U = 4;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int W = a.W, padded = (W + CH - 1) / CH * CH, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, top = a.r.top;
    WT* xs = reinterpret_cast<WT*>(smem);                         // [padded]
    float* rf = reinterpret_cast<float*>(xs + padded);
    float* wts = rf + route_floats(a.r);
    int32_t* ids = reinterpret_cast<int32_t*>(wts + top);
    for (int i = threadIdx.x; i < padded; i += 256) xs[i] = from_f<WT>(i < W ? a.h[i] : 0.f);
    route_row<256>(a.r, rf, threadIdx.x, [&](int e) { return a.logits[e]; }, ids, wts, []() { __syncthreads(); });
    if (blockIdx.x == 0)
        for (int i = threadIdx.x; i < top; i += 256) a.ids[i] = ids[i];
    const int total = top * a.ff;
    for (int o = (blockIdx.x * 4 + wid) * OUT; o < total; o += gridDim.x * 4 * OUT) {
        const int k = o / a.ff, j = o - k * a.ff;                 // (ff is a multiple of 64: all OUT outputs are one expert's)
        const WT* w = reinterpret_cast<const WT*>(a.w_up) + (size_t)ids[k] * 2 * a.ff * W;
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int c0 = 0; c0 < padded; c0 += U * CH) {
            uint4 raw[R][U];
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int r = 0; r < R; ++r)
                    raw[r][u] = load_nt16(w + (size_t)((r / OUT) * a.ff + j + r % OUT) * W + min(c0 + u * CH + lane * NW, W - NW));
#pragma unroll
            for (int u = 0; u < U; ++u) {
                if (c0 + u * CH >= padded) break;                  // (uniform)
                const WT* xp = xs + c0 + u * CH + lane * NW;
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r] = dot_piece<WT>(raw[r][u], xp, acc[r]);
            }
        }
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = wave_sum(acc[r]);
        if (lane == 0) {
#pragma unroll
            for (int r = 0; r < OUT; ++r) a.act[o + r] = silu_f<std::is_same<WT, float>::value>(acc[r]) * acc[r + OUT] * wts[k];
        }
    }
    tls.end();
}

// y = W_o (gate a) + sum over the chosen experts of W_down act: one row of 16-byte pieces that starts in W_o and goes on through the experts'
template <class WT, int R>
__global__ __launch_bounds__(256) void moe_out_one_kernel(unsigned long long* tl, MoeOneArgs a) {
    const TLStamp tls(tl);
    constexpr int NW = WTraits<WT>::NW, U = R >= 4 ? 4 : 8;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ int32_t ids[MOE_MAX_TOP];
    WT* xs = reinterpret_cast<WT*>(smem);                         // [n_att + top ff, one piece of zeros]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, top = a.r.top, na = a.n_att / NW, nf = a.ff / NW, np = na + top * nf, len = np * NW;
    if ((int)threadIdx.x < top) ids[threadIdx.x] = a.ids[threadIdx.x];
    const float gate = a.gate ? *a.gate : 1.0f;
    for (int i = threadIdx.x; i < len + NW; i += 256) xs[i] = from_f<WT>(i < a.n_att ? gate * a.a[i] : i < len ? a.act[i - a.n_att] : 0.f);
    __syncthreads();
    for (int n0 = (blockIdx.x * 4 + wid) * R; n0 < a.N; n0 += gridDim.x * 4 * R) {
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int p0 = lane; p0 - lane < np; p0 += 64 * U) {
            uint4 raw[U][R];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int p = min(p0 + 64 * u, np - 1), q = max(p - na, 0), k = q / (nf > 0 ? nf : 1);
                const WT* at = p < na ? reinterpret_cast<const WT*>(a.w_o) + p * NW : reinterpret_cast<const WT*>(a.w_down) + (size_t)ids[k] * a.N * a.ff + (q - k * nf) * NW;
                const size_t ld = p < na ? a.n_att : a.ff;
#pragma unroll
                for (int r = 0; r < R; ++r) raw[u][r] = load_nt16(at + min(n0 + r, a.N - 1) * ld);
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const WT* xp = xs + min(p0 + 64 * u, np) * NW;
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r] = dot_piece<WT>(raw[u][r], xp, acc[r]);
            }
        }
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float y = wave_sum(acc[r]);
            if (lane == 0 && n0 + r < a.N) a.y[n0 + r] = y;
        }
    }
    tls.end();
}

template <class T>
static pgk_status moe_up_one(const MoeOneArgs& a, hipStream_t st) {
    constexpr int CH = 64 * WTraits<T>::NW;
    const size_t lds = (size_t)ceil_div(a.W, CH) * CH * sizeof(T) + (size_t)(route_floats(a.r) + 2 * a.r.top) * 4;
    PGK_REQUIRE(lds <= 64 * 1024, "engine: a row of %d and %d experts do not fit LDS", a.W, a.r.E);
    const int total = a.r.top * a.ff;
    auto go = [&](auto rows) -> pgk_status {
        constexpr int R = decltype(rows)::value;
        const int grid = ceil_div(total, 2 * R);
        PGK_CHECK_HIP(launch_k(&moe_up_one_kernel<T, R>, dim3(grid < 1024 ? grid : 1024), dim3(256), lds, st, a));
        return PGK_OK;
    };
    return total >= 8192 ? go(std::integral_constant<int, 4>{}) : go(std::integral_constant<int, 2>{});
}
template <class T>
static pgk_status moe_out_one(const MoeOneArgs& a, hipStream_t st) {
    const size_t lds = (size_t)(a.n_att + a.r.top * a.ff + WTraits<T>::NW) * sizeof(T);
    PGK_REQUIRE(lds <= 144 * 1024, "engine: %d mixer columns and %d experts of %d do not fit LDS", a.n_att, a.r.top, a.ff);
    auto go = [&](auto rows) -> pgk_status {
        constexpr int R = decltype(rows)::value;
        auto kfn = &moe_out_one_kernel<T, R>;
        static bool done = false;
        if (lds > 48 * 1024 && !done) {
            PGK_CHECK_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024));
            done = true;
        }
        PGK_CHECK_HIP(launch_k(kfn, dim3(ceil_div(a.N, 4 * R)), dim3(256), lds, st, a));
        return PGK_OK;
    };
    return a.N >= 4096 ? go(std::integral_constant<int, 2>{}) : go(std::integral_constant<int, 1>{});
}

// -------------------------------------------------------------------------------------------- rows (prompts, batches)
template <class T>
__global__ void stack_embed_kernel(const T* embed, const T* pos, const int32_t* tok, const int32_t* position, float* h, int W, int ld, int npos) {
    const size_t row = blockIdx.x;
    const T* e = embed + (size_t)tok[row] * W;
    const T* p = pos ? pos + (size_t)min(max(position[row], 0), npos - 1) * W : nullptr;
    if (W == ld) {                                                 // (a multiple of 64)
        for (int i = 4 * threadIdx.x; i < ld; i += 4 * blockDim.x) {
            float4 v = load4<T>(e + i);
            if (p) { const float4 q = load4<T>(p + i); v.x += q.x; v.y += q.y; v.z += q.z; v.w += q.w; }
            *reinterpret_cast<float4*>(h + row * ld + i) = v;
        }
        return;
    }
    for (int i = threadIdx.x; i < ld; i += blockDim.x) h[row * ld + i] = i < W ? to_f(e[i]) + (p ? to_f(p[i]) : 0.f) : 0.f;
}

// latents of positions already in the ring -> scratch rows (a portion that continues a sequence)
template <class T>
__global__ void latent_gather_kernel(const RowPlace* pl, const T* cache, T* c_all, int R, int rank) {
    const RowPlace p = pl[blockIdx.x];
    const T* src = cache + ((size_t)p.slot * R + p.pos % R) * rank;
    for (int r = threadIdx.x; r < rank; r += blockDim.x) c_all[(size_t)p.kv * rank + r] = src[r];
}

// new rows: normalise (and turn) the latent part of the in-projection -> scratch row and, for the last R positions of a sequence, ring
// row; turn the rotated columns of the queries in place
template <class T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const RowPlace* pl, T* in, int ld_in, int off, const float* c_norm, T* cache, T* c_all, int n,
                                                          int R, int rank, int rank_true, float eps, int heads, int D, int dim, int rot, const float* rot_freq) {
    const int i = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (i >= n) return;
    const T* c = in + (size_t)i * ld_in + off;
    float ss = 0.f;
    for (int r = lane; r < rank_true; r += 64) { const float v = to_f(c[r]); ss = fmaf(v, v, ss); }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / rank_true + eps);
    const RowPlace p = pl[i];
    T* ring = cache + ((size_t)p.slot * R + p.pos % R) * rank;
    const int pairs = rot / 2;
    for (int t = lane; t < heads * pairs; t += 64) {
        T* q = in + (size_t)i * ld_in + (t / pairs) * D + dim - rot + 2 * (t % pairs);
        float sn, cs;
        sincosf((float)p.pos * rot_freq[t % pairs], &sn, &cs);
        const float u = to_f(q[0]), v = to_f(q[1]);
        q[0] = from_f<T>(fmaf(u, cs, -v * sn));
        q[1] = from_f<T>(fmaf(v, cs, u * sn));
    }
    for (int r = lane; r < rank; r += 64) {
        const T v = from_f<T>(r >= rank_true && r < rank_true + rot ? rotated(c + rank_true, r - rank_true, p.pos, rot_freq) : to_f(c[r]) * inv * c_norm[r]);
        c_all[(size_t)p.kv * rank + r] = v;
        if (p.store) ring[r] = v;
    }
}

// argmax partials of fp32 logit rows, which are soft-capped on the way (cap 0: not): grid (nblk, rows)
__global__ __launch_bounds__(256) void rows_argmax_kernel(unsigned long long* tl, float* logits, int V, float cap, float* amax_val, int* amax_idx) {
    const TLStamp tls(tl);
    __shared__ float sv[4];
    __shared__ int si[4];
    float* l = logits + (size_t)blockIdx.y * V;
    float bv = -INFINITY;
    int bi = 0x7FFFFFFF;
    for (int i = blockIdx.x * 256 + threadIdx.x; i < V; i += gridDim.x * 256) {
        float v = l[i];
        if (cap > 0.f) l[i] = v = soft_cap(v, cap);
        if (v > bv) { bv = v; bi = i; }
    }
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) {
        const float ov = __shfl_xor(bv, off, 64);
        const int oi = __shfl_xor(bi, off, 64);
        if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    if ((threadIdx.x & 63) == 0) { sv[threadIdx.x >> 6] = bv; si[threadIdx.x >> 6] = bi; }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 4; ++w)
            if (sv[w] > bv || (sv[w] == bv && si[w] < bi)) { bv = sv[w]; bi = si[w]; }
        amax_val[(size_t)blockIdx.y * gridDim.x + blockIdx.x] = bv;
        amax_idx[(size_t)blockIdx.y * gridDim.x + blockIdx.x] = bi;
    }
    tls.end();
}

// -------------------------------------------------------------------------------------------- engine state
static RouterCfg router_of(const pgk_stack_layer_t& L) { return RouterCfg{L.correction, L.experts, L.top, L.groups, L.keep, L.router_scale, L.table}; }
static bool has_experts(const pgk_stack_layer_t& L) { return L.ff_pad && (L.ff == PGK_FF_MOE || L.ff == PGK_FF_TABLE); }
static int router_rows(const pgk_stack_layer_t& L) { return L.ff_pad && L.ff == PGK_FF_MOE ? ceil_div(L.experts, 64) * 64 : 0; }
struct Run { int layer, pass; };          // one pass of one layer; pass >= 0: the loop's pass `pass` starts with it

struct Stack {
    pgk_stack_config_t cfg;
    std::vector<pgk_stack_layer_t> layers;
    std::vector<Run> runs;                 // in the order they are run; without a loop run i is layer i
    int n_runs() const { return (int)runs.size(); }
    const pgk_stack_layer_t& at(int run) const { return layers[runs[run].layer]; }
    const void *embed = nullptr, *pos = nullptr, *head = nullptr;
    const float* final_norm = nullptr;
    int Wp = 0, max_in = 0, max_att = 0, max_ff = 0, max_q = 0, max_top = 0, max_conv = 0, max_z = 0, max_gate = 0, max_low = 0;
    // per run: latent rows [max_batch][R][rank] or K/V rows [max_batch][k, v][kv heads][R][head width] (a layer that takes another
    // one's: that one's pointer) or recurrent states [max_batch][heads][dim][vdim] in fp32
    std::vector<void*> cache;
    std::vector<int> ring, reach;          // R; keys the cache has to keep (the largest window of the layers that read it).  0: no ring
    std::vector<std::vector<std::pair<int, int>>> readers;        // (window, chunked) of the layers that read it, sorted, each once
    // positions before `pos` that a query at `pos` or later may reach through the cache of run `run`
    int past(int run, int pos) const {
        int m = 0;
        for (const auto& r : readers[run]) { const int k = span_keys(pos, r.first, r.second) - 1; m = k > m ? k : m; }
        return m;
    }
    std::vector<void*> taps;               // rings of projected values [max_batch][taps][channels], or null
    std::vector<int32_t> len;              // per slot: positions held (host side; advanced with every step enqueued)
    // decode buffers (rows = max_batch)
    float *in32 = nullptr, *a32 = nullptr, *y32 = nullptr, *act32 = nullptr, *po = nullptr, *pml = nullptr;
    void *qlat = nullptr, *qx = nullptr, *x16 = nullptr, *in16 = nullptr, *a16 = nullptr, *y16 = nullptr, *gu16 = nullptr, *act16 = nullptr;
    float* slabs16 = nullptr;              // split-K slabs of a batch step's projections
    float *y32b = nullptr, *h32 = nullptr, *z32 = nullptr;                          // one row: input of a pass, normed row; rows: decay projections
    int32_t* ids = nullptr;
    float *xs[2] = {nullptr, nullptr}, *xrows = nullptr, *ygate = nullptr;          // hyper-connected layers: streams of one row (two copies), of rows, rows' gates
    void *gate = nullptr, *cat16 = nullptr, *e16 = nullptr, *moe16 = nullptr;       // rows: gates, [x | embedding], experts' rows and workspace
    // fragment-major copies of the layer matrices for 2..128 rows (ops_pkgemm.hip), where its shapes allow; null entries: row-major kernels
    struct Packed { bf16 *in = nullptr, *o = nullptr, *gate_up = nullptr, *down = nullptr; };
    std::vector<Packed> packed;
    size_t slab_elems(int n, bool f32) const;   // fp32 elements the projections of n rows may need
    size_t moe_ws(int n) const {           // workspace of the experts for n rows
        size_t m = 0;
        for (const auto& L : layers)
            if (has_experts(L)) { const size_t z = moe_bytes(n, Wp, L.ff_pad, router_of(L), cfg.dtype); m = z > m ? z : m; }
        return m;
    }
    // prompt buffers, grown on demand outside capture
    void* pf = nullptr; size_t pf_bytes = 0;
    void* tab = nullptr; size_t tab_bytes = 0;
    size_t esize() const { return cfg.dtype == PGK_F32 ? 4 : 2; }
};
static Stack* stack_of(const Engine* e) { return (Stack*)e->kind_state; }
static int kv_source(const pgk_stack_layer_t& L, int l) { return L.kv_from >= 0 ? L.kv_from : l; }
static bool recurrent(const pgk_stack_layer_t& L) { return L.mixer == PGK_MIX_HGRN2 || L.mixer == PGK_MIX_DELTA || L.mixer == PGK_MIX_SSD; }
// channels that pass taps over time before a recurrence, and where the delta rule's projections stand in a row
static int conv_channels(const pgk_stack_layer_t& L) {
    const int V = L.heads * L.vhead_pad, G = L.kv_heads * L.head_pad;
    return L.mixer == PGK_MIX_DELTA || L.mixer == PGK_MIX_SSD ? V + 2 * G : 0;
}
static int delta_a_off(const pgk_stack_layer_t& L) { return ceil_div(conv_channels(L) + L.heads, 64) * 64; }
// the feed-forward that runs for every token (of experts: the shared one): its width and matrices, rows of the first one
static int dense_ff(const pgk_stack_layer_t& L) { return L.ff == PGK_FF_MOE ? 0 : L.ff == PGK_FF_TABLE ? L.shared_pad : L.ff_pad; }
static const void* dense_up(const pgk_stack_layer_t& L) { return L.ff == PGK_FF_TABLE ? L.w_shared_up : L.w_gate_up; }
static const void* dense_down(const pgk_stack_layer_t& L) { return L.ff == PGK_FF_TABLE ? L.w_shared_down : L.w_down; }
static int up_rows(const pgk_stack_layer_t& L) { return (L.ff == PGK_FF_SWIGLU ? 2 : 1) * dense_ff(L); }

static int pick_nsplit(const Engine* e, int B, const pgk_stack_layer_t& L, int R) {
    const int htiles = ceil_div(L.heads, 16);
    int s = ceil_div(R, 64);
    const int want = e->cu_count / (B * htiles) > 0 ? e->cu_count / (B * htiles) : 1;      // one workgroup per CU (its LDS)
    if (s > want) s = want;
    return s > 64 ? 64 : (s < 1 ? 1 : s);
}

constexpr int LATENT_LDS_MAX = 144 * 1024;
#define PGK_ALLOW_LDS(kfn, lds)                                                                                                   \
    {                                                                                                                              \
        static bool done = false;                                                                                                  \
        if ((lds) > 48 * 1024 && !done) {                                                                                          \
            if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, LATENT_LDS_MAX)) return e; \
            done = true;                                                                                                           \
        }                                                                                                                          \
    }

template <class T, int RC>
static hipError_t launch_latent_attn(const LatentArgs& a, hipStream_t st) {
    return launch_k(&latent_attn_kernel<T, RC, 4>, dim3(a.nsplit, ceil_div(a.H, 4), a.B), dim3(256), (size_t)4 * a.rank * 4, st, a);
}
template <int RT>
static hipError_t launch_latent_mfma(const LatentArgs& a, hipStream_t st) {
    const size_t lds = latent_mfma_lds(a.rank);
    PGK_ALLOW_LDS(&latent_attn_mfma_kernel<RT>, lds)
    return launch_k(&latent_attn_mfma_kernel<RT>, dim3(a.nsplit, ceil_div(a.H, 16), a.B), dim3(256), lds, st, a);
}
template <class T, class IT, int MB, int PF>
static hipError_t launch_merge_uv(const LatentArgs& a, hipStream_t st) {
    const size_t lds = (size_t)4 * MB * a.rank * 4;
    auto kfn = &latent_merge_uv_kernel<T, IT, MB, PF>;
    PGK_ALLOW_LDS(kfn, lds)
    return launch_k(kfn, dim3(a.H, ceil_div(a.vdim, 32 * a.vc), ceil_div(a.B, MB)), dim3(256), lds, st, a);
}
template <class T, class IT, class QT, int MB>
static hipError_t launch_absorb(const LatentArgs& a, hipStream_t st) {
    return launch_k(&latent_absorb_kernel<T, IT, QT, MB>, dim3(a.H * ceil_div(a.rank, 128) + 1, ceil_div(a.B, MB)), dim3(256), 0, st, a);
}

// absorb -> attention over the ring -> merge + U_v + gate for B sequences whose in-projection rows are in `in`
template <class T, class IT>
static pgk_status latent_decode(Engine* e, int l, int B, const void* in, void* out, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& L = s->at(l);
    constexpr bool F32 = std::is_same<T, float>::value;
    LatentArgs a{};
    a.in = in; a.ld_in = L.n_in; a.qn = L.heads * L.head_pad; a.g_off = L.gated ? a.qn + L.rank_pad : -1; a.rot = L.rot; a.rot_freq = L.rot_freq;
    a.w_uk = L.w_ukv; a.w_uv = (const char*)L.w_ukv + (size_t)L.heads * L.head_pad * L.rank_pad * sizeof(T);
    a.c_norm = L.c_norm; a.cache = s->cache[l]; a.positions = e->positions;
    a.B = B; a.H = L.heads; a.D = L.head_pad; a.dim = L.dim; a.vdim = L.vdim; a.rank = L.rank_pad; a.rank_true = L.rank; a.R = s->ring[l];
    a.nsplit = pick_nsplit(e, B, L, a.R);
    a.vc = B >= 16 ? 4 : 1;      // many sequences: fewer workgroups, each combines its records once for all its rows
    a.eps = s->cfg.norm_eps; a.scale = L.scale * LOG2E;
    a.qlat = s->qlat; a.po = s->po; a.pml = s->pml; a.out = out; a.ld_out = L.heads * L.head_pad;
    const bool mfma = !F32 && a.rank <= 896;
    if (!mfma) {
        PGK_CHECK_HIP((B == 1 ? launch_absorb<T, IT, float, 1>(a, st) : launch_absorb<T, IT, float, 4>(a, st)));
        if (a.rank <= 64) PGK_CHECK_HIP((launch_latent_attn<T, 1>(a, st)));
        else if (a.rank <= 128) PGK_CHECK_HIP((launch_latent_attn<T, 2>(a, st)));
        else if (a.rank <= 256) PGK_CHECK_HIP((launch_latent_attn<T, 4>(a, st)));
        else if (a.rank <= 512) PGK_CHECK_HIP((launch_latent_attn<T, 8>(a, st)));
        else if (a.rank <= 1024) PGK_CHECK_HIP((launch_latent_attn<T, 16>(a, st)));
        else PGK_CHECK_HIP((launch_latent_attn<T, 32>(a, st)));
    }
    if constexpr (!F32) {
        if (mfma) {
            PGK_CHECK_HIP((B == 1 ? launch_absorb<T, IT, bf16, 1>(a, st) : B < 32 ? launch_absorb<T, IT, bf16, 4>(a, st) : launch_absorb<T, IT, bf16, 8>(a, st)));
            if (a.rank <= 64) PGK_CHECK_HIP(launch_latent_mfma<1>(a, st));
            else if (a.rank <= 128) PGK_CHECK_HIP(launch_latent_mfma<2>(a, st));
            else if (a.rank <= 256) PGK_CHECK_HIP(launch_latent_mfma<4>(a, st));
            else if (a.rank <= 512) PGK_CHECK_HIP(launch_latent_mfma<8>(a, st));
            else PGK_CHECK_HIP(launch_latent_mfma<14>(a, st));
        }
    }
    if constexpr (!F32) {
        if (a.rank <= 256) PGK_CHECK_HIP((B < 16 ? launch_merge_uv<T, IT, 1, 2>(a, st) : launch_merge_uv<T, IT, 4, 2>(a, st)));
        else if (a.rank <= 512) PGK_CHECK_HIP((B < 16 ? launch_merge_uv<T, IT, 1, 4>(a, st) : launch_merge_uv<T, IT, 4, 4>(a, st)));
        else PGK_CHECK_HIP((B < 16 ? launch_merge_uv<T, IT, 1, 0>(a, st) : launch_merge_uv<T, IT, 4, 0>(a, st)));
    } else PGK_CHECK_HIP((B < 16 ? launch_merge_uv<T, IT, 1, 0>(a, st) : launch_merge_uv<T, IT, 4, 0>(a, st)));
    *launches += 3;
    return PGK_OK;
}

// taps and norms -> attention over the ring (split) -> combine and gate
template <class T, class IT>
static pgk_status attention_decode(Engine* e, int l, int B, const void* in, void* out, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& L = s->at(l);
    const int src = kv_source(L, l), HD = L.heads * L.head_pad, GD = L.kv_from >= 0 ? 0 : L.kv_heads * L.head_pad;
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    constexpr bool IO32 = std::is_same<IT, float>::value;
    ConvArgs c{};
    c.in = in; c.ld_in = L.n_in; c.bias = L.b_in; c.conv = L.conv; c.taps = L.taps; c.n_q = HD; c.n_kv = GD; c.D = L.head_pad; c.n = B; c.R = s->ring[src];
    c.q_norm = L.q_norm; c.k_norm = L.k_norm; c.q_true = L.heads * L.dim; c.k_true = L.kv_heads * L.dim; c.eps = s->cfg.norm_eps; c.q_mult = L.scale * LOG2E;
    c.tap_ring = s->taps[l]; c.positions = e->positions; c.q_out = s->qx; c.ld_q = HD; c.cache = s->cache[src];
    if (pgk_status r = conv_rows(c, DT, IO32, kv_attn_q32(L.head_pad, DT), st)) return r;
    KvAttnArgs a{};
    a.q = s->qx; a.cache = s->cache[src]; a.slopes = L.slopes; a.positions = e->positions;
    a.B = B; a.H = L.heads; a.G = L.kv_heads; a.D = L.head_pad; a.R = s->ring[src]; a.window = L.window;
    a.nsplit = kv_attn_splits(B, L.heads, L.kv_heads, L.window < a.R ? L.window : a.R, e->cu_count);
    a.po = s->po; a.pml = s->pml; a.gate = (const IT*)in + HD + 2 * GD; a.ld_gate = L.n_in; a.out = out; a.ld_out = HD;
    *launches += 1;
    return kv_attn_decode(a, DT, IO32, st, launches);
}

static HeadRowsArgs head_args(const Stack* s, int l, const void* in, int n) {
    const auto& L = s->at(l);
    HeadRowsArgs a{};
    a.in = in; a.ld_in = L.n_in; a.bias = L.b_in; a.q_norm = L.q_norm; a.k_norm = L.k_norm; a.H = L.heads; a.G = L.kv_from >= 0 ? 0 : L.kv_heads; a.D = L.head_pad; a.dim = L.dim;
    a.rot = L.rot; a.rot_freq = L.rot_freq; a.n = n; a.R = s->ring[kv_source(L, l)]; a.eps = s->cfg.norm_eps; a.ld_q = L.heads * L.head_pad; a.cache = s->cache[kv_source(L, l)];
    return a;
}
static TalkArgs talk_args(const Stack* s, int l, int n, void* out) {
    const auto& L = s->at(l);
    TalkArgs a{};
    a.ld_q = L.heads * L.head_pad; a.talk = L.talk; a.sink = L.sink; a.H = L.heads; a.G = L.kv_heads; a.D = L.head_pad; a.n = n; a.window = L.window; a.chunked = L.chunked;
    a.scale = L.scale; a.nsplit = 1; a.out = out; a.ld_out = L.n_att;
    return a;
}

// norms and rotation, new k and v -> ring -> attention over it (split) -> combine
template <class T, class IT>
static pgk_status talk_decode(Engine* e, int l, int B, const void* in, void* out, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& L = s->at(l);
    const int src = kv_source(L, l);
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    constexpr bool IO32 = std::is_same<IT, float>::value;
    HeadRowsArgs h = head_args(s, l, in, B);
    h.positions = e->positions; h.q_out = s->qx;
    if (pgk_status r = head_rows(h, DT, IO32, st)) return r;
    TalkArgs a = talk_args(s, l, B, out);
    a.q = s->qx; a.cache = s->cache[src]; a.positions = e->positions; a.R = s->ring[src];
    a.nsplit = talk_splits(B, L.heads, L.kv_heads, L.window < a.R ? L.window : a.R, e->cu_count);
    a.po = s->po; a.pml = s->pml;
    *launches += 1;
    return talk_attention(a, DT, IO32, st, launches);
}

static RecurArgs recur_args(const Stack* s, int l, const void* in, void* out, int n) {
    const auto& L = s->at(l);
    RecurArgs a{};
    a.in = in; a.ld_in = L.n_in; a.H = L.heads; a.dim = L.head_pad; a.vdim = L.vhead_pad; a.vdim_true = L.vdim; a.n = n; a.eps = s->cfg.norm_eps;
    a.state = (float*)s->cache[l]; a.out = out; a.ld_out = L.n_att;
    if (L.mixer == PGK_MIX_SSD) {          // x | B | C | z | dt; the norm in parts is a launch of its own
        const int V = L.heads * L.vhead_pad, G = L.kv_heads * L.head_pad;
        a.kind = RECUR_SSD; a.G = L.kv_heads; a.f_off = V; a.q_off = V + G; a.z_off = V + 2 * G; a.dt_off = a.z_off + V;
        a.dt_bias = L.dt_bias; a.decay = L.decay; a.skip = L.skip;
        a.conv = ConvStep{L.conv, L.conv_bias, L.taps, conv_channels(L), s->taps[l]};
        return a;
    }
    a.f_off = L.heads * L.head_pad; a.v_off = 2 * a.f_off;
    a.bias = L.b_in ? L.b_in + a.f_off : nullptr; a.lower = L.lower; a.norm = L.o_norm;
    return a;
}
static pgk_status ssd_norm(const Stack* s, int l, void* rows, int n, pgk_dtype dt, hipStream_t st) {
    const auto& L = s->at(l);
    return parts_norm(rows, L.n_att, n, L.heads, L.vhead_pad, L.vdim, L.norm_parts, L.o_norm, s->cfg.norm_eps, dt, st);
}

static DeltaArgs delta_args(const Stack* s, int l, const void* in, const float* z, const void* gate, void* out, int n) {
    const auto& L = s->at(l);
    DeltaArgs a{};
    a.in = in; a.ld_in = L.n_in; a.b_off = conv_channels(L);
    a.z = z; a.ld_z = L.heads * L.head_pad; a.gate = gate; a.ld_gate = L.heads * L.vhead_pad;
    a.conv = ConvStep{L.conv, nullptr, L.taps, conv_channels(L), s->taps[l]};
    a.decay = L.decay; a.dt_bias = L.dt_bias; a.norm = L.o_norm;
    a.H = L.heads; a.G = L.kv_heads; a.dim = L.head_pad; a.vdim = L.vhead_pad; a.dim_true = L.dim; a.vdim_true = L.vdim; a.n = n; a.eps = s->cfg.norm_eps;
    a.state = (float*)s->cache[l]; a.out = out; a.ld_out = L.n_att;
    return a;
}

// The mixer of layer l for the next token of B sequences: in-projection rows `in` -> out-projection rows `out`
template <class T, class IT>
static pgk_status mix_decode(Engine* e, int l, int B, const void* in, void* out, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& L = s->at(l);
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16, IDT = std::is_same<IT, float>::value ? PGK_F32 : PGK_BF16;
    constexpr bool IO32 = std::is_same<IT, float>::value;
    switch (L.mixer) {
        case PGK_MIX_LATENT: return latent_decode<T, IT>(e, l, B, in, out, st, launches);
        case PGK_MIX_ATTENTION: return attention_decode<T, IT>(e, l, B, in, out, st, launches);
        case PGK_MIX_TALK: return talk_decode<T, IT>(e, l, B, in, out, st, launches);
        case PGK_MIX_DELTA: {
            const int a_off = delta_a_off(L);
            if (pgk_status r = lowrank_rows(in, L.n_in, B, a_off, L.rank_a, L.w_a2, s->z32, L.heads * L.head_pad, a_off + L.rank_a, L.rank_g, L.w_g2, s->gate, L.heads * L.vhead_pad,
                                            DT, IO32, st))
                return r;
            DeltaArgs a = delta_args(s, l, in, s->z32, s->gate, out, B);
            a.positions = e->positions;
            *launches += 2;
            return delta_rows(a, DT, IO32, st);
        }
        default: {
            RecurArgs a = recur_args(s, l, in, out, B);
            a.positions = e->positions;
            *launches += 1;
            if (pgk_status r = recur_rows(a, DT, IO32, st)) return r;
            if (L.mixer != PGK_MIX_SSD) return PGK_OK;
            *launches += 1;
            return ssd_norm(s, l, out, B, IDT, st);
        }
    }
}

// Parallel layers, one sequence
template <class T>
static pgk_status step_parallel(Engine* e, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& c = s->cfg;
    float *x = e->h, *xn = e->h2;
    const float *pend = nullptr, *base = nullptr;      // what is still to be added to the stream (or to the vector that takes its place)
    auto input = [&](StackGemvArgs& a, int K) {
        a.K = K; a.W = c.width; a.x = x; a.eps = c.norm_eps; a.mult = base ? 1.f : c.residual_mult; a.y = pend; a.base = base;
    };
    auto norm_in = [&](StackGemvArgs& a, const float* gamma) {
        input(a, s->Wp);
        a.gamma = gamma; a.layer_norm = c.layer_norm;
        a.x_out = pend ? xn : nullptr;
    };
    for (int l = 0; l < s->n_runs(); ++l) {
        const auto& L = s->at(l);
        const int er = router_rows(L);
        StackGemvArgs a{};
        mark(KC_NORM_QKV);
        if (s->runs[l].pass >= 0) {
            input(a, 2 * s->Wp);
            a.embed = s->embed; a.tok = e->tokens; a.w = c.loop_in; a.N = s->Wp; a.out = s->y32b;
            if (pgk_status r = stack_gemv<T, SP_CAT, SE_STORE>(a, st)) return r;
            pend = s->y32b;
            base = c.loop_step + (size_t)s->runs[l].pass * s->Wp;
            *launches += 1;
            a = StackGemvArgs{};
        }
        norm_in(a, L.norm1);
        a.h_out = er ? s->h32 : nullptr;
        a.w = L.w_in; a.N = L.n_in + er; a.out = s->in32;
        if (pgk_status r = stack_gemv<T, SP_ADD, SE_STORE>(a, st)) return r;
        if (pend) { float* t = x; x = xn; xn = t; }
        mark(recurrent(L) ? KC_RECUR : KC_ATTN);
        if (pgk_status r = mix_decode<T, float>(e, l, 1, s->in32, s->a32, st, launches)) return r;
        MoeOneArgs m{};
        m.r = router_of(L); m.W = s->Wp; m.ff = L.ff_pad; m.logits = s->in32 + L.n_in; m.h = s->h32; m.w_up = L.w_gate_up; m.w_down = L.w_down; m.act = s->act32; m.ids = s->ids;
        m.w_o = L.w_o; m.a = s->a32; m.n_att = L.n_att; m.y = s->y32; m.N = s->Wp;
        if (er) {
            mark(KC_GATEUP);
            if (pgk_status r = moe_up_one<T>(m, st)) return r;
            mark(KC_DOWN);
            if (pgk_status r = moe_out_one<T>(m, st)) return r;
            *launches += 1;
        } else {
            mark(KC_OPROJ);
            a = StackGemvArgs{};
            a.w = L.w_o; a.N = s->Wp; a.K = L.n_att; a.x = s->a32; a.out = s->y32;
            if (pgk_status r = stack_gemv<T, SP_PLAIN, SE_STORE>(a, st)) return r;
        }
        pend = s->y32; base = nullptr;
        *launches += 2;
    }
    mark(KC_LMHEAD);
    StackGemvArgs a{};
    norm_in(a, s->final_norm);
    a.x_out = nullptr;
    a.w = s->head; a.N = c.vocab_size; a.out = e->logits; a.amax_val = e->amax_val; a.amax_idx = e->amax_idx;
    if (pgk_status r = stack_gemv<T, SP_ADD, SE_LOGITS>(a, st, e->lm_blocks)) return r;
    *launches += 1;
    return PGK_OK;
}

// Hyper-connected layers, one sequence
template <class T>
static pgk_status step_hyper(Engine* e, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& c = s->cfg;
    const float *x = e->h, *pend = nullptr;   // the streams (at first all the embedded row), the numbers of the sublayer whose output waits in y32
    int stream = 0, buf = 0;
    auto input = [&](StackGemvArgs& a, const float* in, const float* gamma) {
        a.K = s->Wp; a.W = c.width; a.x = x; a.x_stream = stream; a.S = c.streams; a.groups = c.norm_groups; a.in = in; a.gamma = gamma; a.eps = c.norm_eps;
        if (pend) { a.y = s->y32; a.upd = pend; a.x_out = s->xs[buf]; }
    };
    auto settle = [&]() {
        if (!pend) return;
        x = s->xs[buf]; stream = s->Wp; buf ^= 1;
        pend = nullptr;
    };
    for (int l = 0; l < c.num_layers; ++l) {
        const auto& L = s->layers[l];
        StackGemvArgs a{};
        mark(KC_NORM_QKV);
        input(a, L.hyper1, L.norm1);
        a.w = L.w_in; a.N = L.n_in; a.out = s->in32;
        if (pgk_status r = stack_gemv<T, SP_HYPER, SE_STORE>(a, st)) return r;
        settle();
        mark(KC_ATTN);
        if (pgk_status r = mix_decode<T, float>(e, l, 1, s->in32, s->a32, st, launches)) return r;
        mark(KC_OPROJ);
        a = StackGemvArgs{};
        a.w = L.w_o; a.N = s->Wp; a.K = L.n_att; a.x = s->a32; a.out = s->y32; a.bias = L.b_o;
        if (pgk_status r = stack_gemv<T, SP_PLAIN, SE_STORE>(a, st)) return r;
        pend = L.hyper1;
        *launches += 2;
        if (!L.ff_pad) continue;
        mark(KC_GATEUP);
        a = StackGemvArgs{};
        input(a, L.hyper2, L.norm2);
        a.out = s->act32;
        if (L.ff == PGK_FF_TABLE) {
            a.w = L.w_shared_up; a.w2 = L.w_gate_up; a.w3 = L.w_shared_gate; a.table = L.table; a.tok = e->tokens; a.fs = L.shared_pad; a.top = L.top; a.ff = L.ff_pad; a.ids = s->ids;
            a.N = L.shared_pad + L.top * L.ff_pad + (L.shared_pad ? 1 : 0);
            if (pgk_status r = stack_gemv<T, SP_HYPER, SE_TABLE>(a, st)) return r;
        } else {
            a.w = L.w_gate_up; a.N = L.ff_pad;
            if (pgk_status r = stack_gemv<T, SP_HYPER, SE_STORE>(a, st)) return r;
        }
        settle();
        mark(KC_DOWN);
        if (L.ff == PGK_FF_TABLE) {
            MoeOneArgs m{};
            m.r = router_of(L); m.ff = L.ff_pad; m.w_down = L.w_down; m.act = s->act32 + L.shared_pad; m.ids = s->ids; m.w_o = L.w_shared_down; m.a = s->act32; m.n_att = L.shared_pad;
            m.gate = L.shared_pad ? s->act32 + L.shared_pad + L.top * L.ff_pad : nullptr; m.y = s->y32; m.N = s->Wp;
            if (pgk_status r = moe_out_one<T>(m, st)) return r;
        } else {
            a = StackGemvArgs{};
            a.w = L.w_down; a.N = s->Wp; a.K = L.ff_pad; a.W = L.ff_dim; a.eps = c.norm_eps; a.act = L.act; a.x = s->act32; a.out = s->y32;
            if (pgk_status r = stack_gemv<T, SP_POLY, SE_STORE>(a, st)) return r;
        }
        pend = L.hyper2;
        *launches += 2;
    }
    mark(KC_LMHEAD);
    StackGemvArgs a{};
    input(a, nullptr, s->final_norm);
    a.x_out = nullptr;
    a.w = s->head; a.N = c.vocab_size; a.out = e->logits; a.cap = c.logit_cap; a.amax_val = e->amax_val; a.amax_idx = e->amax_idx;
    if (pgk_status r = stack_gemv<T, SP_HYPER, SE_LOGITS>(a, st, e->lm_blocks)) return r;
    *launches += 1;
    return PGK_OK;
}

// ---- one sequence: fused steps, fp32 between kernels ----
template <class T>
static pgk_status step_one(Engine* e, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    const auto& c = s->cfg;
    float *x = e->h, *xn = e->h2;
    const float* pend = nullptr;              // post-norm weight of the sublayer output waiting in y32
    auto norm_in = [&](StackGemvArgs& a, const float* gamma) {
        a.K = s->Wp; a.W = c.width; a.x = x; a.gamma = gamma; a.eps = c.norm_eps; a.mult = c.residual_mult;
        if (pend) { a.y = s->y32; a.g_post = pend; a.x_out = xn; }
    };
    auto settle = [&]() { if (pend) { float* t = x; x = xn; xn = t; } pend = nullptr; };
    for (int l = 0; l < c.num_layers; ++l) {
        const auto& L = s->layers[l];
        StackGemvArgs a{};
        mark(KC_NORM_QKV);
        norm_in(a, L.norm1);
        a.w = L.w_in; a.N = L.n_in; a.out = s->in32;
        if (pgk_status r = stack_gemv<T, SP_NORM, SE_STORE>(a, st)) return r;
        settle();
        mark(recurrent(L) ? KC_RECUR : KC_ATTN);
        if (pgk_status r = mix_decode<T, float>(e, l, 1, s->in32, s->a32, st, launches)) return r;
        mark(KC_OPROJ);
        a = StackGemvArgs{};
        a.w = L.w_o; a.N = s->Wp; a.K = L.n_att; a.x = s->a32; a.out = s->y32;
        if (pgk_status r = stack_gemv<T, SP_PLAIN, SE_STORE>(a, st)) return r;
        pend = L.norm1b;
        *launches += 2;
        if (!L.ff_pad) continue;
        mark(KC_GATEUP);
        a = StackGemvArgs{};
        norm_in(a, L.norm2);
        a.w = L.w_gate_up; a.N = L.ff_pad; a.out = s->act32;
        a.act_pos = L.act_pos; a.act_neg = L.act_neg;
        if (pgk_status r = L.ff == PGK_FF_SWIGLU ? stack_gemv<T, SP_NORM, SE_SWIGLU>(a, st) : stack_gemv<T, SP_NORM, SE_XIELU>(a, st)) return r;
        settle();
        mark(KC_DOWN);
        a = StackGemvArgs{};
        a.w = L.w_down; a.N = s->Wp; a.K = L.ff_pad; a.x = s->act32; a.out = s->y32;
        if (pgk_status r = stack_gemv<T, SP_PLAIN, SE_STORE>(a, st)) return r;
        pend = L.norm2b;
        *launches += 2;
    }
    mark(KC_LMHEAD);
    StackGemvArgs a{};
    norm_in(a, s->final_norm);
    a.x_out = nullptr;
    a.w = s->head; a.N = c.vocab_size; a.out = e->logits; a.amax_val = e->amax_val; a.amax_idx = e->amax_idx;
    if (pgk_status r = stack_gemv<T, SP_NORM, SE_LOGITS>(a, st, e->lm_blocks)) return r;
    *launches += 1;
    return PGK_OK;
}

// fp32 logits of `n` normalised rows (element type T, row stride Wp), before any soft cap
template <class T>
static pgk_status logit_rows(Stack* s, const T* x, float* logits, int n, hipStream_t st) {
    const int V = s->cfg.vocab_size;
    if constexpr (std::is_same<T, float>::value) return pgk_gemm_nt(x, s->head, nullptr, logits, n, V, s->Wp, PGK_F32, st);
    for (int r = 0; r < n; r += 128) {
        const int m = n - r < 128 ? n - r : 128;
        if (pgk_status q = wsgemm_nt((const bf16*)x + (size_t)r * s->Wp, s->Wp, s->head, nullptr, false, logits + (size_t)r * V, nullptr, 1, 1, m, V, s->Wp, st)) return q;
    }
    return PGK_OK;
}

struct RowBufs {
    float* h; void *x, *in, *a, *y, *gu, *act; float* slabs; void* q;
    void *cat, *e, *moe; const int32_t* tok;      // parallel layers: [x | embedding] rows, experts' rows, their workspace, the rows' tokens
    float *xs, *ygate;                            // hyper-connected layers: streams [n][S][Wp], gates of the shared experts
};

// How a [N, K] projection of n bf16 rows runs: fragment-major copy (<= 128 rows), weight-streaming kernel (<= 128 rows) or tiled
// MFMA, and over how many split-K slabs its result is left (0: one bf16 result).
struct ProjPlan { bool pk; int slabs; };
static ProjPlan plan_proj(const bf16* packed, int n, int N, int K, bool split) {
    if (n <= 128) {
        if (packed) return {true, split ? pkgemm_pick_splits(n, N, K) : 0};
        const int s = split && n > 1 ? wsgemm_pick_splits(N, K, true) : 1;
        return {false, s > 1 ? s : 0};
    }
    const int s = split ? engine_gemm_pick_splits(n, N, K) : 1;
    return {false, s > 1 ? s : 0};
}
// fp32 results of n bf16 rows, as one or more slabs
static int plan_f32(int n, int N, int K) { return n <= 128 ? wsgemm_pick_splits(N, K, true) : engine_gemm_pick_splits(n, N, K); }
static pgk_status gemm_f32(const void* x, const void* w, float* out, int splits, int n, int N, int K, hipStream_t st) {
    if (n <= 128) return wsgemm_nt((const bf16*)x, K, w, nullptr, false, out, nullptr, 1, splits, n, N, K, st);
    return engine_gemm_nt_slabs((const bf16*)x, w, out, splits, n, N, K, st);
}
size_t Stack::slab_elems(int n, bool f32) const {
    size_t m = 64;
    if (f32) return m;
    if (cfg.loop_times) m = (size_t)plan_f32(n, Wp, 2 * Wp) * n * Wp;
    for (size_t l = 0; l < layers.size(); ++l) {
        const auto& L = layers[l];
        const Packed P = packed.empty() ? Packed{} : packed[l];
        const size_t need[] = {(size_t)plan_proj(P.o, n, Wp, L.n_att, true).slabs * n * Wp,
                               dense_ff(L) ? (size_t)plan_proj(P.down, n, Wp, dense_ff(L), true).slabs * n * Wp : 0,
                               P.in || n > 128 ? 0 : (size_t)plan_proj(nullptr, n, L.n_in, Wp, true).slabs * n * L.n_in,
                               L.ff != PGK_FF_POLY || P.gate_up || n > 128 ? 0 : (size_t)plan_proj(nullptr, n, L.ff_pad, Wp, true).slabs * n * L.ff_pad};
        for (size_t z : need) m = z > m ? z : m;
    }
    return m;
}

// bf16 rows = sum of fp32 slabs
__global__ __launch_bounds__(256) void slab_rows_kernel(const float* slabs, int ns, bf16* out, size_t n4) {
    for (size_t i = blockIdx.x * (size_t)256 + threadIdx.x; i < n4; i += (size_t)gridDim.x * 256) {
        float4 t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int s = 0; s < ns; ++s) {
            const float4 q = reinterpret_cast<const float4*>(slabs)[s * n4 + i];
            t.x += q.x; t.y += q.y; t.z += q.z; t.w += q.w;
        }
        store4<bf16>(out + 4 * i, t);
    }
}

// A sublayer's last projection: y rows in the element type, or *slabs split-K slabs for the norm that follows
template <class T>
static pgk_status rows_out_proj(Stack* s, const RowBufs& b, const void* x, const void* w, const bf16* packed, int n, int K, int* slabs, hipStream_t st) {
    *slabs = 0;
    if constexpr (std::is_same<T, float>::value) return pgk_gemm_nt(x, w, nullptr, b.y, n, s->Wp, K, PGK_F32, st);
    const ProjPlan p = plan_proj(packed, n, s->Wp, K, true);
    *slabs = p.slabs;
    if (p.pk) return pkgemm_nt((const bf16*)x, K, packed, b.slabs, s->Wp, PK_EPI_SLAB, p.slabs, n, s->Wp, K, nullptr, st);
    if (!p.slabs) return pgk_gemm_nt(x, w, nullptr, b.y, n, s->Wp, K, PGK_BF16, st);
    if (n <= 128) return wsgemm_nt((const bf16*)x, K, w, nullptr, false, b.slabs, nullptr, 1, p.slabs, n, s->Wp, K, st);
    return engine_gemm_nt_slabs((const bf16*)x, w, b.slabs, p.slabs, n, s->Wp, K, st);
}

// out = x W^T in the element type, K = Wp
template <class T>
static pgk_status rows_proj(Stack* s, const RowBufs& b, const void* w, const bf16* packed, void* out, int n, int N, hipStream_t st) {
    if constexpr (std::is_same<T, float>::value) return pgk_gemm_nt(b.x, w, nullptr, out, n, N, s->Wp, PGK_F32, st);
    if (n <= 128 && packed) return pkgemm_nt((const bf16*)b.x, s->Wp, packed, out, N, PK_EPI_BF16, 1, n, N, s->Wp, nullptr, st);
    const int slabs = n <= 128 ? plan_proj(nullptr, n, N, s->Wp, true).slabs : 0;
    if (!slabs) return pgk_gemm_nt(b.x, w, nullptr, out, n, N, s->Wp, PGK_BF16, st);
    if (pgk_status r = wsgemm_nt((const bf16*)b.x, s->Wp, w, nullptr, false, b.slabs, nullptr, 1, slabs, n, N, s->Wp, st)) return r;
    const size_t n4 = (size_t)n * N / 4;
    slab_rows_kernel<<<(unsigned)(n4 / 256 > 2048 ? 2048 : (n4 + 255) / 256), 256, 0, st>>>(b.slabs, slabs, (bf16*)out, n4);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}
template <class T>
static pgk_status rows_in_proj(Stack* s, const pgk_stack_layer_t& L, const bf16* packed, const RowBufs& b, int n, hipStream_t st) {
    return rows_proj<T>(s, b, L.w_in, packed, b.in, n, L.n_in, st);
}

// first feed-forward projection of n rows: act = silu(x W_g) * (x W_u), xIELU(x W_u), or (a shared expert) gelu(x W_u)
template <class T>
static pgk_status rows_gate_up(Stack* s, const pgk_stack_layer_t& L, const bf16* packed, const RowBufs& b, int n, hipStream_t st) {
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    if (L.ff == PGK_FF_XIELU || L.ff == PGK_FF_TABLE) {
        const bool gelu = L.ff == PGK_FF_TABLE;
        const int ff = dense_ff(L);
        const void* w = dense_up(L);
        if (DT == PGK_BF16 && n <= 128 && packed) {
            PkArgs g{};
            g.act_pos = L.act_pos; g.act_neg = L.act_neg;
            return pkgemm_nt((const bf16*)b.x, s->Wp, packed, b.act, ff, gelu ? PK_EPI_GELU : PK_EPI_XIELU, 1, n, ff, s->Wp, &g, st);
        }
        if (DT == PGK_BF16 && engine_gemm_act_ok(n, ff, s->Wp))
            return engine_gemm_act_nt((const bf16*)b.x, (const bf16*)w, (bf16*)b.act, n, ff, s->Wp, ActArgs{L.act_pos, L.act_neg, gelu}, st);
        if (pgk_status r = pgk_gemm_nt(b.x, w, nullptr, b.act, n, ff, s->Wp, DT, st)) return r;
        return gelu ? pgk_gelu_erf(b.act, b.act, (size_t)n * ff, DT, st) : pgk_xielu(b.act, b.act, (size_t)n * ff, L.act_pos, L.act_neg, DT, st);
    }
    if (DT == PGK_BF16 && n <= 128 && packed)
        return pkgemm_nt((const bf16*)b.x, s->Wp, packed, b.act, L.ff_pad, PK_EPI_SWIGLU, 1, n, 2 * L.ff_pad, s->Wp, nullptr, st);
    if (DT == PGK_BF16 && engine_gemm_swiglu_ok(n, L.ff_pad, s->Wp, false))
        return engine_gemm_swiglu_nt((const bf16*)b.x, L.w_gate_up, nullptr, false, (bf16*)b.act, n, L.ff_pad, s->Wp, st);
    if (pgk_status r = pgk_gemm_nt(b.x, L.w_gate_up, nullptr, b.gu, n, 2 * L.ff_pad, s->Wp, DT, st)) return r;
    return pgk_glu_packed(b.gu, b.act, n, L.ff_pad, 0, DT, st);
}

struct Pending { const float* gain = nullptr; int slabs = 0; };     // the sublayer output whose norm and residual add are still to come

static RowsNormArgs norm_args(const Stack* s, const RowBufs& b, int n, const Pending& p, const float* gamma, void* out) {
    RowsNormArgs a{};
    a.h = b.h; a.y = !p.gain ? nullptr : p.slabs ? (const void*)b.slabs : b.y; a.ldy = s->Wp; a.g_post = p.gain; a.mult = s->cfg.residual_mult;
    a.gamma = gamma; a.out = out; a.W = s->cfg.width; a.ld = s->Wp; a.eps = s->cfg.norm_eps; a.store_h = 1;
    a.nslabs = p.gain ? p.slabs : 0; a.slab_stride = (long long)n * s->Wp;
    return a;
}

// The layers on n rows of b.h; `mix(l)` turns in-projection rows b.in into attention rows b.a.  Leaves the last sublayer pending.
template <class T, class Mix>
static pgk_status rows_layers(Stack* s, const RowBufs& b, int n, hipStream_t st, Pending* pend, Mix mix) {
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    *pend = Pending{};
    for (int l = 0; l < s->cfg.num_layers; ++l) {
        const auto& L = s->layers[l];
        const Stack::Packed P = s->packed.empty() ? Stack::Packed{} : s->packed[l];
        mark(KC_NORM_QKV);
        if (pgk_status r = rows_norm(norm_args(s, b, n, *pend, L.norm1, b.x), n, DT, st)) return r;
        if (pgk_status r = rows_in_proj<T>(s, L, P.in, b, n, st)) return r;
        mark(recurrent(L) ? KC_RECUR : KC_ATTN);
        if (pgk_status r = mix(l)) return r;
        mark(KC_OPROJ);
        if (pgk_status r = rows_out_proj<T>(s, b, b.a, L.w_o, P.o, n, L.n_att, &pend->slabs, st)) return r;
        pend->gain = L.norm1b;
        if (!L.ff_pad) continue;
        mark(KC_GATEUP);
        if (pgk_status r = rows_norm(norm_args(s, b, n, *pend, L.norm2, b.x), n, DT, st)) return r;
        if (pgk_status r = rows_gate_up<T>(s, L, P.gate_up, b, n, st)) return r;
        mark(KC_DOWN);
        if (pgk_status r = rows_out_proj<T>(s, b, b.act, L.w_down, P.down, n, L.ff_pad, &pend->slabs, st)) return r;
        pend->gain = L.norm2b;
    }
    return PGK_OK;
}

// Parallel layers: what is still to be added to the stream, y rows (or slabs) on the stream or on `base`, and the experts' rows
struct PendingAdd { bool y = false; int slabs = 0, top = 0; const float* base = nullptr; };

static RowsNormArgs add_args(const Stack* s, const RowBufs& b, int n, const PendingAdd& p, const float* gamma, void* out) {
    RowsNormArgs a{};
    a.plain = 1; a.layer_norm = s->cfg.layer_norm;
    a.h = b.h; a.y = !p.y ? nullptr : p.slabs ? (const void*)b.slabs : b.y; a.ldy = s->Wp; a.mult = p.base ? 1.f : s->cfg.residual_mult;
    a.gamma = gamma; a.out = out; a.W = s->cfg.width; a.ld = s->Wp; a.eps = s->cfg.norm_eps; a.store_h = p.y;
    a.nslabs = p.y ? p.slabs : 0; a.slab_stride = (long long)n * s->Wp;
    a.base = p.base; a.e = p.top ? b.e : nullptr; a.e_top = p.top;
    return a;
}

template <class T, class Mix>
static pgk_status rows_parallel(Stack* s, const RowBufs& b, int n, hipStream_t st, PendingAdd* pend, Mix mix) {
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    const auto& c = s->cfg;
    *pend = PendingAdd{};
    for (int l = 0; l < s->n_runs(); ++l) {
        const auto& L = s->at(l);
        const Stack::Packed P = s->packed.empty() ? Stack::Packed{} : s->packed[s->runs[l].layer];
        mark(KC_NORM_QKV);
        if (s->runs[l].pass >= 0) {
            RowsNormArgs a = add_args(s, b, n, *pend, nullptr, b.cat);
            a.embed = s->embed; a.tok = b.tok; a.store_h = 0;      // (`base` takes the stream's place)
            if (pgk_status r = rows_norm(a, n, DT, st)) return r;
            *pend = PendingAdd{};
            pend->y = true;
            pend->base = c.loop_step + (size_t)s->runs[l].pass * s->Wp;
            if (DT == PGK_F32) { if (pgk_status r = pgk_gemm_nt(b.cat, c.loop_in, nullptr, b.y, n, s->Wp, 2 * s->Wp, PGK_F32, st)) return r; }
            else {
                pend->slabs = plan_f32(n, s->Wp, 2 * s->Wp);
                if (pgk_status r = gemm_f32(b.cat, c.loop_in, b.slabs, pend->slabs, n, s->Wp, 2 * s->Wp, st)) return r;
            }
        }
        if (pgk_status r = rows_norm(add_args(s, b, n, *pend, L.norm1, b.x), n, DT, st)) return r;
        *pend = PendingAdd{};
        if (pgk_status r = rows_in_proj<T>(s, L, P.in, b, n, st)) return r;
        mark(recurrent(L) ? KC_RECUR : KC_ATTN);
        if (pgk_status r = mix(l)) return r;
        mark(KC_OPROJ);
        if (pgk_status r = rows_out_proj<T>(s, b, b.a, L.w_o, P.o, n, L.n_att, &pend->slabs, st)) return r;
        pend->y = true;
        if (!L.ff_pad) continue;
        mark(KC_GATEUP);
        MoeArgs m{b.x, n, s->Wp, L.ff_pad, router_of(L), (const T*)L.w_in + (size_t)L.n_in * s->Wp, L.w_gate_up, L.w_down, b.e, b.moe};
        if (pgk_status r = moe_rows(m, DT, st)) return r;
        pend->top = L.top;
    }
    return PGK_OK;
}

// Hyper-connected layers: the sublayer output that is still to go into the streams (its numbers `upd`; null: none)
struct PendingHyper { const float *upd = nullptr, *bias = nullptr; int slabs = 0, top = 0; bool y = true, gated = false, spread = false; };

static HyperArgs hyper_args(const Stack* s, const RowBufs& b, int n, const PendingHyper& p, const float* in, const float* gamma, void* out) {
    HyperArgs a{};
    const int ld = s->Wp;
    a.S = s->cfg.streams; a.W = s->cfg.width; a.ld = ld; a.groups = s->cfg.norm_groups; a.eps = s->cfg.norm_eps;
    a.src = p.spread ? b.xs : b.h; a.src_row = p.spread ? (long long)a.S * ld : ld; a.src_stream = p.spread ? ld : 0;
    a.in = in; a.gamma = gamma; a.out = out;
    if (!p.upd) return a;
    a.dst = b.xs; a.upd = p.upd; a.y = !p.y ? nullptr : p.slabs ? (const void*)b.slabs : b.y; a.ldy = ld; a.nslabs = p.slabs; a.slab_stride = (long long)n * ld;
    a.y_bias = p.bias; a.y_gate = p.gated ? b.ygate : nullptr; a.e = p.top ? b.e : nullptr; a.e_top = p.top;
    return a;
}

template <class T, class Mix>
static pgk_status rows_hyper(Stack* s, const RowBufs& b, int n, hipStream_t st, PendingHyper* pend, Mix mix) {
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    *pend = PendingHyper{};
    auto settle = [&]() {
        const bool spread = pend->spread || pend->upd;
        *pend = PendingHyper{};
        pend->spread = spread;
    };
    for (int l = 0; l < s->cfg.num_layers; ++l) {
        const auto& L = s->layers[l];
        const Stack::Packed P = s->packed.empty() ? Stack::Packed{} : s->packed[l];
        mark(KC_NORM_QKV);
        if (pgk_status r = hyper_rows(hyper_args(s, b, n, *pend, L.hyper1, L.norm1, b.x), n, DT, st)) return r;
        settle();
        if (pgk_status r = rows_in_proj<T>(s, L, P.in, b, n, st)) return r;
        mark(KC_ATTN);
        if (pgk_status r = mix(l)) return r;
        mark(KC_OPROJ);
        if (pgk_status r = rows_out_proj<T>(s, b, b.a, L.w_o, P.o, n, L.n_att, &pend->slabs, st)) return r;
        pend->upd = L.hyper1; pend->bias = L.b_o;
        if (!L.ff_pad) continue;
        mark(KC_GATEUP);
        HyperArgs h = hyper_args(s, b, n, *pend, L.hyper2, L.norm2, b.x);
        const bool shared = L.ff == PGK_FF_TABLE && L.shared_pad;
        if (shared) { h.gate_w = L.w_shared_gate; h.gate_out = b.ygate; }
        if (pgk_status r = hyper_rows(h, n, DT, st)) return r;
        settle();
        if (L.ff == PGK_FF_TABLE) {
            MoeArgs m{b.x, n, s->Wp, L.ff_pad, router_of(L), nullptr, L.w_gate_up, L.w_down, b.e, b.moe, true, b.tok};
            if (pgk_status r = moe_rows(m, DT, st)) return r;
            pend->top = L.top;
            if (shared) { if (pgk_status r = rows_gate_up<T>(s, L, P.gate_up, b, n, st)) return r; }
        } else {
            if (pgk_status r = rows_proj<T>(s, b, L.w_gate_up, P.gate_up, b.gu, n, L.ff_pad, st)) return r;
            if (pgk_status r = poly_rows(b.gu, b.act, n, L.ff_dim, L.ff_pad, L.act, s->cfg.norm_eps, DT, st)) return r;
        }
        mark(KC_DOWN);
        if (dense_ff(L)) { if (pgk_status r = rows_out_proj<T>(s, b, b.act, dense_down(L), P.down, n, dense_ff(L), &pend->slabs, st)) return r; }
        pend->upd = L.hyper2; pend->gated = shared; pend->y = dense_ff(L) > 0;
    }
    return PGK_OK;
}

// The launch that completes the stream and leaves normed rows
struct LastRows { bool hyper = false; RowsNormArgs norm; HyperArgs streams; };
// ... for n rows (`rows`: which, null: the first n) into `out`; the stream itself stays as it is
static pgk_status last_rows(const LastRows& l, void* out, const int32_t* rows, int n, pgk_dtype dt, hipStream_t st) {
    if (l.hyper) {
        HyperArgs a = l.streams;
        a.out = out; a.rows = rows; a.dst = nullptr;
        return hyper_rows(a, n, dt, st);
    }
    RowsNormArgs a = l.norm;
    a.out = out; a.rows = rows; a.store_h = 0;
    return rows_norm(a, n, dt, st);
}

// All layers on n rows of b.h (embedded tokens)
template <class T, class Mix>
static pgk_status rows_model(Stack* s, const RowBufs& b, int n, hipStream_t st, Mix mix, LastRows* last) {
    if (s->cfg.block == PGK_BLOCK_HYPER) {
        PendingHyper p;
        if (pgk_status r = rows_hyper<T>(s, b, n, st, &p, mix)) return r;
        last->hyper = true;
        last->streams = hyper_args(s, b, n, p, nullptr, s->final_norm, b.x);
        return PGK_OK;
    }
    if (s->cfg.block == PGK_BLOCK_PARALLEL) {
        PendingAdd p;
        if (pgk_status r = rows_parallel<T>(s, b, n, st, &p, mix)) return r;
        last->norm = add_args(s, b, n, p, s->final_norm, b.x);
        return PGK_OK;
    }
    Pending p;
    if (pgk_status r = rows_layers<T>(s, b, n, st, &p, mix)) return r;
    last->norm = norm_args(s, b, n, p, s->final_norm, b.x);
    return PGK_OK;
}

constexpr int ROWS_ARGMAX_BLOCKS = 64;

template <class T>
static pgk_status step_rows(Engine* e, int B, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    const auto& c = s->cfg;
    const RowBufs b{e->h, s->x16, s->in16, s->a16, s->y16, s->gu16, s->act16, s->slabs16, nullptr, s->cat16, s->e16, s->moe16, e->tokens, s->xrows, s->ygate};
    LastRows last;
    if (pgk_status r = rows_model<T>(s, b, B, st, [&](int l) { return mix_decode<T, T>(e, l, B, b.in, b.a, st, launches); }, &last)) return r;
    mark(KC_LMHEAD);
    if (pgk_status r = last_rows(last, b.x, nullptr, B, DT, st)) return r;
    if (pgk_status r = logit_rows<T>(s, (const T*)b.x, e->logits, B, st)) return r;
    PGK_CHECK_HIP(launch_k(rows_argmax_kernel, dim3(ROWS_ARGMAX_BLOCKS, B), dim3(256), 0, st, e->logits, c.vocab_size, c.logit_cap, e->amax_val, e->amax_idx));
    *launches += 3;
    for (const auto& r : s->runs) {                    // (one more where a projection's slabs or SwiGLU take a launch of their own)
        const auto& L = s->layers[r.layer];
        *launches += 3 + (!L.ff_pad ? 0 : L.ff == PGK_FF_MOE ? 5 : L.ff == PGK_FF_TABLE ? (L.shared_pad ? 7 : 5) : L.ff == PGK_FF_POLY ? 4 : 3) + (r.pass >= 0 ? 2 : 0);
    }
    return PGK_OK;
}

template <class T>
static pgk_status stack_step(Engine* e, int batch, hipStream_t st, int* launches) {
    Stack* s = stack_of(e);
    int nblk = ROWS_ARGMAX_BLOCKS;
    if (batch == 1) {
        nblk = e->lm_blocks;
        if (pgk_status r = s->cfg.block == PGK_BLOCK_HYPER ? step_hyper<T>(e, st, launches) : s->cfg.block == PGK_BLOCK_PARALLEL ? step_parallel<T>(e, st, launches) : step_one<T>(e, st, launches)) return r;
    } else if (pgk_status r = step_rows<T>(e, batch, st, launches)) return r;
    mark(KC_ARGMAX);
    const int32_t* sampled = nullptr;
    if (e->sample_temperature > 0.f) {
        if (pgk_status r = engine_sample(e, 0, batch, st)) return r;
        sampled = e->sampled;
        *launches += 1;
    }
    PGK_CHECK_HIP(launch_k(&finalize_kernel<T>, dim3(batch), dim3(256), 0, st, e->amax_val, e->amax_idx, nblk, e->tokens, e->positions, e->token_log,
                           e->step_counter, e->cfg.max_batch, e->log_cap, (const T*)s->embed, e->h, s->cfg.width, 1, e->clk_log, (const float*)nullptr,
                           (const float*)nullptr, (float*)nullptr, (float*)nullptr, 0, e->cfg.max_seq_len, batch, sampled, (const T*)s->pos, s->Wp));
    *launches += 1;
    return PGK_OK;
}

static pgk_status stack_decode_step(Engine* e, int batch, hipStream_t st, int* launches, bool) {
    return stack_of(e)->cfg.dtype == PGK_F32 ? stack_step<float>(e, batch, st, launches) : stack_step<bf16>(e, batch, st, launches);
}

static pgk_status stack_embed_state(Engine* e, int batch, hipStream_t st) {
    Stack* s = stack_of(e);
    const auto& c = s->cfg;
    if (c.dtype == PGK_F32) stack_embed_kernel<float><<<batch, 256, 0, st>>>((const float*)s->embed, (const float*)s->pos, e->tokens, e->positions, e->h, c.width, s->Wp, c.max_positions);
    else stack_embed_kernel<bf16><<<batch, 256, 0, st>>>((const bf16*)s->embed, (const bf16*)s->pos, e->tokens, e->positions, e->h, c.width, s->Wp, c.max_positions);
    PGK_LAUNCH_CHECK();
    return PGK_OK;
}

// May slot `slot` go on at `pos`?  Position 0 starts a new sequence; otherwise the rows its windows and taps reach must still be in the
// rings (a ring row is overwritten by the position `R` later), and a recurrent state only goes on where it stands.
static pgk_status check_position(const Engine* e, int slot, int pos) {
    const Stack* s = stack_of(e);
    const int len = s->len[slot];
    PGK_REQUIRE(pos <= len, "engine: slot %d holds %d positions, cannot go on at position %d", slot, len, pos);
    if (pos == 0 || pos == len) return PGK_OK;
    for (int l = 0; l < s->n_runs(); ++l) {
        const auto& L = s->at(l);
        PGK_REQUIRE(!recurrent(L), "engine: slot %d has moved on to position %d; its recurrent state cannot go back to position %d", slot, len, pos);
        auto kept = [&](int back, int R) { return (pos - back > 0 ? pos - back : 0) + R >= len; };
        PGK_REQUIRE(kept(span_keys(pos, L.window, L.chunked) - 1, s->ring[kv_source(L, l)]) && (L.mixer != PGK_MIX_ATTENTION || !L.conv || kept(L.taps - 1, L.taps)),
                    "engine: slot %d has moved on to position %d; the window of position %d is no longer in its ring", slot, len, pos);
    }
    return PGK_OK;
}

static pgk_status stack_check_state(Engine* e, const int32_t* h_positions, int batch) {
    for (int b = 0; b < batch; ++b)
        if (pgk_status r = check_position(e, b, h_positions[b])) return r;
    for (int b = 0; b < batch; ++b) stack_of(e)->len[b] = h_positions[b];      // the step that follows writes position h_positions[b]
    return PGK_OK;
}

static void stack_advance(Engine* e, int batch, int steps) {
    for (int b = 0; b < batch; ++b) stack_of(e)->len[b] += steps;
}

template <class T>
static pgk_status stack_prefill_t(Engine* e, int n_seqs, const int32_t* slots, const int32_t* lens, const int32_t* starts, const int32_t* tokens, int n_want,
                                  const int32_t* want, float* h_logits, hipStream_t st) {
    Stack* s = stack_of(e);
    constexpr pgk_dtype DT = std::is_same<T, float>::value ? PGK_F32 : PGK_BF16;
    const auto& c = s->cfg;
    for (int i = 0; i < n_seqs; ++i)
        if (pgk_status r = check_position(e, slots[i], starts[i])) return r;
    int n = 0;
    for (int i = 0; i < n_seqs; ++i) n += lens[i];
    // per layer with a ring: which cached rows a sequence's queries reach (its own and those before them in a window or chunk)
    struct LayerRows { size_t past0 = 0; int n_past = 0, n_kv = 0; };
    const int n_runs = s->n_runs();
    std::vector<LayerRows> lr(n_runs);
    std::vector<RowPlace> place;                        // per layer: n_past gathered rows, then n new rows (equal layers share them)
    std::vector<int> share(n_runs, -1);
    int max_kv = 0;
    auto past_of = [&](int l, int i) { return s->past(l, starts[i]); };
    for (int l = 0; l < n_runs; ++l) {
        if (!s->reach[l]) continue;
        for (int k = 0; k < l && share[l] < 0; ++k)
            if (share[k] < 0 && s->ring[k] == s->ring[l] && s->readers[k] == s->readers[l]) share[l] = k;
        if (share[l] >= 0) { lr[l] = lr[share[l]]; continue; }
        lr[l].past0 = place.size();
        int kv = 0;
        std::vector<RowPlace> fresh;
        for (int i = 0; i < n_seqs; ++i) {
            const int past = past_of(l, i), end = starts[i] + lens[i];
            for (int p = starts[i] - past; p < starts[i]; ++p) place.push_back(RowPlace{p, slots[i], kv++, 0});
            for (int p = starts[i]; p < end; ++p) fresh.push_back(RowPlace{p, slots[i], kv++, p >= end - s->ring[l] ? 1 : 0});
            lr[l].n_past += past;
        }
        lr[l].n_kv = kv;
        if (kv > max_kv) max_kv = kv;
        place.insert(place.end(), fresh.begin(), fresh.end());
    }
    // K/V scratch: one region that the layers use in turn, and one of its own for every layer whose keys others take
    size_t kv_elems = 0, c_elems = 0, own_elems = 0;
    std::vector<size_t> own(n_runs, 0);           // 1 + offset
    for (int l = 0; l < n_runs; ++l)
        if (s->at(l).kv_from >= 0) own[s->at(l).kv_from] = 1;
    for (int l = 0; l < n_runs; ++l) {
        const auto& L = s->at(l);
        if (!s->reach[l]) continue;
        const size_t ke = (size_t)lr[l].n_kv * 2 * L.kv_heads * L.head_pad, ce = (size_t)lr[l].n_kv * L.rank_pad;
        if (own[l]) { own[l] = 1 + own_elems; own_elems += (ke + 127) & ~(size_t)127; }
        else if (ke > kv_elems) kv_elems = ke;
        if (ce > c_elems) c_elems = ce;
    }
    // chunk tables of the recurrent layers, one per chunk length
    int longest = 0;
    for (int i = 0; i < n_seqs; ++i) longest = lens[i] > longest ? lens[i] : longest;
    struct Chunks { int rows = 0; std::vector<RecurChunk> list; std::vector<int32_t> of_seq; size_t o_list = 0, o_seq = 0; };
    std::vector<Chunks> chunkings;
    std::vector<int> chunking(n_runs, -1);
    size_t chunk_ws = 0, chunk_tab = 0;
    for (int l = 0; l < n_runs; ++l) {
        const auto& L = s->at(l);
        const int C = !recurrent(L) || longest < RECUR_CHUNKED_FROM ? 0 : L.mixer != PGK_MIX_DELTA ? recur_chunk_rows(L.head_pad, L.vhead_pad) : delta_chunk_ok(L.head_pad, L.vhead_pad) ? DELTA_CHUNK : 0;
        if (!C) continue;
        for (size_t k = 0; k < chunkings.size(); ++k) if (chunkings[k].rows == C) chunking[l] = (int)k;
        if (chunking[l] < 0) {
            Chunks t;
            t.rows = C;
            for (int i = 0, row = 0; i < n_seqs; row += lens[i++]) {
                t.of_seq.push_back((int32_t)t.list.size());
                for (int r = 0; r < lens[i]; r += C) t.list.push_back(RecurChunk{row + r, lens[i] - r < C ? lens[i] - r : C});
            }
            t.of_seq.push_back((int32_t)t.list.size());
            chunking[l] = (int)chunkings.size();
            chunkings.push_back(t);
        }
        const int n_chunks = (int)chunkings[chunking[l]].list.size();
        const size_t need = L.mixer == PGK_MIX_DELTA ? delta_chunk_bytes(delta_args(s, l, nullptr, nullptr, nullptr, nullptr, n), n_chunks) : recur_chunk_bytes(recur_args(s, l, nullptr, nullptr, n), n_chunks);
        if (need > chunk_ws) chunk_ws = need;
    }
    const int wrows = n_want < 128 ? n_want : 128;
    auto up = [](size_t v) { return (v + 255) & ~(size_t)255; };
    const size_t E = sizeof(T);
    const size_t sizes[] = {(size_t)n * s->Wp * 4, (size_t)n * s->Wp * E, (size_t)n * s->max_in * E, (size_t)n * s->max_att * E, (size_t)n * s->Wp * E,
                            (size_t)n * 2 * s->max_ff * E, (size_t)n * s->max_ff * E, c_elems * E, kv_elems * E, (size_t)wrows * s->Wp * E, (size_t)wrows * c.vocab_size * 4,
                            s->slab_elems(n, DT == PGK_F32) * 4, (size_t)n * s->max_q * E, own_elems * E, chunk_ws, (size_t)n * s->max_conv * E, (size_t)n * s->max_z * 4,
                            (size_t)n * s->max_gate * E, (size_t)n * s->max_low * E, c.loop_times ? (size_t)n * 2 * s->Wp * E : 0, (size_t)n * s->max_top * s->Wp * E, s->moe_ws(n),
                            c.block == PGK_BLOCK_HYPER ? (size_t)n * c.streams * s->Wp * 4 : 0, c.block == PGK_BLOCK_HYPER ? (size_t)n * 4 : 0};
    for (auto& t : chunkings) {
        t.o_list = chunk_tab;
        t.o_seq = t.o_list + up(t.list.size() * sizeof(RecurChunk));
        chunk_tab = t.o_seq + up(t.of_seq.size() * 4);
    }
    size_t need = 0;
    for (size_t z : sizes) need += up(z);
    const size_t tab_need = up((size_t)n * 4) * 2 + up(place.size() * sizeof(RowPlace)) + up((size_t)n_want * 4) + up((size_t)n * sizeof(RowSrc)) + up(n_seqs * sizeof(SeqSpan)) + chunk_tab;
    auto grow = [&](void** p, size_t* have, size_t want_bytes) -> pgk_status {
        if (want_bytes <= *have) return PGK_OK;
        if (*p) { PGK_CHECK_HIP(hipStreamSynchronize(st)); pgk_free(*p); }
        *p = nullptr; *have = 0;
        if (pgk_status r = pgk_malloc(p, want_bytes)) return r;
        *have = want_bytes;
        return PGK_OK;
    };
    const size_t before = s->pf_bytes + s->tab_bytes;
    if (pgk_status r = grow(&s->pf, &s->pf_bytes, need)) return r;
    if (pgk_status r = grow(&s->tab, &s->tab_bytes, tab_need)) return r;
    e->ws_bytes += s->pf_bytes + s->tab_bytes - before;
    char* p = (char*)s->pf;
    auto take = [&](size_t bytes) { char* q = p; p += up(bytes); return (void*)q; };
    RowBufs b;
    b.h = (float*)take(sizes[0]); b.x = take(sizes[1]); b.in = take(sizes[2]); b.a = take(sizes[3]); b.y = take(sizes[4]); b.gu = take(sizes[5]); b.act = take(sizes[6]);
    T* c_all = (T*)take(sizes[7]);
    T* kv = (T*)take(sizes[8]);
    void* xw = take(sizes[9]);
    float* lg = (float*)take(sizes[10]);
    b.slabs = (float*)take(sizes[11]);
    b.q = take(sizes[12]);
    T* kv_own = (T*)take(sizes[13]);
    void* ws_chunk = take(sizes[14]);
    void* conv_rows_buf = take(sizes[15]);
    float* z_rows = (float*)take(sizes[16]);
    void *gate_rows = take(sizes[17]), *low_rows = take(sizes[18]);
    b.cat = take(sizes[19]); b.e = take(sizes[20]); b.moe = take(sizes[21]); b.xs = (float*)take(sizes[22]); b.ygate = (float*)take(sizes[23]);
    // one host image of the index tables, one copy
    std::vector<char> img(tab_need, 0);
    const size_t o_pos = up((size_t)n * 4), o_place = 2 * o_pos, o_want = o_place + up(place.size() * sizeof(RowPlace)),
                 o_rows = o_want + up((size_t)n_want * 4), o_seqs = o_rows + up((size_t)n * sizeof(RowSrc)), o_chunk = o_seqs + up(n_seqs * sizeof(SeqSpan));
    memcpy(img.data(), tokens, (size_t)n * 4);
    for (int i = 0, row = 0; i < n_seqs; ++i) {
        ((SeqSpan*)(img.data() + o_seqs))[i] = SeqSpan{row, lens[i], starts[i], slots[i]};
        for (int j = 0, first = row; j < lens[i]; ++j, ++row) {
            ((int32_t*)(img.data() + o_pos))[row] = starts[i] + j;
            ((RowSrc*)(img.data() + o_rows))[row] = RowSrc{starts[i] + j, slots[i], first};
        }
    }
    if (!place.empty()) memcpy(img.data() + o_place, place.data(), place.size() * sizeof(RowPlace));
    if (n_want) memcpy(img.data() + o_want, want, (size_t)n_want * 4);
    for (const auto& t : chunkings) {
        memcpy(img.data() + o_chunk + t.o_list, t.list.data(), t.list.size() * sizeof(RecurChunk));
        memcpy(img.data() + o_chunk + t.o_seq, t.of_seq.data(), t.of_seq.size() * 4);
    }
    PGK_CHECK_HIP(hipMemcpyAsync(s->tab, img.data(), tab_need, hipMemcpyHostToDevice, st));
    PGK_CHECK_HIP(hipStreamSynchronize(st));      // the image is pageable host memory
    const int32_t* d_tok = (const int32_t*)s->tab;
    b.tok = d_tok;
    const int32_t* d_pos = (const int32_t*)((char*)s->tab + o_pos);
    const RowPlace* d_place = (const RowPlace*)((char*)s->tab + o_place);
    const int32_t* d_want = (const int32_t*)((char*)s->tab + o_want);
    const RowSrc* d_rows = (const RowSrc*)((char*)s->tab + o_rows);
    const SeqSpan* d_seqs = (const SeqSpan*)((char*)s->tab + o_seqs);
    stack_embed_kernel<T><<<n, 256, 0, st>>>((const T*)s->embed, (const T*)s->pos, d_tok, d_pos, b.h, c.width, s->Wp, c.max_positions);
    PGK_LAUNCH_CHECK();
    auto latent = [&](int l) -> pgk_status {
        const auto& L = s->at(l);
        const LayerRows& w = lr[l];
        const int HD = L.heads * L.head_pad, R = s->ring[l];
        if (w.n_past) {
            latent_gather_kernel<T><<<w.n_past, 64, 0, st>>>(d_place + w.past0, (const T*)s->cache[l], c_all, R, L.rank_pad);
            PGK_LAUNCH_CHECK();
        }
        latent_rows_kernel<T><<<ceil_div(n, 4), 256, 0, st>>>(d_place + w.past0 + w.n_past, (T*)b.in, L.n_in, HD, L.c_norm, (T*)s->cache[l], c_all, n, R,
                                                              L.rank_pad, L.rank, c.norm_eps, L.heads, L.head_pad, L.dim, L.rot, L.rot_freq);
        PGK_LAUNCH_CHECK();
        if (pgk_status r = pgk_gemm_nt(c_all, L.w_ukv, nullptr, kv, w.n_kv, 2 * HD, L.rank_pad, DT, st)) return r;
        int row = 0, kv0 = 0;
        const WindowStrides sd{L.head_pad, L.n_in, L.head_pad, 2 * HD, L.head_pad, 2 * HD, L.head_pad, HD};
        for (int i = 0; i < n_seqs; ++i) {
            const int klen = past_of(l, i) + lens[i];
            const T* q = (const T*)b.in + (size_t)row * L.n_in;
            const T* k = kv + (size_t)kv0 * 2 * HD;
            if (pgk_status r = window_attention(q, k, k + HD, (T*)b.a + (size_t)row * HD, L.heads, L.heads, lens[i], klen, L.head_pad, L.head_pad, L.scale, L.window, sd,
                                                OutGate{L.gated ? q + HD + L.rank_pad : nullptr, L.n_in, 1, 0}, nullptr, DT, st))
                return r;
            row += lens[i];
            kv0 += klen;
        }
        return PGK_OK;
    };
    auto attention = [&](int l) -> pgk_status {
        const auto& L = s->at(l);
        const int src = kv_source(L, l), HD = L.heads * L.head_pad, GD = L.kv_heads * L.head_pad, R = s->ring[src];
        const bool mine = src == l;
        const LayerRows& w = lr[src];
        T* rows = own[src] ? kv_own + (own[src] - 1) : kv;
        if (mine)
            if (pgk_status r = kv_gather(d_place + w.past0, w.n_past, s->cache[l], rows, 2 * GD, GD, L.head_pad, R, DT, st)) return r;
        ConvArgs a{};
        a.in = b.in; a.ld_in = L.n_in; a.bias = L.b_in; a.conv = L.conv; a.taps = L.taps; a.n_q = HD; a.n_kv = mine ? GD : 0; a.D = L.head_pad; a.n = n; a.R = R;
        a.q_norm = L.q_norm; a.k_norm = L.k_norm; a.q_true = L.heads * L.dim; a.k_true = L.kv_heads * L.dim; a.eps = c.norm_eps; a.q_mult = 1.f;
        a.tap_ring = s->taps[l]; a.rows = d_rows; a.place = d_place + w.past0 + w.n_past; a.q_out = b.q; a.ld_q = HD; a.kv_rows = rows; a.ld_kv = 2 * GD; a.cache = s->cache[src];
        if (pgk_status r = conv_rows(a, DT, DT == PGK_F32, DT == PGK_F32, st)) return r;
        const int channels = HD + 2 * a.n_kv;
        if (L.conv)
            if (pgk_status r = conv_save(b.in, L.n_in, d_seqs, n_seqs, s->taps[l], L.taps, channels, DT, st)) return r;
        int row = 0, kv0 = 0;
        const WindowStrides sd{L.head_pad, HD, L.head_pad, 2 * GD, L.head_pad, 2 * GD, L.head_pad, HD};
        for (int i = 0; i < n_seqs; ++i) {
            const int klen = past_of(src, i) + lens[i];
            const T* k = rows + (size_t)kv0 * 2 * GD;
            const OutGate gate{(const T*)b.in + (size_t)row * L.n_in + channels, L.n_in, L.head_pad, 1};
            if (pgk_status r = window_attention((const T*)b.q + (size_t)row * HD, k, k + GD, (T*)b.a + (size_t)row * HD, L.heads, L.kv_heads, lens[i], klen, L.head_pad, L.head_pad,
                                                L.scale, L.window, sd, gate, L.slopes, DT, st))
                return r;
            row += lens[i];
            kv0 += klen;
        }
        return PGK_OK;
    };
    auto talk = [&](int l) -> pgk_status {
        const auto& L = s->at(l);
        const int src = kv_source(L, l), HD = L.heads * L.head_pad, GD = L.kv_heads * L.head_pad;
        const LayerRows& w = lr[src];
        T* rows = own[src] ? kv_own + (own[src] - 1) : kv;
        if (src == l)
            if (pgk_status r = kv_gather(d_place + w.past0, w.n_past, s->cache[l], rows, 2 * GD, GD, L.head_pad, s->ring[l], DT, st)) return r;
        HeadRowsArgs h = head_args(s, l, b.in, n);
        h.rows = d_rows; h.place = d_place + w.past0 + w.n_past; h.q_out = b.q; h.kv_rows = rows; h.ld_kv = 2 * GD;
        if (pgk_status r = head_rows(h, DT, DT == PGK_F32, st)) return r;
        int none = 0;
        for (int i = 0, row = 0, kv0 = 0; i < n_seqs; ++i) {
            const int past = past_of(src, i);
            TalkArgs a = talk_args(s, l, lens[i], (T*)b.a + (size_t)row * HD);
            a.q = (const T*)b.q + (size_t)row * HD; a.k = rows + (size_t)kv0 * 2 * GD; a.v = (const T*)a.k + GD; a.ld_kv = 2 * GD;
            a.kv_len = past + lens[i]; a.pos0 = starts[i] - past;
            if (pgk_status r = talk_attention(a, DT, DT == PGK_F32, st, &none)) return r;
            row += lens[i];
            kv0 += past + lens[i];
        }
        return PGK_OK;
    };
    // taps over time and SiLU on the projected channels; then the rings take the last rows
    auto convolve = [&](int l) -> pgk_status {
        const auto& L = s->at(l);
        const int ch = conv_channels(L);
        if (pgk_status r = conv_silu_rows(ConvSiluArgs{b.in, L.n_in, L.conv, L.conv_bias, L.taps, ch, n, s->taps[l], d_rows, conv_rows_buf, ch}, DT, st)) return r;
        return conv_save(b.in, L.n_in, d_seqs, n_seqs, s->taps[l], L.taps, ch, DT, st);
    };
    auto in_chunks = [&](int l, auto go) -> pgk_status {           // go(chunk list, its length, first chunk of every sequence)
        const Chunks& t = chunkings[chunking[l]];
        const char* tab = (const char*)s->tab + o_chunk;
        return go((const RecurChunk*)(tab + t.o_list), (int)t.list.size(), (const int32_t*)(tab + t.o_seq));
    };
    auto recurrence = [&](int l) -> pgk_status {
        RecurArgs a = recur_args(s, l, b.in, b.a, n);
        a.seqs = d_seqs; a.n_seqs = n_seqs;
        if (a.kind == RECUR_SSD) {
            if (pgk_status r = convolve(l)) return r;
            a.rows = conv_rows_buf; a.ld_rows = conv_channels(s->at(l));
        }
        if (pgk_status r = chunking[l] < 0 ? recur_rows(a, DT, DT == PGK_F32, st)
                                           : in_chunks(l, [&](const RecurChunk* ch, int nc, const int32_t* of) { return recur_chunked(a, ch, nc, of, ws_chunk, DT, st); }))
            return r;
        return a.kind == RECUR_SSD ? ssd_norm(s, l, b.a, n, DT, st) : PGK_OK;
    };
    auto delta = [&](int l) -> pgk_status {
        const auto& L = s->at(l);
        const int a_off = delta_a_off(L), g_off = a_off + L.rank_a, NZ = L.heads * L.head_pad, NG = L.heads * L.vhead_pad;
        if (pgk_status r = convolve(l)) return r;
        if (n <= 16) {
            if (pgk_status r = lowrank_rows(b.in, L.n_in, n, a_off, L.rank_a, L.w_a2, z_rows, NZ, g_off, L.rank_g, L.w_g2, gate_rows, NG, DT, DT == PGK_F32, st)) return r;
        } else {
            if (pgk_status r = rows_slice(b.in, L.n_in, a_off, L.rank_a, low_rows, n, DT, st)) return r;
            if (pgk_status r = DT == PGK_F32 ? pgk_gemm_nt(low_rows, L.w_a2, nullptr, z_rows, n, NZ, L.rank_a, PGK_F32, st) : gemm_f32(low_rows, L.w_a2, z_rows, 1, n, NZ, L.rank_a, st)) return r;
            if (pgk_status r = rows_slice(b.in, L.n_in, g_off, L.rank_g, low_rows, n, DT, st)) return r;
            if (pgk_status r = pgk_gemm_nt(low_rows, L.w_g2, nullptr, gate_rows, n, NG, L.rank_g, DT, st)) return r;
        }
        DeltaArgs a = delta_args(s, l, b.in, z_rows, gate_rows, b.a, n);
        a.rows = conv_rows_buf; a.ld_rows = conv_channels(L); a.seqs = d_seqs; a.n_seqs = n_seqs;
        if (chunking[l] < 0) return delta_rows(a, DT, DT == PGK_F32, st);
        return in_chunks(l, [&](const RecurChunk* ch, int nc, const int32_t* of) { return delta_chunked(a, ch, nc, of, ws_chunk, DT, st); });
    };
    auto mix = [&](int l) -> pgk_status {
        switch (s->at(l).mixer) {
            case PGK_MIX_LATENT: return latent(l);
            case PGK_MIX_ATTENTION: return attention(l);
            case PGK_MIX_TALK: return talk(l);
            case PGK_MIX_DELTA: return delta(l);
            default: return recurrence(l);
        }
    };
    LastRows last;
    if (pgk_status r = rows_model<T>(s, b, n, st, mix, &last)) return r;
    for (int i = 0; i < n_seqs; ++i) s->len[slots[i]] = starts[i] + lens[i];
    for (int w0 = 0; w0 < n_want; w0 += 128) {
        const int m = n_want - w0 < 128 ? n_want - w0 : 128;
        if (pgk_status r = last_rows(last, xw, d_want + w0, m, DT, st)) return r;      // (a wanted row may be asked for twice)
        if (pgk_status r = logit_rows<T>(s, (const T*)xw, lg, m, st)) return r;
        if (c.logit_cap > 0.f) { if (pgk_status r = soft_cap_rows(lg, (size_t)m * c.vocab_size, c.logit_cap, st)) return r; }
        PGK_CHECK_HIP(hipMemcpyAsync(h_logits + (size_t)w0 * c.vocab_size, lg, (size_t)m * c.vocab_size * 4, hipMemcpyDeviceToHost, st));
        PGK_CHECK_HIP(hipStreamSynchronize(st));
    }
    return PGK_OK;
}

static pgk_status stack_prefill(Engine* e, int n_seqs, const int32_t* slots, const int32_t* lens, const int32_t* starts, const int32_t* tokens, int n_want,
                                const int32_t* want, float* h_logits, hipStream_t st) {
    if (stack_of(e)->cfg.dtype == PGK_F32) return stack_prefill_t<float>(e, n_seqs, slots, lens, starts, tokens, n_want, want, h_logits, st);
    return stack_prefill_t<bf16>(e, n_seqs, slots, lens, starts, tokens, n_want, want, h_logits, st);
}

// layer l's latent ring, K/V ring (values after the keys of a slot: v points at the first slot's) or recurrent states
static pgk_status stack_kv_ptr(Engine* e, int layer, void** k, void** v) {
    const Stack* s = stack_of(e);
    const auto& L = s->at(layer);
    *k = s->cache[layer];
    *v = L.mixer == PGK_MIX_ATTENTION || L.mixer == PGK_MIX_TALK ? (char*)s->cache[layer] + (size_t)L.kv_heads * s->ring[kv_source(L, layer)] * L.head_pad * s->esize() : nullptr;
    return PGK_OK;
}

static void stack_destroy(Engine* e) {
    Stack* s = stack_of(e);
    if (s->pf) (void)pgk_free(s->pf);
    if (s->tab) (void)pgk_free(s->tab);
    delete s;
    e->kind_state = nullptr;
}

static const EngineKind STACK_KIND = {stack_decode_step, stack_prefill, nullptr, stack_embed_state, stack_check_state, stack_advance, stack_kv_ptr, stack_destroy};

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_engine_create_stack(const pgk_stack_config_t* cfg, const void* embed, const void* pos_embed, const void* head, const float* final_norm,
                                   const pgk_stack_layer_t* layers, pgk_engine* out) {
    PGK_REQUIRE(cfg && embed && head && final_norm && layers && out, "pgk_engine_create_stack: null argument");
    const auto& c = *cfg;
    PGK_REQUIRE(c.dtype == PGK_BF16 || c.dtype == PGK_F32, "pgk_engine_create_stack: dtype %d (bf16 or f32)", (int)c.dtype);
    PGK_REQUIRE(c.vocab_size >= 1 && c.width >= 1 && c.num_layers >= 1 && c.max_batch >= 1 && c.max_seq_len >= 1, "pgk_engine_create_stack: bad sizes");
    PGK_REQUIRE(!pos_embed || c.max_seq_len <= c.max_positions, "pgk_engine_create_stack: %d positions of cache but %d learned positions", c.max_seq_len, c.max_positions);
    const int Wp = ceil_div(c.width, 64) * 64;
    for (int l = 0; l < c.num_layers; ++l) {
        const auto& L = layers[l];
        PGK_REQUIRE(L.mixer >= PGK_MIX_LATENT && L.mixer <= PGK_MIX_TALK && L.ff >= PGK_FF_SWIGLU && L.ff <= PGK_FF_TABLE, "pgk_engine_create_stack: layer %d: mixer %d, feed-forward %d", l, L.mixer, L.ff);
        PGK_REQUIRE(L.heads >= 1 && L.dim >= 1 && L.vdim >= 1, "pgk_engine_create_stack: layer %d: bad mixer sizes", l);
        PGK_REQUIRE(L.ff_pad % 64 == 0 && L.ff_pad >= 0, "pgk_engine_create_stack: layer %d: feed-forward pad %d", l, L.ff_pad);
        PGK_REQUIRE(L.n_in % 64 == 0 && L.n_att % 64 == 0, "pgk_engine_create_stack: layer %d: %d in-projection rows, %d out-projection columns", l, L.n_in, L.n_att);
        PGK_REQUIRE(L.w_in && L.w_o && (!L.ff_pad || (L.w_gate_up && L.w_down)), "pgk_engine_create_stack: layer %d: missing weights", l);
        PGK_REQUIRE((c.block == PGK_BLOCK_HYPER) == (L.mixer == PGK_MIX_TALK), "pgk_engine_create_stack: layer %d: mixer %d in block kind %d", l, L.mixer, c.block);
        if (c.block == PGK_BLOCK_HYPER) {
            PGK_REQUIRE(L.norm1 && L.hyper1 && (!L.ff_pad || (L.norm2 && L.hyper2)), "pgk_engine_create_stack: layer %d: missing norms or stream weights", l);
            PGK_REQUIRE(!L.ff_pad || (L.ff == PGK_FF_POLY ? L.act && L.ff_dim >= 1 && L.ff_dim <= L.ff_pad
                                                         : L.ff == PGK_FF_TABLE && L.table && L.experts >= 1 && L.experts <= MOE_MAX_EXPERTS && L.top >= 1 && L.top <= L.experts && L.top <= MOE_MAX_TOP &&
                                                               L.shared_pad >= 0 && L.shared_pad % 64 == 0 && (!L.shared_pad || (L.w_shared_up && L.w_shared_down && L.w_shared_gate))),
                        "pgk_engine_create_stack: layer %d: feed-forward %d of %d, %d experts, top %d, shared %d", l, L.ff, L.ff_pad, L.experts, L.top, L.shared_pad);
        } else if (c.block == PGK_BLOCK_PARALLEL) {
            PGK_REQUIRE(L.norm1 && (!L.ff_pad || (L.ff == PGK_FF_MOE && L.correction)), "pgk_engine_create_stack: layer %d: a parallel layer has one norm and experts or no feed-forward", l);
            if (L.ff_pad)
                PGK_REQUIRE(L.experts >= 1 && L.experts <= MOE_MAX_EXPERTS && L.top >= 1 && L.top <= L.experts && L.top <= MOE_MAX_TOP && L.groups >= 0 &&
                                (L.groups == 0 || (L.experts % L.groups == 0 && L.keep >= 1 && L.keep <= L.groups && L.keep * (L.experts / L.groups) >= L.top)),
                            "pgk_engine_create_stack: layer %d: %d experts, top %d, %d of %d groups", l, L.experts, L.top, L.keep, L.groups);
        } else {
            PGK_REQUIRE(L.norm1b && (!L.ff_pad || (L.ff <= PGK_FF_XIELU && L.norm2b)), "pgk_engine_create_stack: layer %d: missing norms", l);
        }
        const int HD = L.heads * L.head_pad;
        if (L.mixer == PGK_MIX_DELTA || L.mixer == PGK_MIX_SSD) {
            const bool delta = L.mixer == PGK_MIX_DELTA;
            PGK_REQUIRE(L.kv_heads >= 1 && L.heads % L.kv_heads == 0 && L.head_pad % 16 == 0 && L.vhead_pad % 16 == 0 && L.head_pad >= L.dim && L.vhead_pad >= L.vdim && L.taps >= 1 && L.kv_from < 0 &&
                            L.n_att >= L.heads * L.vhead_pad && L.n_in >= (delta ? delta_a_off(L) + L.rank_a + L.rank_g : conv_channels(L) + L.heads * L.vhead_pad + L.heads),
                        "pgk_engine_create_stack: layer %d: %d / %d heads of %d / %d padded to %d / %d, %d taps", l, L.heads, L.kv_heads, L.dim, L.vdim, L.head_pad, L.vhead_pad, L.taps);
            PGK_REQUIRE(L.conv && L.o_norm && L.decay && L.dt_bias && (delta ? L.w_a2 && L.w_g2 : L.skip != nullptr), "pgk_engine_create_stack: layer %d: missing weights", l);
            PGK_REQUIRE(delta ? L.rank_a % 64 == 0 && L.rank_a >= 64 && L.rank_g % 64 == 0 && L.rank_g >= 64 : L.norm_parts >= 1 && L.heads * L.vdim % L.norm_parts == 0,
                        "pgk_engine_create_stack: layer %d: ranks %d / %d, %d norm parts", l, L.rank_a, L.rank_g, L.norm_parts);
            continue;
        }
        if (L.mixer == PGK_MIX_HGRN2) {
            PGK_REQUIRE(L.head_pad % 16 == 0 && L.vhead_pad % 16 == 0 && L.head_pad >= L.dim && L.vhead_pad >= L.vdim && L.n_in >= 2 * HD + L.heads * L.vhead_pad && L.n_att >= L.heads * L.vhead_pad,
                        "pgk_engine_create_stack: layer %d: head widths %d / %d padded to %d / %d", l, L.dim, L.vdim, L.head_pad, L.vhead_pad);
            PGK_REQUIRE(L.lower && L.o_norm, "pgk_engine_create_stack: layer %d: missing weights", l);
            continue;
        }
        PGK_REQUIRE(L.window >= 1 && L.head_pad % 64 == 0 && L.head_pad >= L.dim && L.head_pad >= L.vdim && L.n_att == HD, "pgk_engine_create_stack: layer %d: window %d, head pad %d for widths %d / %d", l, L.window, L.head_pad, L.dim, L.vdim);
        if (L.mixer == PGK_MIX_LATENT) {
            PGK_REQUIRE(L.rank >= 1 && L.rank_pad % 64 == 0 && L.rank_pad >= L.rank + L.rot && L.rank_pad <= 2048 && L.rot >= 0 && L.rot % 2 == 0 && L.rot <= L.dim && (!L.rot || L.rot_freq), "pgk_engine_create_stack: layer %d: latent size %d padded to %d (at most 2048)", l, L.rank, L.rank_pad);
            PGK_REQUIRE(L.n_in >= HD + L.rank_pad + (L.gated ? L.heads : 0) && L.kv_heads == L.heads && L.kv_from < 0, "pgk_engine_create_stack: layer %d: in-projection rows %d", l, L.n_in);
            PGK_REQUIRE(L.norm1 && L.c_norm && L.w_ukv, "pgk_engine_create_stack: layer %d: missing weights", l);
        } else if (L.mixer == PGK_MIX_TALK) {
            PGK_REQUIRE(L.kv_heads >= 1 && L.heads % L.kv_heads == 0 && L.head_pad <= 1024 && L.rot >= 0 && L.rot % 2 == 0 && L.rot <= L.dim && (!L.rot || L.rot_freq) && L.q_norm && (L.kv_from >= 0 || L.k_norm) &&
                            L.n_in >= HD + (L.kv_from < 0 ? 2 * L.kv_heads * L.head_pad : 0),
                        "pgk_engine_create_stack: layer %d: %d / %d heads of %d, %d turned, in-projection rows %d", l, L.heads, L.kv_heads, L.head_pad, L.rot, L.n_in);
            PGK_REQUIRE(L.kv_from < 0 || (L.kv_from < l && layers[L.kv_from].mixer == PGK_MIX_TALK && layers[L.kv_from].kv_from < 0 && layers[L.kv_from].kv_heads == L.kv_heads && layers[L.kv_from].head_pad == L.head_pad),
                        "pgk_engine_create_stack: layer %d cannot take the keys and values of layer %d", l, L.kv_from);
        } else {
            PGK_REQUIRE(L.kv_heads >= 1 && L.heads % L.kv_heads == 0 && L.head_pad <= 1024 && L.taps >= 1, "pgk_engine_create_stack: layer %d: %d / %d heads of %d, %d taps", l, L.heads, L.kv_heads, L.head_pad, L.taps);
            PGK_REQUIRE(L.n_in >= 2 * HD + (L.kv_from < 0 ? 2 * L.kv_heads * L.head_pad : 0), "pgk_engine_create_stack: layer %d: in-projection rows %d", l, L.n_in);
            if (L.kv_from >= 0) {
                PGK_REQUIRE(L.kv_from < l && layers[L.kv_from].mixer == PGK_MIX_ATTENTION && layers[L.kv_from].kv_from < 0 && layers[L.kv_from].kv_heads == L.kv_heads && layers[L.kv_from].head_pad == L.head_pad,
                            "pgk_engine_create_stack: layer %d cannot take the keys and values of layer %d", l, L.kv_from);
            }
        }
    }
    PGK_REQUIRE(c.block != PGK_BLOCK_HYPER || (c.streams >= 1 && c.streams <= HYPER_MAX_STREAMS && c.norm_groups >= 1 && c.norm_groups <= NORM_MAX_GROUPS && c.width % c.norm_groups == 0),
                "pgk_engine_create_stack: %d streams, %d norm groups of %d", c.streams, c.norm_groups, c.width);
    PGK_REQUIRE(c.block == PGK_BLOCK_HYPER || (c.norm_groups <= 1 && !(c.logit_cap > 0.f)), "pgk_engine_create_stack: norms in groups and capped logits belong to hyper-connected layers");
    PGK_REQUIRE(c.loop_times >= 0 && (!c.loop_times || (c.block == PGK_BLOCK_PARALLEL && c.loop_start >= 0 && c.loop_start < c.loop_stop && c.loop_stop <= c.num_layers && c.loop_in && c.loop_step)),
                "pgk_engine_create_stack: layers %d .. %d of %d, %d times", c.loop_start, c.loop_stop - 1, c.num_layers, c.loop_times);
    Engine* e = new Engine();
    Stack* s = new Stack();
    e->kind = &STACK_KIND;
    e->kind_state = s;
    e->one_sequence = true;
    s->cfg = c;
    s->layers.assign(layers, layers + c.num_layers);
    for (int l = 0; l < c.num_layers; ++l) {
        if (c.loop_times && l == c.loop_start) {
            for (int t = 0; t < c.loop_times; ++t)
                for (int k = c.loop_start; k < c.loop_stop; ++k) s->runs.push_back(Run{k, k == c.loop_start ? t : -1});
            l = c.loop_stop - 1;
        } else s->runs.push_back(Run{l, -1});
    }
    for (int l = 0; l < c.num_layers; ++l)
        if (c.loop_times && layers[l].kv_from >= 0) { delete s; delete e; return set_error(PGK_ERR_UNSUPPORTED, "pgk_engine_create_stack: layer %d takes another layer's keys in a model with a loop", l); }
    s->embed = embed; s->pos = pos_embed; s->head = head; s->final_norm = final_norm;
    s->Wp = Wp;
    s->len.assign(c.max_batch, 0);
    e->cfg = pgk_model_config_t{};
    e->cfg.vocab_size = c.vocab_size; e->cfg.hidden_size = c.width; e->cfg.num_layers = s->n_runs();
    e->cfg.max_seq_len = c.max_seq_len; e->cfg.max_batch = c.max_batch; e->cfg.norm_eps = c.norm_eps;
    {
        int dev = 0;
        hipDeviceProp_t prop;
        if (hipGetDevice(&dev) == hipSuccess && hipGetDeviceProperties(&prop, dev) == hipSuccess && prop.multiProcessorCount > 0) e->cu_count = prop.multiProcessorCount;
    }
    e->lm_blocks = ceil_div(c.vocab_size, 16) < 1024 ? ceil_div(c.vocab_size, 16) : 1024;
    if (c.block == PGK_BLOCK_HYPER && hyper_wide(s->Wp)) e->lm_blocks = min(e->lm_blocks, HYPER_WIDE_GRID);
    e->lm_cap = e->lm_blocks > ROWS_ARGMAX_BLOCKS ? e->lm_blocks : ROWS_ARGMAX_BLOCKS;
    pgk_status r = PGK_OK;
    std::vector<std::pair<void*, size_t>> clear;
    auto A = [&](void** p, size_t bytes, size_t* acct, bool zero = false) {
        if (r == PGK_OK) r = dev_alloc(e, p, bytes, acct);
        if (r == PGK_OK && zero) clear.push_back({*p, bytes});
    };
    const size_t B = c.max_batch, E = s->esize();
    size_t part = 0, ml = 0, ql = 0;
    int max_router = 0, max_act = 0;
    auto most = [](auto& m, auto v) { if (v > m) m = v; };
    s->reach.assign(s->n_runs(), 0);
    s->readers.resize(s->n_runs());
    for (int l = 0; l < s->n_runs(); ++l) {
        const auto& L = s->at(l);
        if (recurrent(L)) continue;
        auto& rd = s->readers[kv_source(L, l)];
        const std::pair<int, int> span{L.window, L.chunked ? 1 : 0};
        most(s->reach[kv_source(L, l)], L.window);
        const auto at = std::lower_bound(rd.begin(), rd.end(), span);
        if (at == rd.end() || *at != span) rd.insert(at, span);
    }
    for (int l = 0; l < s->n_runs(); ++l) {
        const auto& L = s->at(l);
        const int R = s->reach[l] < c.max_seq_len ? s->reach[l] : c.max_seq_len, HD = L.heads * L.head_pad;
        s->ring.push_back(R);
        void *p = nullptr, *t = nullptr;
        if (L.mixer == PGK_MIX_LATENT) A(&p, B * R * L.rank_pad * E, &e->kv_bytes, true);
        else if (recurrent(L)) {
            A(&p, B * HD * L.vhead_pad * 4, &e->kv_bytes, true);
            const int ch = conv_channels(L);
            if (ch) A(&t, B * L.taps * ch * E, &e->kv_bytes, true);
            most(s->max_conv, ch);
            if (L.mixer == PGK_MIX_DELTA) {
                most(s->max_z, HD);
                most(s->max_gate, L.heads * L.vhead_pad);
                most(s->max_low, L.rank_a > L.rank_g ? L.rank_a : L.rank_g);
            }
        }
        else {
            const int GD = L.kv_heads * L.head_pad;
            if (L.kv_from < 0) A(&p, B * 2 * R * GD * E, &e->kv_bytes, true);
            else p = s->cache[L.kv_from];
            if (L.conv) A(&t, B * L.taps * (HD + (L.kv_from < 0 ? 2 * GD : 0)) * E, &e->kv_bytes, true);
            most(s->max_q, HD);
        }
        s->cache.push_back(p);
        s->taps.push_back(t);
        most(s->max_in, L.n_in);
        most(s->max_att, L.n_att);
        if (has_experts(L)) { most(s->max_top, L.top); most(max_router, router_rows(L)); most(max_act, L.top * L.ff_pad + L.shared_pad + 64); }
        else most(max_act, L.ff_pad);
        most(s->max_ff, dense_ff(L));
        for (int m = 1; m <= c.max_batch && !recurrent(L); ++m) {
            const int src = kv_source(L, l), keys = L.window < s->ring[src] ? L.window : s->ring[src];
            const size_t ns = (size_t)(L.mixer == PGK_MIX_LATENT ? pick_nsplit(e, m, L, R) : L.mixer == PGK_MIX_TALK ? talk_splits(m, L.heads, L.kv_heads, keys, e->cu_count) : kv_attn_splits(m, L.heads, L.kv_heads, keys, e->cu_count)) * m * L.heads;
            most(part, ns * (L.mixer == PGK_MIX_LATENT ? L.rank_pad : L.head_pad));
            most(ml, ns * 2);
        }
        if (L.mixer == PGK_MIX_LATENT) most(ql, B * L.heads * L.rank_pad);
    }
    A((void**)&e->tokens, B * 4, &e->ws_bytes, true);
    A((void**)&e->positions, B * 4, &e->ws_bytes, true);
    A((void**)&e->token_log, (size_t)e->log_cap * B * 4, &e->ws_bytes);
    A((void**)&e->step_counter, 16, &e->ws_bytes, true);
    A((void**)&e->h, B * Wp * 4, &e->ws_bytes, true);
    A((void**)&e->h2, B * Wp * 4, &e->ws_bytes, true);
    A((void**)&e->logits, B * c.vocab_size * 4, &e->ws_bytes);
    A((void**)&e->amax_val, B * e->lm_cap * 4, &e->ws_bytes);
    A((void**)&e->amax_idx, B * e->lm_cap * 4, &e->ws_bytes);
    A((void**)&e->clk_log, (size_t)e->log_cap * 16, &e->ws_bytes);
    A((void**)&s->in32, (size_t)(s->max_in + max_router) * 4, &e->ws_bytes);
    A((void**)&s->a32, (size_t)s->max_att * 4, &e->ws_bytes, true);     // padding columns of a head are never written: zero
    A((void**)&s->y32, (size_t)Wp * 4, &e->ws_bytes, true);
    A((void**)&s->act32, (size_t)(max_act ? max_act : 64) * 4, &e->ws_bytes);
    if (c.block == PGK_BLOCK_HYPER) {
        for (auto& x : s->xs) A((void**)&x, (size_t)c.streams * Wp * 4, &e->ws_bytes, true);
        A((void**)&s->xrows, B * c.streams * Wp * 4, &e->ws_bytes, true);
        A((void**)&s->ygate, B * 4, &e->ws_bytes, true);
    }
    if (c.block == PGK_BLOCK_PARALLEL || c.block == PGK_BLOCK_HYPER) {
        A((void**)&s->y32b, (size_t)Wp * 4, &e->ws_bytes, true);
        A((void**)&s->h32, (size_t)Wp * 4, &e->ws_bytes, true);
        A((void**)&s->ids, MOE_MAX_TOP * 4, &e->ws_bytes, true);
        if (c.loop_times) A(&s->cat16, B * 2 * Wp * E, &e->ws_bytes);
        if (s->max_top) A(&s->e16, B * s->max_top * Wp * E, &e->ws_bytes);
        size_t ws = 0;
        for (int m = 2; m <= c.max_batch; ++m) most(ws, s->moe_ws(m));
        if (ws) A(&s->moe16, ws, &e->ws_bytes);
    }
    if (s->max_z) {
        A((void**)&s->z32, B * s->max_z * 4, &e->ws_bytes);
        A(&s->gate, B * s->max_gate * 4, &e->ws_bytes);
    }
    auto some = [](size_t v) { return v ? v : (size_t)64; };
    A(&s->qlat, some(ql) * 4, &e->ws_bytes);
    A(&s->qx, some(B * s->max_q) * 4, &e->ws_bytes);
    A((void**)&s->po, some(part) * 4, &e->ws_bytes);
    A((void**)&s->pml, some(ml) * 4, &e->ws_bytes);
    A(&s->x16, B * Wp * E, &e->ws_bytes);
    A(&s->in16, B * s->max_in * E, &e->ws_bytes);
    A(&s->a16, B * s->max_att * E, &e->ws_bytes, true);
    A(&s->y16, B * Wp * E, &e->ws_bytes);
    A(&s->gu16, B * 2 * (s->max_ff ? s->max_ff : 64) * E, &e->ws_bytes);
    A(&s->act16, B * (s->max_ff ? s->max_ff : 64) * E, &e->ws_bytes);
    if (r == PGK_OK && c.dtype == PGK_BF16) {
        // a second, fragment-major copy of the layer matrices where the skinny GEMM takes their shapes, unless that is more than a
        // quarter of the free memory; PGK_PACKED_PREFILL=0: none
        hipStream_t st = resolve_stream(nullptr);
        const char* ep = getenv("PGK_PACKED_PREFILL");
        size_t total = 0, free_b = 0, total_b = 0;
        auto visit = [&](auto fn) {
            for (int l = 0; l < c.num_layers; ++l) {
                const auto& L = s->layers[l];
                auto& P = s->packed[l];
                if (pkgemm_shape_ok(L.n_in, Wp, false)) fn(&P.in, L.w_in, L.n_in, Wp);
                if (pkgemm_shape_ok(Wp, L.n_att, true)) fn(&P.o, L.w_o, Wp, L.n_att);
                if (!dense_ff(L)) continue;
                if (pkgemm_shape_ok(up_rows(L), Wp, false)) fn(&P.gate_up, dense_up(L), up_rows(L), Wp);
                if (pkgemm_shape_ok(Wp, dense_ff(L), true)) fn(&P.down, dense_down(L), Wp, dense_ff(L));
            }
        };
        s->packed.resize(c.num_layers);
        visit([&](bf16**, const void*, int N, int K) { total += (size_t)N * K * 2; });
        if (!(ep && atoi(ep) == 0) && hipMemGetInfo(&free_b, &total_b) == hipSuccess && total < free_b / 4)
            visit([&](bf16** dst, const void* w, int N, int K) {
                A((void**)dst, (size_t)N * K * 2, &e->packed_bytes);
                if (r == PGK_OK) r = pack_weights_bf16(w, *dst, N, K, st);
            });
    }
    size_t slab = 64;
    for (int m = 2; m <= c.max_batch; ++m) { const size_t z = s->slab_elems(m, c.dtype == PGK_F32); slab = z > slab ? z : slab; }
    A((void**)&s->slabs16, slab * 4, &e->ws_bytes);
    if (r == PGK_OK) {
        hipStream_t st = resolve_stream(nullptr);
        hipError_t he = hipSuccess;
        for (const auto& z : clear) if (he == hipSuccess) he = hipMemsetAsync(z.first, 0, z.second, st);
        if (he == hipSuccess) he = hipStreamSynchronize(st);
        if (he != hipSuccess) r = set_error(PGK_ERR_HIP, "pgk_engine_create_stack: %s", hipGetErrorString(he));
    }
    if (r != PGK_OK) { pgk_engine_destroy(e); return r; }
    *out = e;
    return PGK_OK;
}

}  // extern "C"
