// Mixture of experts (ops_moe.hip; the one-row kernels of a decode step are in engine_stack.hip): a router, or a table of token ids, picks
// `top` of E experts per row; every expert is a SwiGLU or a gelu feed-forward.
#pragma once

#include "engine_common.hip.h"
#include "latent.hip.h"

namespace pgk {

// Choice: s = sigmoid(z), c = s + correction.  With groups > 0 only experts of the `keep` groups of neighbours with the largest sum of
// their two largest c can be chosen.  The `top` experts with the largest c (lowest index on ties), weights s / (sum of the chosen s + 1e-20)
// * scale.
// With a table [tokens][top] there is no router: its row of the token names the experts, each with weight 1 / top.
struct RouterCfg { const float* correction; int E, top, groups, keep; float scale; const int32_t* table; };

constexpr int MOE_MAX_EXPERTS = 1024, MOE_MAX_TOP = 64;
struct RouteScratch { float *s, *c, *g, *w; };                     // LDS: [E], [E], [2 groups], [top]
__host__ __device__ inline int route_floats(const RouterCfg& r) { return 2 * r.E + 2 * r.groups + r.top; }

// NT threads (tid 0 .. NT - 1) choose for one row; `logit(e)` is z_e, ids and weights go to LDS or memory, `sync` separates the phases
// and is called once more at the end.
template <int NT, class L, class Sync>
__device__ __forceinline__ void route_row(const RouterCfg& r, float* lds, int tid, L logit, int32_t* ids, float* wts, Sync sync) {
    float *s = lds, *c = s + r.E, *gs = c + r.E, *gk = gs + r.groups, *w = gk + r.groups;
    for (int e = tid; e < r.E; e += NT) {
        s[e] = 1.0f / (1.0f + expf(-logit(e)));
        c[e] = s[e] + r.correction[e];
    }
    for (int i = tid; i < r.top; i += NT) { ids[i] = 0; w[i] = 0.f; }
    sync();
    if (r.groups > 0) {
        const int n = r.E / r.groups;
        for (int g = tid; g < r.groups; g += NT) {
            float a = -INFINITY, b = -INFINITY;
            for (int i = 0; i < n; ++i) { const float v = c[g * n + i]; if (v > a) { b = a; a = v; } else b = fmaxf(b, v); }
            gs[g] = n > 1 ? a + b : a;
        }
        sync();
        for (int g = tid; g < r.groups; g += NT) {
            int rank = 0;
            for (int j = 0; j < r.groups; ++j) rank += gs[j] > gs[g] || (gs[j] == gs[g] && j < g);
            gk[g] = rank < r.keep ? 1.f : 0.f;
        }
        sync();
        for (int e = tid; e < r.E; e += NT) if (gk[e / n] == 0.f) c[e] = -INFINITY;
        sync();
    }
    for (int e = tid; e < r.E; e += NT) {
        const float v = c[e];
        if (v == -INFINITY) continue;
        int rank = 0;
        for (int j = 0; j < r.E; ++j) rank += c[j] > v || (c[j] == v && j < e);
        if (rank < r.top) { ids[rank] = e; w[rank] = s[e]; }
    }
    sync();
    float sum = 0.f;
    for (int i = 0; i < r.top; ++i) sum += w[i];
    for (int i = tid; i < r.top; i += NT) wts[i] = w[i] / (sum + 1e-20f) * r.scale;
    sync();
}

// A run of rows of one expert: rows row0 .. row0 + rows - 1 of the rows sorted by expert
struct MoeTile { int32_t expert, row0, rows, pad; };
// Operands of a product over rows sorted by expert: tile list, its length, the sorted rows' places (row * top + k), their weights, elements
// between two experts' matrices.  A's row of sorted row p is place / div (div > 0) or p.
struct GroupArgs { const MoeTile* tiles; const int32_t* n_tiles; const int32_t* order; const float* wts; long long w_stride; int div; };

// What a product over rows sorted by expert leaves: SwiGLU rows of fused gate | up matrices, gelu rows, or weighted rows at their places
enum MoeProduct { MOE_SWIGLU = 0, MOE_GELU = 1, MOE_DOWN = 2 };

struct MoeArgs {
    const void* x;                        // [n][W], element type; W a multiple of 64
    int n, W, ff;                         // ff: a multiple of 64
    RouterCfg router;
    const void *w_router, *w_up, *w_down; // [E up to a multiple of 64][W] (with a table: unused), [E][2 ff][W] (gate rows, up rows; gelu: [E][ff][W]), [E][W][ff]
    void* out;                            // [n][top][W], element type: weighted expert outputs
    void* ws;                             // moe_bytes(...)
    bool gelu = false;
    const int32_t* tok = nullptr;         // with a table: the rows' tokens
};
size_t moe_bytes(int n, int W, int ff, const RouterCfg& r, pgk_dtype dt);
pgk_status moe_rows(const MoeArgs& a, pgk_dtype dt, hipStream_t st);

// ops_gemm256.hip: 128 x 128 tiles over rows sorted by expert (tile list of runs of up to 128 rows): SwiGLU rows act [p][N] from fused
// gate | up matrices [2 N, K], gelu rows from [N, K], or (down) weighted rows C [place][N]
pgk_status gemm128s_grouped(const bf16* A, const bf16* W, bf16* C, MoeProduct what, const GroupArgs& g, int max_tiles, int rows, int N, int K, hipStream_t st);

}  // namespace pgk
