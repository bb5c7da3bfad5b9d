// Mixture of experts over rows (moe.hip.h): router logits (fp32) -> choice, or a table of tokens -> rows sorted by expert -> grouped SwiGLU or gelu -> grouped down
// projection, each result weighted and stored at [row][k].  The rows' sum over k is left to the norm that follows (rows_norm).
// Nothing about the distribution is known on the host: grids are sized for the worst case, a tile list says what a workgroup does.

#include <type_traits>

#include "moe.hip.h"

namespace pgk {

pgk_status wsgemm_nt(const bf16* a, int lda, const void* w, const bf16* wscale, bool fp8, void* c, const bf16* bias, int mode,
                     int splits, int M, int N, int K, hipStream_t st);
int wsgemm_pick_splits(int N, int K, bool allow_split);
bool gemm128s_ok(int M, int N, int K);
struct QkvHeadArgs;
struct ActArgs;
pgk_status gemm128s_bf16_nt(const bf16* A, const bf16* W, const bf16* bias, void* C, int mode, int splits, int M, int N, int K, hipStream_t st,
                            const QkvHeadArgs* heads, bool packed, const ActArgs* act);

// -------------------------------------------------------------------------------------------- choice and sorting
// A wave per row; logits are the sum of `slabs` fp32 slabs
__global__ __launch_bounds__(256) void moe_route_kernel(RouterCfg r, const float* logits, int ld, int slabs, size_t slab_stride, int n, int32_t* ids, float* wts) {
    extern __shared__ float rt_smem[];
    const int wid = threadIdx.x >> 6, row = blockIdx.x * 4 + wid;
    if (row >= n) return;                                          // (no workgroup barrier below)
    auto logit = [&](int e) {
        float z = 0.f;
        for (int s = 0; s < slabs; ++s) z += logits[s * slab_stride + (size_t)row * ld + e];
        return z;
    };
    auto sync = []() { __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront"); __builtin_amdgcn_wave_barrier(); __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront"); };
    route_row<64>(r, rt_smem + wid * route_floats(r), threadIdx.x & 63, logit, ids + (size_t)row * r.top, wts + (size_t)row * r.top, sync);
}

__global__ __launch_bounds__(256) void moe_table_kernel(const int32_t* table, const int32_t* tok, int total, int top, int32_t* ids, float* wts) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= total) return;
    ids[i] = table[(size_t)tok[i / top] * top + i % top];
    wts[i] = 1.0f / top;
}

// Workgroup e writes expert e's places in ascending order and its runs of `tm` rows to the tile list
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int32_t* ids, int total, int E, int tm, int32_t* order, MoeTile* tiles, int32_t* n_tiles) {
    __shared__ int hist[MOE_MAX_EXPERTS], sum[16][3], base_s[3];
    const int e = blockIdx.x, NT = blockDim.x, tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, nw = NT >> 6;
    for (int i = tid; i < E; i += NT) hist[i] = 0;
    __syncthreads();
    const int per = (total + NT - 1) / NT, i0 = min(tid * per, total), i1 = min(i0 + per, total);
    int own = 0;
    for (int i = i0; i < i1; ++i) {
        const int id = ids[i];
        atomicAdd(&hist[id], 1);
        own += id == e;
    }
    __syncthreads();
    int before = 0, tiles_before = 0, tiles_all = 0;
    for (int i = tid; i < E; i += NT) {
        const int c = hist[i], t = (c + tm - 1) / tm;
        tiles_all += t;
        if (i < e) { before += c; tiles_before += t; }
    }
    int scan = own;                                                // inclusive scan over the workgroup
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const int t = __shfl_up(scan, off, 64);
        if (lane >= off) scan += t;
        before += __shfl_xor(before, off, 64);
        tiles_before += __shfl_xor(tiles_before, off, 64);
        tiles_all += __shfl_xor(tiles_all, off, 64);
    }
    __shared__ int wsum[16];
    if (lane == 63) wsum[wid] = scan;
    if (lane == 0) { sum[wid][0] = before; sum[wid][1] = tiles_before; sum[wid][2] = tiles_all; }
    __syncthreads();
    if (tid < 3) {
        int t = 0;
        for (int w = 0; w < nw; ++w) t += sum[w][tid];
        base_s[tid] = t;
    }
    int at = scan - own;
    for (int w = 0; w < wid; ++w) at += wsum[w];
    __syncthreads();
    at += base_s[0];
    for (int i = i0; i < i1; ++i)
        if (ids[i] == e) order[at++] = i;
    const int count = hist[e];
    for (int t = tid; t * tm < count; t += NT) tiles[base_s[1] + t] = MoeTile{e, base_s[0] + t * tm, min(tm, count - t * tm), 0};
    if (e == 0 && tid == 0) *n_tiles = base_s[2];
}

// -------------------------------------------------------------------------------------------- few rows per expert, bf16
// The weight-streaming product of ops_wsgemm.hip on a tile list: a wave has 16 weight rows (SwiGLU: 16 gate rows and the matching up rows),
// which are read once from memory as the MFMA operand; the tile's rows (up to 16 MT) pass through LDS in pieces of 256 k.
typedef __bf16 bf16x8_me __attribute__((ext_vector_type(8)));
typedef float f32x4_me __attribute__((ext_vector_type(4)));
constexpr int ME_KT = 256;
__device__ __forceinline__ int me_off(int r, int c) { return r * (ME_KT * 2) + (((c & ~15) | ((c ^ r) & 15)) << 4); }

template <int MT, MoeProduct P>
__global__ __launch_bounds__(256) void moe_stream_kernel(const bf16* A, const bf16* W, bf16* C, int N, int K, GroupArgs ga) {
    __shared__ __attribute__((aligned(16))) char a_lds[MT * 16 * ME_KT * 2];
    if ((int)blockIdx.y >= *ga.n_tiles) return;
    const MoeTile t = ga.tiles[blockIdx.y];
    constexpr int NB = P == MOE_SWIGLU ? 2 : 1;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l15 = lane & 15, q4 = lane >> 4, n0 = (blockIdx.x * 4 + wid) * 16, kl = 8 * q4;
    const bf16* wr[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) wr[b] = W + t.expert * ga.w_stride + (size_t)(b * N + min(n0 + l15, N - 1)) * K;
    constexpr int ACH = MT * 2;
    const bf16* ar[ACH];
#pragma unroll
    for (int i = 0; i < ACH; ++i) {
        const int p = t.row0 + min((int)(threadIdx.x + i * 256) >> 5, t.rows - 1);
        ar[i] = A + (size_t)(ga.div > 0 ? ga.order[p] / ga.div : p) * K;
    }
    uint4 wreg[NB][8], areg[ACH];
    auto load_w = [&](int kt) {
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int s = 0; s < 8; ++s) wreg[b][s] = load_nt16(wr[b] + min(kt + s * 32 + kl, K - 8));
    };
    auto load_a = [&](int kt) {
#pragma unroll
        for (int i = 0; i < ACH; ++i) areg[i] = *reinterpret_cast<const uint4*>(ar[i] + min(kt + (int)((threadIdx.x + i * 256) & 31) * 8, K - 8));
    };
    f32x4_me acc[NB][MT];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[b][m] = f32x4_me{0.f, 0.f, 0.f, 0.f};
    load_w(0);
    load_a(0);
    for (int kt = 0; kt < K; kt += ME_KT) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < ACH; ++i) {
            const int chn = threadIdx.x + i * 256, r = chn >> 5, c = chn & 31;
            const bool ok = r < t.rows && kt + c * 8 < K;
            *reinterpret_cast<uint4*>(a_lds + me_off(r, c)) = make_uint4(ok ? areg[i].x : 0u, ok ? areg[i].y : 0u, ok ? areg[i].z : 0u, ok ? areg[i].w : 0u);
        }
        __syncthreads();
        uint4 wcur[NB][8];
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int s = 0; s < 8; ++s) wcur[b][s] = wreg[b][s];
        if (kt + ME_KT < K) { load_w(kt + ME_KT); load_a(kt + ME_KT); }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int s = 0; s < 8; ++s) {
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                const uint4 af = *reinterpret_cast<const uint4*>(a_lds + me_off(m * 16 + l15, s * 4 + q4));
#pragma unroll
                for (int b = 0; b < NB; ++b)
                    acc[b][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_me, af), __builtin_bit_cast(bf16x8_me, wcur[b][s]), acc[b][m], 0, 0, 0);
            }
        }
    }
    const int n = n0 + l15;
    if (n >= N) return;
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 16 * m + 4 * q4 + r;
            if (row >= t.rows) continue;
            if constexpr (P == MOE_SWIGLU) {
                const float g = acc[0][m][r];
                C[(size_t)(t.row0 + row) * N + n] = from_f<bf16>(g / (1.0f + __expf(-g)) * acc[NB - 1][m][r]);
            } else if constexpr (P == MOE_GELU) {
                C[(size_t)(t.row0 + row) * N + n] = from_f<bf16>(gelu_erf(acc[0][m][r]));
            } else {
                const int place = ga.order[t.row0 + row];
                C[(size_t)place * N + n] = from_f<bf16>(acc[0][m][r] * ga.wts[place]);
            }
        }
}

// -------------------------------------------------------------------------------------------- fp32
template <MoeProduct P>
__global__ __launch_bounds__(256) void moe_f32_kernel(const float* A, const float* W, float* C, int N, int K, GroupArgs ga) {
    constexpr int NB = P == MOE_SWIGLU ? 2 : 1, TM = 32, TN = 64, TK = 16;
    __shared__ float As[TK][TM + 1], Bs[NB][TK][TN + 1];
    if ((int)blockIdx.y >= *ga.n_tiles) return;
    const MoeTile t = ga.tiles[blockIdx.y];
    const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4, n0 = blockIdx.x * TN;
    const float* w = W + t.expert * ga.w_stride;
    float acc[NB][2][4] = {};
    for (int k0 = 0; k0 < K; k0 += TK) {
        for (int i = threadIdx.x; i < TM * TK; i += 256) {
            const int r = i / TK, k = i % TK, p = t.row0 + min(r, t.rows - 1);
            As[k][r] = A[(size_t)(ga.div > 0 ? ga.order[p] / ga.div : p) * K + k0 + k];
        }
#pragma unroll
        for (int b = 0; b < NB; ++b)
            for (int i = threadIdx.x; i < TN * TK; i += 256) Bs[b][i % TK][i / TK] = w[(size_t)(b * N + min(n0 + i / TK, N - 1)) * K + k0 + i % TK];
        __syncthreads();
#pragma unroll
        for (int k = 0; k < TK; ++k)
#pragma unroll
            for (int b = 0; b < NB; ++b)
#pragma unroll
                for (int i = 0; i < 2; ++i)
#pragma unroll
                    for (int j = 0; j < 4; ++j) acc[b][i][j] = fmaf(As[k][2 * ty + i], Bs[b][k][4 * tx + j], acc[b][i][j]);
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int row = 2 * ty + i, n = n0 + 4 * tx + j;
            if (row >= t.rows || n >= N) continue;
            if constexpr (P == MOE_SWIGLU) {
                const float g = acc[0][i][j];
                C[(size_t)(t.row0 + row) * N + n] = g / (1.0f + expf(-g)) * acc[NB - 1][i][j];
            } else if constexpr (P == MOE_GELU) {
                C[(size_t)(t.row0 + row) * N + n] = gelu_erf(acc[0][i][j]);
            } else {
                const int place = ga.order[t.row0 + row];
                C[(size_t)place * N + n] = acc[0][i][j] * ga.wts[place];
            }
        }
}

// -------------------------------------------------------------------------------------------- all of it
namespace {
struct MoePlan {
    int Ep, slabs, tm, max_tiles, total;
    size_t logits, act, ids, wts, order, tiles, count, bytes;
};
size_t up256(size_t v) { return (v + 255) & ~(size_t)255; }
MoePlan moe_plan(int n, int W, int ff, const RouterCfg& r, pgk_dtype dt) {
    MoePlan p{};
    p.Ep = ceil_div(r.E, 64) * 64;
    p.total = n * r.top;
    const double per = (double)p.total / r.E;                      // rows per expert
    p.tm = dt == PGK_F32 ? 32 : n > 128 && per > 40 ? 128 : per > 12 ? 32 : 16;
    p.max_tiles = p.total / p.tm + (p.total < r.E ? p.total : r.E);
    p.slabs = 1;
    if (dt != PGK_F32) {
        if (n <= 128) p.slabs = wsgemm_pick_splits(p.Ep, W, true);
        else {
            const int blocks = ceil_div(n, 128) * ceil_div(p.Ep, 128);
            while (p.slabs < 16 && 2 * p.slabs * blocks <= 512 && W % (128 * p.slabs) == 0 && W / (2 * p.slabs) >= 256) p.slabs *= 2;
        }
    }
    size_t at = 0;
    auto take = [&](size_t b) { const size_t o = at; at += up256(b); return o; };
    p.logits = take((size_t)p.slabs * n * p.Ep * 4);
    p.act = take((size_t)p.total * ff * (dt == PGK_F32 ? 4 : 2));
    p.ids = take((size_t)p.total * 4);
    p.wts = take((size_t)p.total * 4);
    p.order = take((size_t)p.total * 4);
    p.tiles = take((size_t)p.max_tiles * sizeof(MoeTile));
    p.count = take(4);
    p.bytes = at;
    return p;
}
}  // namespace

size_t moe_bytes(int n, int W, int ff, const RouterCfg& r, pgk_dtype dt) { return moe_plan(n, W, ff, r, dt).bytes; }

pgk_status moe_rows(const MoeArgs& a, pgk_dtype dt, hipStream_t st) {
    const RouterCfg& r = a.router;
    PGK_REQUIRE(a.n >= 1 && a.W % 64 == 0 && a.ff % 64 == 0 && r.E >= 1 && r.E <= MOE_MAX_EXPERTS && r.top >= 1 && r.top <= MOE_MAX_TOP && r.top <= r.E &&
                    (r.groups == 0 || (r.E % r.groups == 0 && r.keep >= 1 && r.keep <= r.groups && r.keep * (r.E / r.groups) >= r.top)),
                "moe: %d rows of %d, %d experts of %d, top %d, %d of %d groups", a.n, a.W, r.E, a.ff, r.top, r.keep, r.groups);
    PGK_REQUIRE((long long)a.n * r.top < (1LL << 30), "moe: %d rows x %d", a.n, r.top);
    const MoePlan p = moe_plan(a.n, a.W, a.ff, r, dt);
    char* ws = (char*)a.ws;
    float *logits = (float*)(ws + p.logits), *wts = (float*)(ws + p.wts);
    int32_t *ids = (int32_t*)(ws + p.ids), *order = (int32_t*)(ws + p.order), *count = (int32_t*)(ws + p.count);
    MoeTile* tiles = (MoeTile*)(ws + p.tiles);
    if (r.table) {
        PGK_REQUIRE(a.tok, "moe: a table of experts needs the rows' tokens");
        moe_table_kernel<<<ceil_div(p.total, 256), 256, 0, st>>>(r.table, a.tok, p.total, r.top, ids, wts);
    } else {
        if (dt == PGK_F32) { if (pgk_status q = pgk_gemm_nt(a.x, a.w_router, nullptr, logits, a.n, p.Ep, a.W, PGK_F32, st)) return q; }
        else if (a.n <= 128) { if (pgk_status q = wsgemm_nt((const bf16*)a.x, a.W, a.w_router, nullptr, false, logits, nullptr, 1, p.slabs, a.n, p.Ep, a.W, st)) return q; }
        else if (pgk_status q = gemm128s_bf16_nt((const bf16*)a.x, (const bf16*)a.w_router, nullptr, logits, 2, p.slabs, a.n, p.Ep, a.W, st, nullptr, false, nullptr)) return q;
        const size_t lds = (size_t)4 * route_floats(r) * 4;
        PGK_REQUIRE(lds <= 60 * 1024, "moe: %d experts", r.E);
        moe_route_kernel<<<ceil_div(a.n, 4), 256, lds, st>>>(r, logits, p.Ep, p.slabs, (size_t)a.n * p.Ep, a.n, ids, wts);
    }
    PGK_LAUNCH_CHECK();
    moe_sort_kernel<<<r.E, p.total > 2048 ? 1024 : 256, 0, st>>>(ids, p.total, r.E, p.tm, order, tiles, count);
    PGK_LAUNCH_CHECK();
    const GroupArgs up{tiles, count, order, wts, (long long)(a.gelu ? 1 : 2) * a.ff * a.W, r.top}, down{tiles, count, order, wts, (long long)a.ff * a.W, 0};
    const int tn_up = ceil_div(a.ff, 64), tn_down = ceil_div(a.W, 64);
    if (dt == PGK_F32) {
        const float *x = (const float*)a.x, *wu = (const float*)a.w_up;
        if (a.gelu) moe_f32_kernel<MOE_GELU><<<dim3(tn_up, p.max_tiles), 256, 0, st>>>(x, wu, (float*)(ws + p.act), a.ff, a.W, up);
        else moe_f32_kernel<MOE_SWIGLU><<<dim3(tn_up, p.max_tiles), 256, 0, st>>>(x, wu, (float*)(ws + p.act), a.ff, a.W, up);
        PGK_LAUNCH_CHECK();
        moe_f32_kernel<MOE_DOWN><<<dim3(tn_down, p.max_tiles), 256, 0, st>>>((const float*)(ws + p.act), (const float*)a.w_down, (float*)a.out, a.W, a.ff, down);
        PGK_LAUNCH_CHECK();
        return PGK_OK;
    }
    const bf16 *x = (const bf16*)a.x, *wu = (const bf16*)a.w_up, *wd = (const bf16*)a.w_down;
    bf16 *act = (bf16*)(ws + p.act), *out = (bf16*)a.out;
    if (p.tm == 128) {
        if (pgk_status q = gemm128s_grouped(x, wu, act, a.gelu ? MOE_GELU : MOE_SWIGLU, up, p.max_tiles, p.total, a.ff, a.W, st)) return q;
        return gemm128s_grouped(act, wd, out, MOE_DOWN, down, p.max_tiles, p.total, a.W, a.ff, st);
    }
    PGK_REQUIRE(p.max_tiles <= 65535, "moe: %d tiles", p.max_tiles);
    auto go = [&](auto mt) -> pgk_status {
        constexpr int MT = decltype(mt)::value;
        if (a.gelu) moe_stream_kernel<MT, MOE_GELU><<<dim3(tn_up, p.max_tiles), 256, 0, st>>>(x, wu, act, a.ff, a.W, up);
        else moe_stream_kernel<MT, MOE_SWIGLU><<<dim3(tn_up, p.max_tiles), 256, 0, st>>>(x, wu, act, a.ff, a.W, up);
        PGK_LAUNCH_CHECK();
        moe_stream_kernel<MT, MOE_DOWN><<<dim3(tn_down, p.max_tiles), 256, 0, st>>>(act, wd, out, a.W, a.ff, down);
        PGK_LAUNCH_CHECK();
        return PGK_OK;
    };
    return p.tm == 32 ? go(std::integral_constant<int, 2>{}) : go(std::integral_constant<int, 1>{});
}

template <class T>
__global__ __launch_bounds__(256) void moe_sum_kernel(const T* e, float* out, int W, int top) {
    const size_t row = blockIdx.x;
    for (int i = threadIdx.x; i < W; i += 256) {
        float s = 0.f;
        for (int k = 0; k < top; ++k) s += to_f(e[(row * top + k) * W + i]);
        out[row * W + i] = s;
    }
}

}  // namespace pgk

using namespace pgk;

// rows through `m` (out and ws are set here), summed over the chosen experts
static pgk_status moe_op(MoeArgs m, float* out, pgk_dtype dt, hipStream_t st) {
    const size_t rows = (((size_t)m.n * m.router.top * m.W * dtype_size(dt)) + 255) & ~(size_t)255;
    char* ws = nullptr;
    if (pgk_status q = pgk_malloc((void**)&ws, rows + moe_bytes(m.n, m.W, m.ff, m.router, dt))) return q;
    m.out = ws;
    m.ws = ws + rows;
    pgk_status q = moe_rows(m, dt, st);
    if (q == PGK_OK) {
        if (dt == PGK_F32) moe_sum_kernel<float><<<m.n, 256, 0, st>>>((const float*)ws, out, m.W, m.router.top);
        else moe_sum_kernel<bf16><<<m.n, 256, 0, st>>>((const bf16*)ws, out, m.W, m.router.top);
        if (hipError_t e = hipGetLastError()) q = set_error(PGK_ERR_HIP, "pgk_moe: %s", hipGetErrorString(e));
    }
    pgk_free(ws);       // stream-ordered reuse
    return q;
}

extern "C" {

pgk_status pgk_moe(const void* x, const void* router, const float* correction, const void* w_up, const void* w_down, float* out, int n, int width, int ff, int experts, int top, int groups,
                   int keep, float scale, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && router && correction && w_up && w_down && out && n >= 1 && top >= 1, "pgk_moe: null pointer or empty");
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_moe: dtype %d (bf16 or f32)", (int)dt);
    PGK_REQUIRE(width >= 64 && width % 64 == 0 && ff >= 64 && ff % 64 == 0 && experts >= 1, "pgk_moe: %d experts of %d x %d", experts, width, ff);
    const RouterCfg r{correction, experts, top, groups, keep, scale, nullptr};
    return moe_op(MoeArgs{x, n, width, ff, r, router, w_up, w_down, nullptr, nullptr}, out, dt, resolve_stream(s));
}

pgk_status pgk_table_moe(const void* x, const int32_t* table, const int32_t* tokens, const void* w_up, const void* w_down, float* out, int n, int width, int ff, int experts, int top,
                         pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(x && table && tokens && w_up && w_down && out && n >= 1 && top >= 1, "pgk_table_moe: null pointer or empty");
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_table_moe: dtype %d (bf16 or f32)", (int)dt);
    PGK_REQUIRE(width >= 64 && width % 64 == 0 && ff >= 64 && ff % 64 == 0 && experts >= 1, "pgk_table_moe: %d experts of %d x %d", experts, width, ff);
    return moe_op(MoeArgs{x, n, width, ff, RouterCfg{nullptr, experts, top, 0, 0, 1.0f, table}, nullptr, w_up, w_down, nullptr, nullptr, true, tokens}, out, dt, resolve_stream(s));
}

}  // extern "C"
