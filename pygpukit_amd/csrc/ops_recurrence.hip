// Linear recurrences (mixers.hip.h): per head a state S [dim][vdim] in fp32, S <- diag(f) S + k v^T, o = S^T q.
// Gates, decays, state and norms are fp32 whatever the element type.  SRC: where f, k, q, v come from (RECUR_HGRN2, RECUR_SSD).
//
// Two forms.  Token by token (decode, short portions): one workgroup per sequence and head walks its rows.  Chunked (prompts): rows in
// chunks of C, all chunks at once -
//   1. every chunk on its own:  U = sum_j (k_j prod_{t > j} f_t) v_j^T and D = prod_t f_t over its rows         (k = 1 - f)
//   2. along the chunks of a sequence:  S_c = S before chunk c,  S <- diag(D) S + U
//   3. every chunk:  o_i = S_c^T (q_i prod_{t <= i} f_t) + sum_{j <= i} A_ij v_j,  A_ij = sum_d q_i k_j prod_{j < t <= i} f_t
// Decays are products of f over rows, never quotients or differences of logarithms, so a gate near zero costs no accuracy and nothing
// overflows.  A is built in blocks of 16 rows: off the diagonal from factors that reach to a block's edge (q from the block's start, k to
// its block's end, whole blocks between), on the diagonal pair by pair.  All products are fp32 (v_mfma_f32_16x16x4_f32).

#include <type_traits>
#include <vector>

#include "mixers.hip.h"

namespace pgk {

// EXACT: the fp32 engines' form; otherwise the hardware's exponential and reciprocal (fp32, a few units in the last place)
template <bool EXACT> __device__ __forceinline__ float rc_exp(float z) { return EXACT ? expf(z) : __expf(z); }
template <bool EXACT> __device__ __forceinline__ float rc_recip(float z) { return EXACT ? 1.0f / z : __builtin_amdgcn_rcpf(z); }
template <bool EXACT> __device__ __forceinline__ float rc_silu(float z) { return z * rc_recip<EXACT>(1.0f + rc_exp<EXACT>(-z)); }

// forget gate and write strength: f = l + (1 - l) sigmoid(z), 1 - f = (1 - l) sigmoid(-z) (no cancellation near f = 1)
template <bool EXACT> __device__ __forceinline__ void rc_gate(float z, float lower, float& f, float& k) {
    const float e = rc_exp<EXACT>(-fabsf(z)), big = rc_recip<EXACT>(1.0f + e), small = e * big;
    f = fmaf(1.0f - lower, z >= 0.f ? big : small, lower);
    k = (1.0f - lower) * (z >= 0.f ? small : big);
}

// step size and decay of a state-space row (both forms: a scalar per head and row)
__device__ __forceinline__ void ssd_step(float dt, float bias, float decay, float& step, float& fade) {
    const float z = dt + bias;
    step = z > 20.f ? z : log1pf(expf(z));
    fade = expf(-decay * step);
}

// -------------------------------------------------------------------------------------------- token by token
// One workgroup per (sequence, head).  A thread owns VEC columns of every NG-th state row (VEC = 4: one 16-byte access each); a
// sequence that starts (position 0) begins with a zero state without reading the slot.
template <class T, class IT, bool EXACT, int VEC, int SRC>
__global__ __launch_bounds__(512) void recur_scan_kernel(unsigned long long* tl, RecurArgs a) {
    const TLStamp tls(tl);
    extern __shared__ float sm[];
    __shared__ float red[16];
    const int tid = threadIdx.x, NT = blockDim.x, h = blockIdx.x, dim = a.dim, vdim = a.vdim;
    const int NC = vdim / VEC, NG = max(NT / NC, 1), c = tid % NC, g = tid / NC;
    float *q = sm, *f = q + dim, *k = f + dim, *v = k + dim, *po = v + vdim;          // po [NG][vdim]
    SeqSpan s;
    if (a.seqs) s = a.seqs[blockIdx.y];
    else { s.row0 = blockIdx.y; s.len = 1; s.start = max(a.positions[blockIdx.y], 0); s.slot = blockIdx.y; }
    float* S = a.state + ((size_t)s.slot * a.H + h) * dim * vdim;
    for (int t = 0; t < s.len; ++t) {
        const IT* in = reinterpret_cast<const IT*>(a.in) + (size_t)(s.row0 + t) * a.ld_in;
        const bool fresh = s.start + t == 0;
        if constexpr (SRC == RECUR_SSD) {
            const int rep = a.H / a.G, grp = h / rep, pos = s.start + t;
            float step, fade;
            ssd_step(to_f(in[a.dt_off + h]), a.dt_bias[h], a.decay[h], step, fade);
            const T* row = reinterpret_cast<const T*>(a.rows) + (size_t)(s.row0 + t) * a.ld_rows;
            auto channel = [&](int c, bool own) { return a.seqs ? to_f(row[c]) : conv_step<T, IT, EXACT>(a.conv, in, c, s.slot, pos, own); };
            for (int i = tid; i < 2 * dim + vdim; i += NT) {
                if (i < dim) q[i] = channel(a.q_off + grp * dim + i, h % rep == 0);
                else if (i < 2 * dim) { k[i - dim] = step * channel(a.f_off + grp * dim + i - dim, h % rep == 0); f[i - dim] = fade; }
                else v[i - 2 * dim] = channel(a.v_off + h * vdim + i - 2 * dim, true);
            }
        } else {
        for (int d = tid; d < dim; d += NT) {
            const float zq = to_f(in[a.q_off + h * dim + d]), zf = to_f(in[a.f_off + h * dim + d]) + (a.bias ? a.bias[h * dim + d] : 0.f);
            q[d] = rc_silu<EXACT>(zq);
            rc_gate<EXACT>(zf, a.lower[h * dim + d], f[d], k[d]);
        }
        for (int i = tid; i < vdim; i += NT) v[i] = to_f(in[a.v_off + h * vdim + i]);
        }
        __syncthreads();
        if (g < NG) {
            for (int cc = c; cc < NC; cc += NT) {                  // (one trip unless a head has more columns than the workgroup threads)
                float acc[VEC], vv[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) { acc[e] = 0.f; vv[e] = v[cc * VEC + e]; }
                constexpr int U = 4;
                for (int d0 = g; d0 < dim; d0 += U * NG) {
                    float x[U][VEC];
#pragma unroll
                    for (int u = 0; u < U; ++u) {
                        const int d = min(d0 + u * NG, dim - 1);
                        if (fresh) {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) x[u][e] = 0.f;
                        } else if constexpr (VEC == 4) {
                            const float4 r = *reinterpret_cast<const float4*>(S + (size_t)d * vdim + cc * 4);
                            x[u][0] = r.x; x[u][1] = r.y; x[u][2] = r.z; x[u][3] = r.w;
                        } else x[u][0] = S[(size_t)d * vdim + cc];
                    }
#pragma unroll
                    for (int u = 0; u < U; ++u) {
                        const int d = d0 + u * NG;
                        if (d >= dim) break;
#pragma unroll
                        for (int e = 0; e < VEC; ++e) {
                            x[u][e] = fmaf(f[d], x[u][e], k[d] * vv[e]);
                            acc[e] = fmaf(q[d], x[u][e], acc[e]);
                        }
                        if constexpr (VEC == 4) *reinterpret_cast<float4*>(S + (size_t)d * vdim + cc * 4) = make_float4(x[u][0], x[u][1], x[u][2], x[u][3]);
                        else S[(size_t)d * vdim + cc] = x[u][0];
                    }
                }
#pragma unroll
                for (int e = 0; e < VEC; ++e) po[g * vdim + cc * VEC + e] = acc[e];
            }
        }
        __syncthreads();
        float ss = 0.f;
        for (int i = tid; i < vdim; i += NT) {
            float o = 0.f;
            for (int j = 0; j < NG; ++j) o += po[j * vdim + i];
            if constexpr (SRC == RECUR_SSD) o = fmaf(a.skip[h], v[i], o) * silu_f<EXACT>(to_f(in[a.z_off + h * vdim + i]));
            v[i] = o;                                              // the column's own thread: read again below
            ss = fmaf(o, o, ss);
        }
        float inv = 1.f;
        if (a.norm) inv = 1.0f / sqrtf(block_sum(ss, red) / a.vdim_true + a.eps);
        IT* out = reinterpret_cast<IT*>(a.out) + (size_t)(s.row0 + t) * a.ld_out;
        for (int i = tid; i < vdim; i += NT) out[h * vdim + i] = from_f<IT>(v[i] * inv * (a.norm ? a.norm[i] : 1.f));
        if (h == a.H - 1)
            for (int i = a.H * vdim + tid; i < a.ld_out; i += NT) out[i] = from_f<IT>(0.f);
        __syncthreads();                                           // q, f, k, v and po are rewritten by the next token
    }
    tls.end();
}

template <class T, class IT, bool EXACT, int SRC>
static pgk_status recur_scan(const RecurArgs& a, hipStream_t st) {
    const int B = a.seqs ? a.n_seqs : a.n, threads = a.dim * a.vdim >= 8192 ? 512 : 256;
    const bool vec = a.vdim % 4 == 0;
    const int cols = vec ? a.vdim / 4 : a.vdim, groups = threads / cols > 0 ? threads / cols : 1;
    const size_t lds = (size_t)(3 * a.dim + a.vdim + groups * a.vdim) * 4;
    PGK_REQUIRE(lds <= 64 * 1024, "recurrence: head widths %d / %d do not fit LDS", a.dim, a.vdim);
    if (vec) PGK_CHECK_HIP(launch_k(&recur_scan_kernel<T, IT, EXACT, 4, SRC>, dim3(a.H, B), dim3(threads), lds, st, a));
    else PGK_CHECK_HIP(launch_k(&recur_scan_kernel<T, IT, EXACT, 1, SRC>, dim3(a.H, B), dim3(threads), lds, st, a));
    return PGK_OK;
}

pgk_status recur_rows(const RecurArgs& a, pgk_dtype dt, bool io32, hipStream_t st) {
    PGK_REQUIRE(a.H >= 1 && a.dim >= 1 && a.vdim >= 1 && a.ld_out >= a.H * a.vdim && (a.seqs || a.positions), "recurrence: bad sizes");
    if (a.kind == RECUR_SSD) {
        PGK_REQUIRE(a.G >= 1 && a.H % a.G == 0 && (a.seqs ? a.rows != nullptr : a.conv.taps >= 1 && a.conv.ring), "recurrence: bad state-space arguments");
        if (dt == PGK_F32) return recur_scan<float, float, true, RECUR_SSD>(a, st);
        return io32 ? recur_scan<bf16, float, false, RECUR_SSD>(a, st) : recur_scan<bf16, bf16, false, RECUR_SSD>(a, st);
    }
    if (dt == PGK_F32) return recur_scan<float, float, true, RECUR_HGRN2>(a, st);
    return io32 ? recur_scan<bf16, float, false, RECUR_HGRN2>(a, st) : recur_scan<bf16, bf16, false, RECUR_HGRN2>(a, st);
}

// -------------------------------------------------------------------------------------------- chunks
typedef float f32x4_rc __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4_rc mfma4(float a, float b, f32x4_rc c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
// Four products in a row take k in the order 4 (lane >> 4) + step instead of 4 step + (lane >> 4), where both operands can: a lane's four
// values of a row are then neighbours, one 16-byte access.
__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 mul4(const float4& a, const float4& b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }

// LDS row strides (floats; widths are multiples of 16).  Operands whose k index runs over rows want 16 x odd, those whose k index runs
// along a row want 4 x odd: the 64 lanes of a load then fall on 64 banks.
__host__ __device__ constexpr int rc_col_stride(int w) { return (w / 16) % 2 ? w : w + 16; }
__host__ __device__ constexpr int rc_row_stride(int w) { return w + 4; }

static size_t rc_state_lds(int C, int dim, int vdim) { return ((size_t)C * (rc_col_stride(dim) + rc_col_stride(vdim)) + (C / 16) * dim + 2 * C) * 4; }
static size_t rc_out_lds(int C, int dim) { return ((size_t)3 * C * rc_row_stride(dim) + C * rc_row_stride(C) + (C / 16) * dim + 10 * C) * 4; }
constexpr size_t RC_LDS_MAX = 156 * 1024;

int recur_chunk_rows(int dim, int vdim) {
    if (dim % 16 || vdim % 16 || vdim > 512) return 0;
    for (int C = 64; C >= 32; C /= 2)
        if (rc_state_lds(C, dim, vdim) <= RC_LDS_MAX && rc_out_lds(C, dim) <= RC_LDS_MAX) return C;
    return 0;
}
size_t recur_chunk_bytes(const RecurArgs& a, int n_chunks) { return (size_t)n_chunks * a.H * ((size_t)a.dim * a.vdim + a.dim) * 4; }

// 1: U [chunk][head][dim][vdim], D [chunk][head][dim].  Eight waves; VT column tiles of 16 at a time (vdim is a multiple of 16 VT).
template <class T, int C, int VT, int SRC>
__global__ __launch_bounds__(512) void recur_chunk_state_kernel(RecurArgs a, const RecurChunk* chunks, float* U, float* D) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    constexpr int NS = C / 16, VB = 4;
    constexpr bool EXACT = std::is_same<T, float>::value;
    const int dim = a.dim, vdim = a.vdim, ks = rc_col_stride(dim), vs = rc_col_stride(vdim), h = blockIdx.x;
    float *kr = sm, *v = kr + C * ks, *F = v + C * vs, *step = F + NS * dim, *fade = step + C;
    const RecurChunk ch = chunks[blockIdx.y];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4, last = ch.len - 1;
    const T* in = reinterpret_cast<const T*>(a.in) + (size_t)ch.row0 * a.ld_in;
    const int ld = SRC == RECUR_SSD ? a.ld_rows : a.ld_in, kh = SRC == RECUR_SSD ? h / (a.H / a.G) : h;
    const T* ch_in = SRC == RECUR_SSD ? reinterpret_cast<const T*>(a.rows) + (size_t)ch.row0 * ld : in;
    const T* vin = ch_in + a.v_off + h * vdim;
    if constexpr (SRC == RECUR_SSD) {
        if (tid < C) ssd_step(to_f(in[(size_t)min(tid, last) * a.ld_in + a.dt_off + h]), a.dt_bias[h], a.decay[h], step[tid], fade[tid]);
        __syncthreads();
    }
    const int nv = C * vdim / 4, v4 = vdim / 4;
    // k times the decay to the end of its block of 16 rows, and the blocks' decays; the first values travel with the first gates
    float4 vv[VB];
    for (int t = tid, t0 = 0; t < NS * dim || t0 == 0; t += 512, t0 = 1) {
        const int b = min(t / dim, NS - 1), d = t % dim;
        const T* z = ch_in + a.f_off + kh * dim + d;
        float zf[16];
#pragma unroll
        for (int r = 0; r < 16; ++r) zf[r] = to_f(z[(size_t)min(16 * b + r, last) * ld]);
        float bias = 0.f, low = 0.f;
        if constexpr (SRC == RECUR_HGRN2) { bias = a.bias ? a.bias[h * dim + d] : 0.f; low = a.lower[h * dim + d]; }
        if (t0 == 0) {
#pragma unroll
            for (int i = 0; i < VB; ++i) { const int e = min(tid + 512 * i, nv - 1); vv[i] = load4<T>(vin + (size_t)min(e / v4, last) * ld + e % v4 * 4); }
        }
        float run = 1.f;
#pragma unroll
        for (int r = 15; r >= 0; --r) {
            float f, k;
            if constexpr (SRC == RECUR_SSD) { f = fade[16 * b + r]; k = step[16 * b + r] * zf[r]; }
            else rc_gate<EXACT>(zf[r] + bias, low, f, k);
            const bool live = 16 * b + r <= last;
            if (t < NS * dim) kr[(16 * b + r) * ks + d] = live ? k * run : 0.f;
            run *= live ? f : 1.f;
        }
        if (t < NS * dim) F[b * dim + d] = run;
    }
#pragma unroll
    for (int i = 0; i < VB; ++i) { const int e = tid + 512 * i; if (e < nv) *reinterpret_cast<float4*>(v + e / v4 * vs + e % v4 * 4) = vv[i]; }
    for (int e = tid + 512 * VB; e < nv; e += 512) *reinterpret_cast<float4*>(v + e / v4 * vs + e % v4 * 4) = load4<T>(vin + (size_t)min(e / v4, last) * ld + e % v4 * 4);
    __syncthreads();
    const size_t rec = (size_t)blockIdx.y * a.H + h;
    for (int d = tid; d < dim; d += 512) {
        float run = 1.f;
#pragma unroll
        for (int b = 0; b < NS; ++b) run *= F[b * dim + d];
        D[rec * dim + d] = run;
    }
    float* u = U + rec * dim * vdim;
    for (int dt = wid; dt < dim / 16; dt += 8) {
        float x[NS][4], m = 1.f;                                   // k times the decay to the chunk's end
#pragma unroll
        for (int b = NS - 1; b >= 0; --b) {
#pragma unroll
            for (int s = 0; s < 4; ++s) x[b][s] = kr[(16 * b + 4 * s + q4) * ks + 16 * dt + l15] * m;
            m *= F[b * dim + 16 * dt + l15];
        }
        for (int v0 = 0; v0 < vdim; v0 += 16 * VT) {
            f32x4_rc acc[VT];
#pragma unroll
            for (int t = 0; t < VT; ++t) acc[t] = f32x4_rc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int b = 0; b < NS; ++b)
#pragma unroll
                for (int s = 0; s < 4; ++s) {
                    const float* vr = v + (16 * b + 4 * s + q4) * vs + v0 + l15;
#pragma unroll
                    for (int t = 0; t < VT; ++t) acc[t] = mfma4(x[b][s], vr[16 * t], acc[t]);
                }
#pragma unroll
            for (int t = 0; t < VT; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) u[(size_t)(16 * dt + 4 * q4 + r) * vdim + v0 + 16 * t + l15] = acc[t][r];
        }
    }
}

// 2: U becomes the state before each chunk, the slot's state moves on
__global__ __launch_bounds__(256) void recur_chunk_scan_kernel(RecurArgs a, const int32_t* chunk_of_seq, float* U, const float* D) {
    const int h = blockIdx.y, n4 = a.dim * a.vdim / 4, i = blockIdx.x * 256 + threadIdx.x;
    if (i >= n4) return;
    const SeqSpan s = a.seqs[blockIdx.z];
    const int c0 = chunk_of_seq[blockIdx.z], c1 = chunk_of_seq[blockIdx.z + 1], d = 4 * i / a.vdim;
    float4* st = reinterpret_cast<float4*>(a.state + ((size_t)s.slot * a.H + h) * a.dim * a.vdim) + i;
    float4 S = s.start > 0 ? *st : make_float4(0.f, 0.f, 0.f, 0.f);
    auto at = [&](int c) { return reinterpret_cast<float4*>(U + ((size_t)c * a.H + h) * a.dim * a.vdim) + i; };
    constexpr int P = 8;                                           // chunks in flight
    for (int c = c0; c < c1; c += P) {
        float4 u[P];
        float w[P];
#pragma unroll
        for (int k = 0; k < P; ++k) {
            const int cc = min(c + k, c1 - 1);
            u[k] = *at(cc);
            w[k] = D[((size_t)cc * a.H + h) * a.dim + d];
        }
#pragma unroll
        for (int k = 0; k < P; ++k) {
            if (c + k >= c1) break;
            *at(c + k) = S;
            S.x = fmaf(w[k], S.x, u[k].x); S.y = fmaf(w[k], S.y, u[k].y); S.z = fmaf(w[k], S.z, u[k].z); S.w = fmaf(w[k], S.w, u[k].w);
        }
    }
    *st = S;
}

// 3: output rows.  Eight waves; NVT column tiles of 16 per wave.  The values and the first rows of the state travel while the gates and
// the decays are worked out.
template <class T, int C, int NVT, int SRC>
__global__ __launch_bounds__(512) void recur_chunk_out_kernel(RecurArgs a, const RecurChunk* chunks, const float* U) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    constexpr int NS = C / 16, AS = rc_row_stride(C);
    constexpr bool EXACT = std::is_same<T, float>::value;
    const int dim = a.dim, vdim = a.vdim, S = rc_row_stride(dim), h = blockIdx.x;
    float *q = sm, *f = q + C * S, *k = f + C * S, *A = k + C * S, *F = A + C * AS, *red = F + NS * dim, *step = red + 8 * C, *fade = step + C;
    const RecurChunk ch = chunks[blockIdx.y];
    const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, l15 = lane & 15, q4 = lane >> 4;
    const T* in = reinterpret_cast<const T*>(a.in) + (size_t)ch.row0 * a.ld_in;
    const int nz = C * dim / 4, d4 = dim / 4, last = ch.len - 1;
    const int ld = SRC == RECUR_SSD ? a.ld_rows : a.ld_in, kh = SRC == RECUR_SSD ? h / (a.H / a.G) : h;
    const T* ch_in = SRC == RECUR_SSD ? reinterpret_cast<const T*>(a.rows) + (size_t)ch.row0 * ld : in;
    const float* st = U + ((size_t)blockIdx.y * a.H + h) * dim * vdim;
    constexpr int ZB = 4, PRE = 8 / NVT;                           // pieces of the rows requested first; blocks of 16 state rows requested ahead
    float4 pq[ZB], pf[ZB];
#pragma unroll
    for (int i = 0; i < ZB; ++i) {
        const int t = min(tid + 512 * i, nz - 1);
        const T* row = ch_in + (size_t)min(t / d4, last) * ld + kh * dim + t % d4 * 4;
        pq[i] = load4<T>(row + a.q_off);
        pf[i] = load4<T>(row + a.f_off);
    }
    int col[NVT];                                                  // this lane's column of each tile (tiles beyond the last repeat it)
#pragma unroll
    for (int t = 0; t < NVT; ++t) col[t] = min(16 * (wid + 8 * t), vdim - 16) + l15;
    float pv[NVT][NS][4], ps[NVT][PRE][4];
    const T* v = ch_in + a.v_off + h * vdim;
#pragma unroll
    for (int t = 0; t < NVT; ++t) {
#pragma unroll
        for (int b = 0; b < NS; ++b)
#pragma unroll
            for (int u = 0; u < 4; ++u) pv[t][b][u] = to_f(v[(size_t)min(16 * b + 4 * q4 + u, last) * ld + col[t]]);
#pragma unroll
        for (int b = 0; b < PRE; ++b)
#pragma unroll
            for (int u = 0; u < 4; ++u) ps[t][b][u] = st[(size_t)min(16 * b + 4 * q4 + u, dim - 1) * vdim + col[t]];
    }
    if constexpr (SRC == RECUR_SSD) {
        if (tid < C) ssd_step(to_f(in[(size_t)min(tid, last) * a.ld_in + a.dt_off + h]), a.dt_bias[h], a.decay[h], step[tid], fade[tid]);
        __syncthreads();
    }
    auto gates = [&](int t, const float4& zq, const float4& zf) {
        const int r = t / d4, c = t % d4 * 4;
        if constexpr (SRC == RECUR_SSD) {
            const bool live = r < ch.len;
            const float fr = live ? fade[r] : 1.f, sr = live ? step[r] : 0.f;
            *reinterpret_cast<float4*>(q + r * S + c) = live ? zq : make_float4(0.f, 0.f, 0.f, 0.f);
            *reinterpret_cast<float4*>(f + r * S + c) = make_float4(fr, fr, fr, fr);
            *reinterpret_cast<float4*>(k + r * S + c) = make_float4(sr * zf.x, sr * zf.y, sr * zf.z, sr * zf.w);
            return;
        }
        const float4 b = a.bias ? *reinterpret_cast<const float4*>(a.bias + h * dim + c) : make_float4(0.f, 0.f, 0.f, 0.f);
        const float4 low = *reinterpret_cast<const float4*>(a.lower + h * dim + c);
        float4 qq = {rc_silu<EXACT>(zq.x), rc_silu<EXACT>(zq.y), rc_silu<EXACT>(zq.z), rc_silu<EXACT>(zq.w)}, ff, kk;
        rc_gate<EXACT>(zf.x + b.x, low.x, ff.x, kk.x); rc_gate<EXACT>(zf.y + b.y, low.y, ff.y, kk.y);
        rc_gate<EXACT>(zf.z + b.z, low.z, ff.z, kk.z); rc_gate<EXACT>(zf.w + b.w, low.w, ff.w, kk.w);
        if (r >= ch.len) { qq = kk = make_float4(0.f, 0.f, 0.f, 0.f); ff = make_float4(1.f, 1.f, 1.f, 1.f); }
        *reinterpret_cast<float4*>(q + r * S + c) = qq;
        *reinterpret_cast<float4*>(f + r * S + c) = ff;
        *reinterpret_cast<float4*>(k + r * S + c) = kk;
    };
#pragma unroll
    for (int i = 0; i < ZB; ++i) if (tid + 512 * i < nz) gates(tid + 512 * i, pq[i], pf[i]);
    for (int t = tid + 512 * ZB; t < nz; t += 512) {
        const T* row = ch_in + (size_t)min(t / d4, last) * ld + kh * dim + t % d4 * 4;
        gates(t, load4<T>(row + a.q_off), load4<T>(row + a.f_off));
    }
    __syncthreads();
    // diagonal blocks, pair by pair: two waves per block, rows 0..7 and 8..15.  Lane: column j = lane & 7 (and j + 8), every eighth
    // group of 8 channels; w = k_j times the decay from j to the row at hand.
    if ((wid >> 1) < NS) {
        // (waves w and w + 4 share a SIMD: one of them takes the shorter half)
        const int r0 = 16 * (wid >> 1), half = (wid ^ (wid >> 2)) & 1, jl = lane & 7, dg = lane >> 3;
        float lo[8], hi[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) lo[i] = hi[i] = 0.f;
        for (int c = 8 * dg; c < dim; c += 64) {
            float wl[8], wh[8];
            auto row8 = [&](const float* p, float (&x)[8]) {
                const float4 u = *reinterpret_cast<const float4*>(p), v = *reinterpret_cast<const float4*>(p + 4);
                x[0] = u.x; x[1] = u.y; x[2] = u.z; x[3] = u.w; x[4] = v.x; x[5] = v.y; x[6] = v.z; x[7] = v.w;
            };
            row8(k + (r0 + jl) * S + c, wl);
            if (half) {
                row8(k + (r0 + 8 + jl) * S + c, wh);
#pragma unroll
                for (int i = 1; i < 8; ++i) {
                    float g[8];
                    row8(f + (r0 + i) * S + c, g);
#pragma unroll
                    for (int e = 0; e < 8; ++e) wl[e] *= i > jl ? g[e] : 1.f;
                }
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                float g[8], x[8];
                const int row = r0 + 8 * half + i;
                row8(f + row * S + c, g);
                row8(q + row * S + c, x);
                if (half) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        wl[e] *= g[e];
                        lo[i] = fmaf(x[e], wl[e], lo[i]);
                        wh[e] *= i > jl ? g[e] : 1.f;
                        hi[i] = fmaf(x[e], wh[e], hi[i]);
                    }
                } else {
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        wl[e] *= i > jl ? g[e] : 1.f;
                        lo[i] = fmaf(x[e], wl[e], lo[i]);
                    }
                }
            }
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            float x = lo[i], y = hi[i];
            x += dpp_f<DPP_ROR8>(x); x += __shfl_xor(x, 16, 64); x += __shfl_xor(x, 32, 64);
            y += dpp_f<DPP_ROR8>(y); y += __shfl_xor(y, 16, 64); y += __shfl_xor(y, 32, 64);
            float* row = A + (r0 + 8 * half + i) * AS + r0;
            if (dg == 0) {
                row[jl] = half || i >= jl ? x : 0.f;
                row[8 + jl] = half && i >= jl ? y : 0.f;
            }
        }
    }
    __syncthreads();
    // q times the decay from its block's start (its own row included), k times the decay to its block's end
    for (int t = tid; t < NS * dim; t += 512) {
        const int b = t / dim, d = t % dim;
        float g[16], run = 1.f;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            g[r] = f[(16 * b + r) * S + d];
            run *= g[r];
            q[(16 * b + r) * S + d] *= run;
        }
        F[b * dim + d] = run;
        run = 1.f;
#pragma unroll
        for (int r = 15; r >= 0; --r) {
            k[(16 * b + r) * S + d] *= run;
            run *= g[r];
        }
    }
    __syncthreads();
    // blocks below the diagonal
    for (int p = wid; p < NS * (NS - 1) / 2; p += 8) {
        int bi = 1, bj = p;
        while (bj >= bi) { bj -= bi; ++bi; }
        f32x4_rc acc[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) acc[u] = f32x4_rc{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int d0 = 0; d0 < dim; d0 += 16) {
            const int d = d0 + 4 * q4;
            float4 x = ld4(q + (16 * bi + l15) * S + d);
            const float4 y = ld4(k + (16 * bj + l15) * S + d);
            if (bj + 1 < bi) x = mul4(x, ld4(F + (bj + 1) * dim + d));
            if (bj + 2 < bi) x = mul4(x, ld4(F + (bj + 2) * dim + d));        // (NS <= 4: at most two blocks between)
            acc[0] = mfma4(x.x, y.x, acc[0]); acc[1] = mfma4(x.y, y.y, acc[1]);
            acc[2] = mfma4(x.z, y.z, acc[2]); acc[3] = mfma4(x.w, y.w, acc[3]);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) A[(16 * bi + 4 * q4 + r) * AS + 16 * bj + l15] = (acc[0][r] + acc[1][r]) + (acc[2][r] + acc[3][r]);
    }
    __syncthreads();
    // o = q S + A v: a wave has every row of its column tiles
    f32x4_rc o[NVT][NS];
#pragma unroll
    for (int t = 0; t < NVT; ++t)
#pragma unroll
        for (int b = 0; b < NS; ++b) o[t][b] = f32x4_rc{0.f, 0.f, 0.f, 0.f};
    auto rows16 = [&](int d0, const float (&x)[NVT][4]) {          // 16 state rows
        const int d = d0 + 4 * q4;
        float4 y[NS], m = ld4(F + d);
#pragma unroll
        for (int b = 0; b < NS; ++b) {
            y[b] = ld4(q + (16 * b + l15) * S + d);
            if (b > 0) y[b] = mul4(y[b], m);
            if (b > 0 && b + 1 < NS) m = mul4(m, ld4(F + b * dim + d));
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int b = 0; b < NS; ++b)
#pragma unroll
                for (int t = 0; t < NVT; ++t) o[t][b] = mfma4(u == 0 ? y[b].x : u == 1 ? y[b].y : u == 2 ? y[b].z : y[b].w, x[t][u], o[t][b]);
    };
#pragma unroll
    for (int i = 0; i < PRE; ++i)
        if (16 * i < dim) {                                        // uniform
            float x[NVT][4];
#pragma unroll
            for (int t = 0; t < NVT; ++t)
#pragma unroll
                for (int u = 0; u < 4; ++u) x[t][u] = ps[t][i][u];
            rows16(16 * i, x);
        }
    for (int d0 = 16 * PRE; d0 < dim; d0 += 16) {
        float x[NVT][4];
#pragma unroll
        for (int t = 0; t < NVT; ++t)
#pragma unroll
            for (int u = 0; u < 4; ++u) x[t][u] = st[(size_t)(d0 + 4 * q4 + u) * vdim + col[t]];
        rows16(d0, x);
    }
#pragma unroll
    for (int bj = 0; bj < NS; ++bj)
#pragma unroll
        for (int b = bj; b < NS; ++b) {
            const float4 y = ld4(A + (16 * b + l15) * AS + 16 * bj + 4 * q4);
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int t = 0; t < NVT; ++t) o[t][b] = mfma4(u == 0 ? y.x : u == 1 ? y.y : u == 2 ? y.z : y.w, pv[t][bj][u], o[t][b]);
        }
    // lane: rows 16 b + 4 q4 + r, column l15 of each tile
    if constexpr (SRC == RECUR_SSD) {
        const float skip = a.skip[h];
#pragma unroll
        for (int t = 0; t < NVT; ++t)
#pragma unroll
            for (int b = 0; b < NS; ++b)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[t][b][r] = fmaf(skip, pv[t][b][r], o[t][b][r]);
    }
    float inv[NS][4];
#pragma unroll
    for (int b = 0; b < NS; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float ss = 0.f;
#pragma unroll
            for (int t = 0; t < NVT; ++t) ss += 16 * (wid + 8 * t) < vdim ? o[t][b][r] * o[t][b][r] : 0.f;
            ss = group16_sum(ss);
            if (l15 == 0) red[wid * C + 16 * b + 4 * q4 + r] = ss;
        }
    __syncthreads();
    if (tid < C) {
        float ss = 0.f;
#pragma unroll
        for (int w = 0; w < 8; ++w) ss += red[w * C + tid];
        A[tid] = a.norm ? 1.0f / sqrtf(ss / a.vdim_true + a.eps) : 1.0f;      // (A has been read)
    }
    __syncthreads();
#pragma unroll
    for (int b = 0; b < NS; ++b) {
        const float4 t = ld4(A + 16 * b + 4 * q4);
        inv[b][0] = t.x; inv[b][1] = t.y; inv[b][2] = t.z; inv[b][3] = t.w;
    }
    T* out = reinterpret_cast<T*>(a.out) + (size_t)ch.row0 * a.ld_out;
    const int ys = rc_row_stride(vdim);
    const bool staged = ys <= 3 * S;                               // the rows leave through the space of q, f and k (no longer read), whole pieces at a time
#pragma unroll
    for (int t = 0; t < NVT; ++t) {
        const int c = 16 * (wid + 8 * t) + l15;
        if (16 * (wid + 8 * t) >= vdim) break;                     // wave-uniform
        const float g = a.norm ? a.norm[c] : 1.f;
#pragma unroll
        for (int b = 0; b < NS; ++b)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = 16 * b + 4 * q4 + r;
                const float y = o[t][b][r] * inv[b][r] * g;
                if (staged) q[row * ys + c] = y;
                else if (row < ch.len) {
                    float w = y;
                    if constexpr (SRC == RECUR_SSD) w *= silu_f<EXACT>(to_f(in[(size_t)row * a.ld_in + a.z_off + h * vdim + c]));
                    out[(size_t)row * a.ld_out + h * vdim + c] = from_f<T>(w);
                }
            }
    }
    if (staged) {
        __syncthreads();
        for (int t = tid; t < ch.len * (vdim / 4); t += 512) {
            const int r = t / (vdim / 4), c = t % (vdim / 4) * 4;
            float4 y = ld4(q + r * ys + c);
            if constexpr (SRC == RECUR_SSD) {
                const float4 z = load4<T>(in + (size_t)r * a.ld_in + a.z_off + h * vdim + c);
                y = mul4(y, make_float4(silu_f<EXACT>(z.x), silu_f<EXACT>(z.y), silu_f<EXACT>(z.z), silu_f<EXACT>(z.w)));
            }
            store4<T>(out + (size_t)r * a.ld_out + h * vdim + c, y);
        }
    }
    if (h == a.H - 1 && a.ld_out > a.H * vdim) {
        const int tail = a.ld_out - a.H * vdim;
        for (int t = tid; t < ch.len * tail; t += 512) out[(size_t)(t / tail) * a.ld_out + a.H * vdim + t % tail] = from_f<T>(0.f);
    }
}

template <class K>
static hipError_t rc_allow_lds(K kfn, size_t lds, bool& done) {
    if (lds <= 48 * 1024 || done) return hipSuccess;
    done = true;
    return hipFuncSetAttribute(reinterpret_cast<const void*>(kfn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)RC_LDS_MAX);
}

template <class T, int C, int NVT, int SRC>
static hipError_t launch_chunk_out(const RecurArgs& a, const RecurChunk* chunks, int n_chunks, const float* U, hipStream_t st) {
    static bool done = false;
    const size_t lds = rc_out_lds(C, a.dim);
    if (hipError_t e = rc_allow_lds(&recur_chunk_out_kernel<T, C, NVT, SRC>, lds, done)) return e;
    recur_chunk_out_kernel<T, C, NVT, SRC><<<dim3(a.H, n_chunks), 512, lds, st>>>(a, chunks, U);
    return hipGetLastError();
}

template <class T, int C, int VT, int SRC>
static hipError_t launch_chunk_state(const RecurArgs& a, const RecurChunk* chunks, int n_chunks, float* U, float* D, hipStream_t st) {
    static bool done = false;
    const size_t lds = rc_state_lds(C, a.dim, a.vdim);
    if (hipError_t e = rc_allow_lds(&recur_chunk_state_kernel<T, C, VT, SRC>, lds, done)) return e;
    recur_chunk_state_kernel<T, C, VT, SRC><<<dim3(a.H, n_chunks), 512, lds, st>>>(a, chunks, U, D);
    return hipGetLastError();
}

template <class T, int C, int SRC>
static pgk_status recur_chunked_t(const RecurArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, void* ws, hipStream_t st) {
    float *U = (float*)ws, *D = U + (size_t)n_chunks * a.H * a.dim * a.vdim;
    if (a.vdim % 128 == 0) PGK_CHECK_HIP((launch_chunk_state<T, C, 8, SRC>(a, chunks, n_chunks, U, D, st)));
    else if (a.vdim % 64 == 0) PGK_CHECK_HIP((launch_chunk_state<T, C, 4, SRC>(a, chunks, n_chunks, U, D, st)));
    else PGK_CHECK_HIP((launch_chunk_state<T, C, 1, SRC>(a, chunks, n_chunks, U, D, st)));
    recur_chunk_scan_kernel<<<dim3(ceil_div(a.dim * a.vdim / 4, 256), a.H, a.n_seqs), 256, 0, st>>>(a, chunk_of_seq, U, D);
    PGK_LAUNCH_CHECK();
    if (a.vdim <= 128) PGK_CHECK_HIP((launch_chunk_out<T, C, 1, SRC>(a, chunks, n_chunks, U, st)));
    else if (a.vdim <= 256) PGK_CHECK_HIP((launch_chunk_out<T, C, 2, SRC>(a, chunks, n_chunks, U, st)));
    else PGK_CHECK_HIP((launch_chunk_out<T, C, 4, SRC>(a, chunks, n_chunks, U, st)));
    return PGK_OK;
}

pgk_status recur_chunked(const RecurArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, void* ws, pgk_dtype dt, hipStream_t st) {
    const int C = recur_chunk_rows(a.dim, a.vdim);
    PGK_REQUIRE(C && a.seqs && chunks && n_chunks >= 1 && n_chunks <= 65535 && a.H * a.vdim <= a.ld_out && a.ld_in % 4 == 0 && a.q_off % 4 == 0 && a.f_off % 4 == 0 && a.v_off % 4 == 0,
                "recurrence: %d chunks of head widths %d / %d", n_chunks, a.dim, a.vdim);
    PGK_REQUIRE(a.kind != RECUR_SSD || (a.rows && a.ld_rows % 4 == 0 && a.z_off % 4 == 0 && a.G >= 1 && a.H % a.G == 0), "recurrence: bad state-space arguments");
    auto go = [&](auto src) -> pgk_status {
        constexpr int SRC = decltype(src)::value;
        if (dt == PGK_F32) return C == 64 ? recur_chunked_t<float, 64, SRC>(a, chunks, n_chunks, chunk_of_seq, ws, st) : recur_chunked_t<float, 32, SRC>(a, chunks, n_chunks, chunk_of_seq, ws, st);
        return C == 64 ? recur_chunked_t<bf16, 64, SRC>(a, chunks, n_chunks, chunk_of_seq, ws, st) : recur_chunked_t<bf16, 32, SRC>(a, chunks, n_chunks, chunk_of_seq, ws, st);
    };
    return a.kind == RECUR_SSD ? go(std::integral_constant<int, RECUR_SSD>{}) : go(std::integral_constant<int, RECUR_HGRN2>{});
}

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_gated_recurrence(const void* q, const void* f, const void* v, const float* f_bias, const float* lower, const float* norm, float* state, void* out, int n,
                                int fresh, int heads, int dim, int vdim, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(q && f && v && lower && state && out, "pgk_gated_recurrence: null pointer");
    PGK_REQUIRE(n >= 1 && heads >= 1 && dim >= 1 && vdim >= 1, "pgk_gated_recurrence: bad shape %d x %d x %d, %d rows", heads, dim, vdim, n);
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_gated_recurrence: dtype %d (bf16 or f32)", (int)dt);
    hipStream_t st = resolve_stream(s);
    // one row buffer q | f | v, the tables and the chunked form's workspace behind it
    const size_t E = dtype_size(dt), row = (size_t)heads * (2 * dim + vdim);
    auto up = [](size_t b) { return (b + 255) & ~(size_t)255; };
    RecurArgs a{};
    a.ld_in = (int)row; a.f_off = heads * dim; a.v_off = 2 * heads * dim;
    a.bias = f_bias; a.lower = lower; a.norm = norm; a.H = heads; a.dim = dim; a.vdim = a.vdim_true = vdim; a.n = n; a.eps = eps;
    a.state = state; a.n_seqs = 1; a.out = out; a.ld_out = heads * vdim;
    const int C = n >= RECUR_CHUNKED_FROM ? recur_chunk_rows(dim, vdim) : 0, nch = C ? ceil_div(n, C) : 0;
    std::vector<RecurChunk> chunks;
    for (int c = 0; c < nch; ++c) chunks.push_back(RecurChunk{c * C, n - c * C < C ? n - c * C : C});
    const int32_t of_seq[2] = {0, nch};
    const SeqSpan span{0, n, fresh ? 0 : 1, 0};
    const size_t o_span = up((size_t)n * row * E), o_of = o_span + up(sizeof(span)), o_ch = o_of + up(sizeof(of_seq)), o_ws = o_ch + up(nch * sizeof(RecurChunk));
    char* ws = nullptr;
    if (pgk_status r = pgk_malloc((void**)&ws, o_ws + (nch ? recur_chunk_bytes(a, nch) : 0) + 256)) return r;
    const size_t wq = (size_t)heads * dim * E, wv = (size_t)heads * vdim * E;
    hipError_t e = hipMemcpy2DAsync(ws, row * E, q, wq, wq, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpy2DAsync(ws + wq, row * E, f, wq, wq, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpy2DAsync(ws + 2 * wq, row * E, v, wv, wv, n, hipMemcpyDeviceToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_span, &span, sizeof(span), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_of, of_seq, sizeof(of_seq), hipMemcpyHostToDevice, st);
    if (e == hipSuccess && nch) e = hipMemcpyAsync(ws + o_ch, chunks.data(), nch * sizeof(RecurChunk), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    a.in = ws; a.seqs = (const SeqSpan*)(ws + o_span);
    pgk_status r;
    if (e != hipSuccess) r = set_error(PGK_ERR_HIP, "pgk_gated_recurrence: %s", hipGetErrorString(e));
    else if (nch) r = recur_chunked(a, (const RecurChunk*)(ws + o_ch), nch, (const int32_t*)(ws + o_of), ws + o_ws, dt, st);
    else r = recur_rows(a, dt, false, st);
    pgk_free(ws);       // stream-ordered reuse: later work on this stream runs after the kernel above
    return r;
}

pgk_status pgk_state_space(const void* xbc, const void* z, const void* t, const float* decay, const float* step_bias, const float* skip, const float* norm, float* state, void* out,
                           int n, int fresh, int heads, int groups, int dim, int vdim, int norm_parts, float eps, pgk_dtype dt, pgk_stream s) {
    PGK_REQUIRE(xbc && z && t && decay && step_bias && skip && norm && state && out, "pgk_state_space: null pointer");
    PGK_REQUIRE(n >= 1 && heads >= 1 && groups >= 1 && heads % groups == 0 && dim >= 1 && vdim >= 1 && norm_parts >= 1 && heads * vdim % norm_parts == 0,
                "pgk_state_space: bad shape %d / %d x %d x %d, %d norm parts, %d rows", heads, groups, dim, vdim, norm_parts, n);
    PGK_REQUIRE(dt == PGK_BF16 || dt == PGK_F32, "pgk_state_space: dtype %d (bf16 or f32)", (int)dt);
    hipStream_t st = resolve_stream(s);
    // one row buffer z | t, the tables and the chunked form's workspace behind it; head widths that are no multiple of 4 run as copies with
    // zeros behind every head
    const int dp = ceil_div(dim, 4) * 4, vp = ceil_div(vdim, 4) * 4, V = heads * vp, ld = (V + heads + 3) / 4 * 4, ld_x = V + 2 * groups * dp;
    const bool pad = dp != dim || vp != vdim;
    const size_t E = dtype_size(dt), row = (size_t)ld * E, wz = (size_t)V * E, wt = (size_t)heads * E, v1 = (size_t)vdim * E, d = (size_t)dim * E, fv = (size_t)vdim * 4, fvp = (size_t)vp * 4;
    auto up = [](size_t b) { return (b + 255) & ~(size_t)255; };
    RecurArgs a{};
    a.kind = RECUR_SSD; a.ld_in = ld; a.rows = xbc; a.ld_rows = ld_x; a.G = groups; a.f_off = V; a.q_off = V + groups * dp; a.z_off = 0; a.dt_off = V;
    a.dt_bias = step_bias; a.decay = decay; a.skip = skip; a.H = heads; a.dim = dp; a.vdim = vp; a.vdim_true = vdim; a.n = n; a.eps = eps;
    a.state = state; a.n_seqs = 1; a.out = out; a.ld_out = V;
    const int C = n >= RECUR_CHUNKED_FROM ? recur_chunk_rows(dp, vp) : 0, nch = C ? ceil_div(n, C) : 0;
    std::vector<RecurChunk> chunks;
    for (int c = 0; c < nch; ++c) chunks.push_back(RecurChunk{c * C, n - c * C < C ? n - c * C : C});
    const int32_t of_seq[2] = {0, nch};
    const SeqSpan span{0, n, fresh ? 0 : 1, 0};
    size_t at = 0;
    auto take = [&](size_t b) { const size_t o = at; at += up(b); return o; };
    const size_t o_in = take(n * row), o_x = take(pad ? (size_t)n * ld_x * E : 0), o_out = take(pad ? n * wz : 0), o_norm = take(pad ? heads * fvp : 0), o_state = take(pad ? heads * dp * fvp : 0), zeroed = at,
                 o_span = take(sizeof(span)), o_of = take(sizeof(of_seq)), o_ch = take(nch * sizeof(RecurChunk)), o_ws = take(nch ? recur_chunk_bytes(a, nch) : 0);
    char* ws = nullptr;
    if (pgk_status r = pgk_malloc((void**)&ws, at + 256)) return r;
    hipError_t e = pad ? hipMemsetAsync(ws, 0, zeroed, st) : hipSuccess;
    auto copy = [&](size_t dst, size_t ld_dst, size_t p_dst, const void* src, size_t ld_src, size_t p_src, size_t rows, int nh) {
        if (e == hipSuccess) e = copy_heads(ws + dst, ld_dst, p_dst, src, ld_src, p_src, rows, nh, st);
    };
    copy(o_in, row, vp * E, z, heads * v1, v1, n, heads);
    copy(o_in + wz, row, wt, t, wt, wt, n, 1);
    if (pad) {
        const size_t lx = heads * v1 + 2 * groups * d, lp = (size_t)ld_x * E;
        copy(o_x, lp, vp * E, xbc, lx, v1, n, heads);
        copy(o_x + V * E, lp, dp * E, (const char*)xbc + heads * v1, lx, d, n, 2 * groups);
        copy(o_norm, heads * fvp, fvp, norm, heads * fv, fv, 1, heads);
        for (int h = 0; h < heads; ++h) copy(o_state + h * dp * fvp, fvp, fvp, state + (size_t)h * dim * vdim, fv, fv, dim, 1);
        a.rows = ws + o_x; a.state = (float*)(ws + o_state); a.out = ws + o_out; norm = (const float*)(ws + o_norm);
    }
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_span, &span, sizeof(span), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipMemcpyAsync(ws + o_of, of_seq, sizeof(of_seq), hipMemcpyHostToDevice, st);
    if (e == hipSuccess && nch) e = hipMemcpyAsync(ws + o_ch, chunks.data(), nch * sizeof(RecurChunk), hipMemcpyHostToDevice, st);
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    a.in = ws + o_in; a.seqs = (const SeqSpan*)(ws + o_span);
    pgk_status r = PGK_OK;
    if (e == hipSuccess) r = nch ? recur_chunked(a, (const RecurChunk*)(ws + o_ch), nch, (const int32_t*)(ws + o_of), ws + o_ws, dt, st) : recur_rows(a, dt, dt == PGK_F32, st);
    if (r == PGK_OK && e == hipSuccess) r = parts_norm(a.out, V, n, heads, vp, vdim, norm_parts, norm, eps, dt, st);
    if (pad && e == hipSuccess && r == PGK_OK) {
        e = copy_heads(out, heads * v1, v1, ws + o_out, wz, vp * E, n, heads, st);
        for (int h = 0; h < heads && e == hipSuccess; ++h) e = copy_heads(state + (size_t)h * dim * vdim, fv, fv, ws + o_state + h * dp * fvp, fvp, fvp, dim, 1, st);
    }
    if (e != hipSuccess) r = set_error(PGK_ERR_HIP, "pgk_state_space: %s", hipGetErrorString(e));
    pgk_free(ws);       // stream-ordered reuse
    return r;
}

}  // extern "C"
