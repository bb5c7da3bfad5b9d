// Sequence mixers of the layer-list engine beside latent attention (engine_stack.hip): short causal convolutions with norms over whole
// projections, attention over a K/V ring with distance bias and elementwise gate (ops_gated_attn.hip), linear recurrences whose decay
// also decides what is written or stands beside it (ops_recurrence.hip), and the gated delta rule with a decay per channel (ops_delta.hip).
#pragma once

#include "engine_common.hip.h"
#include "latent.hip.h"

namespace pgk {

// A prompt row: its position, its slot, and the row its sequence's portion starts with (positions before that live in the slot's state)
struct RowSrc { int32_t pos, slot, first; };
// A sequence's portion: rows row0 .. row0 + len - 1 are positions start .. start + len - 1 of slot `slot`
struct SeqSpan { int32_t row0, len, start, slot; };
// A prompt row's place: position, cache slot, row in the prompt's K/V (or latent) scratch, and whether the ring keeps it
struct RowPlace { int32_t pos, slot, kv, store; };

// How many keys a query at position `pos` sees: a sliding window, or its own chunk of `window` positions, itself included
__host__ __device__ __forceinline__ int span_keys(int pos, int window, int chunked) { return chunked ? pos % window + 1 : pos < window ? pos + 1 : window; }
// The keys of that query in a ring of R rows (position p in row p % R): n keys, oldest first, key t in ring row lo + t (minus R past the
// end) at distance n - 1 - t.
__device__ __forceinline__ void ring_window(int pos, int window, int R, int& n, int& lo, int chunked = 0) {
    n = min(span_keys(pos, window, chunked), R);
    lo = (pos - n + 1) % R;
}
__device__ __forceinline__ int ring_row(int lo, int t, int R) { const int r = lo + t; return r >= R ? r - R : r; }

// n keys over nsplit splits: keys per split (a multiple of 32), the keys [k0, k1) of split s
__device__ __forceinline__ int split_rows(int n, int nsplit) { return ((n + nsplit - 1) / nsplit + 31) / 32 * 32; }
__device__ __forceinline__ void split_range(int n, int nsplit, int s, int& k0, int& k1) {
    const int per = split_rows(n, nsplit);
    k0 = min(s * per, n);
    k1 = min(k0 + per, n);
}

// ---- projection rows -> q, k, v: bias, causal taps over time, RMS norm of the whole q and the whole k row ----
// Channels q (n_q) | k (n_kv) | v (n_kv), heads of width D.  Decode (rows null): row b is the next token of slot b at positions[b]; its
// projected values go to the tap ring [slot][taps][channels] (position p in row p % taps) and k, v to the cache.  Prompt: taps reach
// into the rows above within a portion and into the ring before it; k, v go to scratch rows [k | v] and, where the ring keeps them, to
// the cache [slot][k, v][head][R][D].
struct ConvArgs {
    const void* in; int ld_in;
    const float* bias;                    // [channels] or null
    const void* conv;                     // [taps][channels] (element type) or null (no taps)
    int taps, n_q, n_kv, D, n, R;
    const float *q_norm, *k_norm;         // [n_q], [n_kv]; null: no norm
    int q_true, k_true;                   // channels that are not padding
    float eps, q_mult;
    void* tap_ring;
    const int32_t* positions;
    const RowSrc* rows; const RowPlace* place;
    void* q_out; int ld_q;
    void* kv_rows; int ld_kv;
    void* cache;
};
// dt: cache / ring / scratch element type; in32: the projection rows are fp32 (else dt); q32: q leaves as fp32 (else dt)
pgk_status conv_rows(const ConvArgs& a, pgk_dtype dt, bool in32, bool q32, hipStream_t st);
// after the prompt's rows have been read: the last `taps` projected rows of every sequence -> tap ring
pgk_status conv_save(const void* in, int ld_in, const SeqSpan* seqs, int n_seqs, void* tap_ring, int taps, int channels, pgk_dtype dt, hipStream_t st);
// K/V rows of earlier positions -> prompt scratch (K rows then V rows of n_kv channels each)
pgk_status kv_gather(const RowPlace* place, int n, const void* cache, void* kv_rows, int ld_kv, int n_kv, int D, int R, pgk_dtype dt, hipStream_t st);

// ---- one query per sequence over the K/V ring ----
struct KvAttnArgs {
    const void* q;                        // [B][H * D], times scale * log2e; fp32 or bf16 (kv_attn_q32)
    const void* cache;                    // [slots][k, v][G][R][D]
    const float* slopes;                  // [H]: slope * distance is taken off the score; null: none
    const int32_t* positions;
    int B, H, G, D, R, window, nsplit;
    float *po, *pml;                      // records [B][H][nsplit][D] and [B][H][nsplit][2]
    const void* gate; int ld_gate;        // rows like `out`: the result is multiplied by its sigmoid; null: none
    void* out; int ld_out;                // head h at h * D
    const float* sink;                    // [H]: exp(sink) stands in the denominator (kv_merge only; null: none)
    int chunked;
};
// combine the split records po, pml -> out (gate, sink)
pgk_status kv_merge(const KvAttnArgs& a, bool io32, hipStream_t st);
bool kv_attn_q32(int D, pgk_dtype dt);
int kv_attn_splits(int B, int H, int G, int keys, int cus);
pgk_status kv_attn_decode(const KvAttnArgs& a, pgk_dtype dt, bool io32, hipStream_t st, int* launches);

// ---- projection rows -> q, k, v heads: bias, RMS norm per head, rotation of the first columns by the position (ops_talk.hip) ----
// Heads q (H) | k (G) | v (G) of width D, `dim` of them true; G 0: only q.  Column i < rot / 2 turns with column i + rot / 2.  Rows, k and v go
// where conv_rows puts them; everything but `in` is in the element type.
struct HeadRowsArgs {
    const void* in; int ld_in;
    const float* bias;                    // [(H + 2 G) * D] or null
    const float *q_norm, *k_norm;         // [D] or null
    int H, G, D, dim, rot, n, R;
    const float* rot_freq;                // [rot / 2]
    float eps;
    const int32_t* positions;
    const RowSrc* rows; const RowPlace* place;
    void* q_out; int ld_q;
    void* kv_rows; int ld_kv;
    void* cache;
};
pgk_status head_rows(const HeadRowsArgs& a, pgk_dtype dt, bool in32, hipStream_t st);

// ---- attention whose heads mix their scores, with a sink (ops_talk.hip) ----
// raw_h = scale q_h . k,  score_h = sum_g talk[h][g] raw_g,  weights exp(score_h) / (sum over the keys + exp(sink_h))
struct TalkArgs {
    const void* q; int ld_q;              // rows, head h at h * D
    const float *talk, *sink;             // [H][H] or null (no mixing), [H] or null (no sink)
    int H, G, D, n, window, chunked;      // n: rows
    float scale;
    // decode (cache given): row b is the next token of slot b at positions[b], over the ring [slots][k, v][G][R][D] in nsplit splits
    const void* cache; const int32_t* positions;
    int R, nsplit;
    float *po, *pml;
    // prompt: kv_len rows of k and v (head g at g * D), row t is position pos0 + t; the queries are the last n of them
    const void *k, *v; int ld_kv, kv_len, pos0;
    void* out; int ld_out;                // head h at h * D
    int Dv, ld_v;                         // value heads of another width, rows ld_v apart, heads of `out` too (0: D, ld_kv); prompts only
};
int talk_splits(int B, int H, int G, int keys, int cus);
pgk_status talk_attention(const TalkArgs& a, pgk_dtype dt, bool io32, hipStream_t st, int* launches);   // io32: `out` is fp32 (else dt)

// ---- taps over time and SiLU ----
// y_t = silu(bias + sum_j w_j u_(t - taps + 1 + j)) per channel, zero before a sequence's start.  Ring [slot][taps][channels] of u: position p
// in row p % taps (`taps` rows, so that writing a position touches no row the same step reads).
struct ConvSiluArgs {
    const void* in; int ld_in;            // the first channel of every row
    const void* conv; const float* bias;  // [taps][channels] (element type), [channels] or null
    int taps, channels, n;                // channels: a multiple of 4
    const void* ring; const RowSrc* rows;
    void* out; int ld_out;
};
pgk_status conv_silu_rows(const ConvSiluArgs& a, pgk_dtype dt, hipStream_t st);

// One channel of the next token in a decode step (a kernel that needs a few channels per workgroup convolves them itself); `write`: the new
// row goes to the ring, once per channel.
struct ConvStep { const void* conv; const float* bias; int taps, channels; void* ring; };
template <bool EXACT> __device__ __forceinline__ float silu_f(float z) { return z / (1.0f + (EXACT ? expf(-z) : __expf(-z))); }
template <class T, class IT, bool EXACT>
__device__ __forceinline__ float conv_step(const ConvStep& cs, const IT* in, int c, int slot, int pos, bool write) {
    const T* w = reinterpret_cast<const T*>(cs.conv);
    T* ring = reinterpret_cast<T*>(cs.ring) + (size_t)slot * cs.taps * cs.channels + c;
    const float u = to_f(in[c]);
    float y = fmaf(to_f(w[(size_t)(cs.taps - 1) * cs.channels + c]), u, cs.bias ? cs.bias[c] : 0.f);
    float x[3], g[3];
#pragma unroll
    for (int k = 0; k < 3; ++k) {                                  // three taps back in flight, masked
        const int b = min(k + 1, cs.taps - 1), p = max(pos - b, 0);
        x[k] = to_f(ring[(size_t)(p % cs.taps) * cs.channels]);
        g[k] = k + 1 < cs.taps && pos - b >= 0 ? to_f(w[(size_t)(cs.taps - 1 - b) * cs.channels + c]) : 0.f;
    }
#pragma unroll
    for (int k = 0; k < 3; ++k) y = g[k] != 0.f ? fmaf(g[k], x[k], y) : y;      // (an unread ring row may hold anything)
    for (int b = 4; b < cs.taps && pos - b >= 0; ++b) y = fmaf(to_f(w[(size_t)(cs.taps - 1 - b) * cs.channels + c]), to_f(ring[(size_t)((pos - b) % cs.taps) * cs.channels]), y);
    if (write) ring[(size_t)(pos % cs.taps) * cs.channels] = from_f<T>(u);
    return silu_f<EXACT>(y);
}

// ---- linear recurrences S <- diag(f) S + k v^T, o = S^T q ----
// RECUR_HGRN2: q = silu(z_q),  f = lower + (1 - lower) sigmoid(z_f + bias),  k = 1 - f;  norm given: o / rms(o) * norm.
//   Rows of `in`: z_q at q_off + head * dim, z_f at f_off + head * dim, v at v_off + head * vdim.
// RECUR_SSD: t = softplus(dt + dt_bias), f = exp(-decay t) for every channel, k = t B, q = C, v = x;  (o + skip v) silu(z).
//   x at v_off + head * vdim, B at f_off + group * dim, C at q_off + group * dim: channels of `rows` (prompts: after taps and SiLU) or of `in`
//   (decode: before them, `conv`); z at z_off + head * vdim, dt at dt_off + head of `in`.  Group of a head: head / (H / G).
enum { RECUR_HGRN2 = 0, RECUR_SSD = 1 };
struct RecurArgs {
    int kind;
    const void* in; int ld_in, q_off, f_off, v_off;
    const float *bias, *lower;            // [H * dim]; bias may be null
    const float* norm;                    // [vdim] or null
    const void* rows; int ld_rows;
    int G, z_off, dt_off;
    const float *dt_bias, *decay, *skip;  // [H]
    ConvStep conv;
    int H, dim, vdim, vdim_true, n;       // n: rows (decode: sequences)
    float eps;
    float* state;                         // [slots][H][dim][vdim] fp32
    const SeqSpan* seqs; int n_seqs;      // null: row b is the next token of slot b at positions[b]
    const int32_t* positions;
    void* out; int ld_out;                // head h at h * vdim; columns H * vdim .. ld_out are zeroed
};
pgk_status recur_rows(const RecurArgs& a, pgk_dtype dt, bool io32, hipStream_t st);
size_t recur_chunk_bytes(const RecurArgs& a, int n_chunks);                                     // workspace of the chunked form
struct RecurChunk { int32_t row0, len; };
constexpr int RECUR_CHUNKED_FROM = 16;                                                          // rows of the longest portion from which the chunked form pays
int recur_chunk_rows(int dim, int vdim);                                                        // rows per chunk; 0: sizes the chunked form does not take
// the chunked form: chunks in order, sequence by sequence (chunk_of_seq[i] .. chunk_of_seq[i + 1] are sequence i's)
pgk_status recur_chunked(const RecurArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, void* ws, pgk_dtype dt, hipStream_t st);

// x / rms(x) * norm in `parts` equal parts of each row's heads x vdim_true elements (heads vdim apart), in place
pgk_status parts_norm(void* x, int ld, int n, int heads, int vdim, int vdim_true, int parts, const float* norm, float eps, pgk_dtype dt, hipStream_t st);

// ---- gated delta rule with a decay per key channel ----
//   q, k of unit length (q times dim_true^-1/2),  b = sigmoid(beta),  g = exp(-decay softplus(z + dt_bias));
//   S <- diag(g) S,  u = b (v - S^T k),  S <- S + k u^T,  o = S^T q;  o / rms(o) * norm * sigmoid(gate)
// Channels q (G x dim) | k (G x dim) | v (H x vdim) of `rows` (prompts: after taps and SiLU) or of `in` (decode: before them).
struct DeltaArgs {
    const void* in; int ld_in, b_off;     // beta of head h at b_off + h
    const void* rows; int ld_rows;
    const float* z; int ld_z;             // [n][H * dim]
    const void* gate; int ld_gate;        // [n][H * vdim], typed as the projection rows
    ConvStep conv;
    const float *decay, *dt_bias, *norm;  // [H], [H * dim], [vdim]
    int H, G, dim, vdim, dim_true, vdim_true, n;
    float eps;
    float* state;                         // [slots][H][dim][vdim] fp32
    const SeqSpan* seqs; int n_seqs;      // null: row b is the next token of slot b at positions[b]
    const int32_t* positions;
    void* out; int ld_out;                // head h at h * vdim; columns H * vdim .. ld_out are zeroed
};
pgk_status delta_rows(const DeltaArgs& a, pgk_dtype dt, bool io32, hipStream_t st);
constexpr int DELTA_CHUNK = 64;                                                                 // rows per chunk of the chunked form
bool delta_chunk_ok(int dim, int vdim);
size_t delta_chunk_bytes(const DeltaArgs& a, int n_chunks);
pgk_status delta_chunked(const DeltaArgs& a, const RecurChunk* chunks, int n_chunks, const int32_t* chunk_of_seq, void* ws, pgk_dtype dt, hipStream_t st);

// z = A x_a (fp32 [n][na]) and g = G x_g (IT [n][ng]) for a few rows: x_a, x_g are columns of the projection rows, ka and kg of them
pgk_status lowrank_rows(const void* in, int ld_in, int n, int a_off, int ka, const void* wa, float* z, int na, int g_off, int kg, const void* wg, void* g, int ng,
                        pgk_dtype dt, bool io32, hipStream_t st);
// columns off .. off + cols of rows -> dense rows
pgk_status rows_slice(const void* in, int ld_in, int off, int cols, void* out, int n, pgk_dtype dt, hipStream_t st);

// Device copies of rows [rows][heads * d] to or from rows whose heads are `p` elements apart (bytes throughout; the ends of wider heads are
// left alone).
inline hipError_t copy_heads(void* dst, size_t ld_dst, size_t p_dst, const void* src, size_t ld_src, size_t p_src, size_t rows, int heads, hipStream_t st) {
    if (p_dst == p_src) return hipMemcpy2DAsync(dst, ld_dst, src, ld_src, heads * p_dst, rows, hipMemcpyDeviceToDevice, st);
    const size_t w = p_dst < p_src ? p_dst : p_src;
    hipError_t e = hipSuccess;
    for (int h = 0; h < heads && e == hipSuccess; ++h)
        e = hipMemcpy2DAsync((char*)dst + h * p_dst, ld_dst, (const char*)src + h * p_src, ld_src, w, rows, hipMemcpyDeviceToDevice, st);
    return e;
}

}  // namespace pgk
