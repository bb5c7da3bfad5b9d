// Sequence mixers of the layer-list engine beside latent attention (engine_stack.hip): short causal convolutions with norms over whole
// projections, attention over a K/V ring with distance bias and elementwise gate (ops_gated_attn.hip), and a gated linear recurrence
// whose forget gate also decides what is written (ops_recurrence.hip).
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

// Keys of a query at position `pos` with window `window` in a ring of R rows (position p in row p % R): n keys, oldest first, key t in
// ring row lo + t (minus R past the end) at distance n - 1 - t.
__device__ __forceinline__ void ring_window(int pos, int window, int R, int& n, int& lo) {
    n = min(pos + 1, min(window, R));
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
};
bool kv_attn_q32(int D, pgk_dtype dt);
int kv_attn_splits(int B, int H, int G, int keys, int cus);
pgk_status kv_attn_decode(const KvAttnArgs& a, pgk_dtype dt, bool io32, hipStream_t st, int* launches);

// ---- gated linear recurrence ----
//   q = silu(z_q),  f = lower + (1 - lower) sigmoid(z_f + bias),  S <- diag(f) S + (1 - f) v^T,  o = S^T q;  norm given: o / rms(o) * norm
// Rows of `in`: z_q at q_off + head * dim, z_f at f_off + head * dim, v at v_off + head * vdim.
struct RecurArgs {
    const void* in; int ld_in, q_off, f_off, v_off;
    const float *bias, *lower;            // [H * dim]; bias may be null
    const float* norm;                    // [vdim] or null
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

}  // namespace pgk
