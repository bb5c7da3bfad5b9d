// Engine state and step bookkeeping shared by every kind of model the native engine runs (engine.hip: QKV + RoPE decoders;
// engine_stack.hip: layer lists).  The C entry points that do not depend on the kind are in engine_api.hip.
#pragma once

#include <cstdlib>
#include <type_traits>
#include <vector>

#include "engine_common.hip.h"

namespace pgk {

constexpr int SHORT_CTX = 512;   // contexts up to here take the whole-context attention kernels (direct batch attention); one sequence: SHORT_CTX_B1
constexpr int SHORT_CTX_B1 = 384; // a single sequence's fused attention + o_proj kernel walks the context in chunks of 192 rows (AM_CHUNK) in EVERY one of its
                                  // 256 workgroups: two chunks still beat the split-KV sequence (context 300: 0.616 vs 0.625 ms per step), three do not (400: 0.678 vs 0.627)

// token[b] = argmax over workgroup partials (ties -> lowest index); position[b] += 1; log the token;
// h[b] = E[token] for the next step; the last workgroup of the step's last chunk bumps the step counter.
// One workgroup per sequence (grid = M).  Every workgroup reads the step counter before it takes an arrival ticket
// (step_counter[1]); the bump is made by whoever draws the last ticket, so it cannot overtake a read.  (One workgroup
// for the whole chunk, a wave per sequence, took 25 us at M = 8 and 57 us at M = 16 - a dependent walk per sequence.)
template <class ET>   // ET: type of the embedding tables
__global__ __launch_bounds__(256) void finalize_kernel(unsigned long long* tl, const float* amax_val, const int* amax_idx, int nblk,
                                                       int32_t* tokens, int32_t* positions, int32_t* token_log,
                                                       int32_t* step_counter, int log_width, int log_cap,
                                                       const ET* embed, float* h, int H, int bump,
                                                       unsigned long long* clk_log, const float* rope_cos,
                                                       const float* rope_sin, float* cur_cos, float* cur_sin, int half,
                                                       int max_seq, int M, const int32_t* sampled, const ET* pos_embed, int ld_h) {
    const TLStamp tls(tl);
    __shared__ float sv[4];
    __shared__ int si[4];
    __shared__ int s_tok, s_pos;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, b = blockIdx.x;
    const int step = step_counter[0];
    int bi;
    if (sampled) {
        bi = sampled[b];                                  // temperature / top-k / top-p draw (ops_sampling.hip)
    } else {
        float bv = -INFINITY;
        bi = 0x7FFFFFFF;
        for (int i = threadIdx.x; i < nblk; i += 256) {
            const float v = amax_val[(size_t)b * nblk + i];
            const int ix = amax_idx[(size_t)b * nblk + i];
            if (v > bv || (v == bv && ix < bi)) { bv = v; bi = ix; }
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) {
            const float ov = __shfl_xor(bv, off, 64);
            const int oi = __shfl_xor(bi, off, 64);
            if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
        }
        if (lane == 0) { sv[wid] = bv; si[wid] = bi; }
        __syncthreads();
        bv = sv[0]; bi = si[0];
#pragma unroll
        for (int w = 1; w < 4; ++w)
            if (sv[w] > bv || (sv[w] == bv && si[w] < bi)) { bv = sv[w]; bi = si[w]; }
        if (bi == 0x7FFFFFFF) bi = 0;
    }
    if (threadIdx.x == 0) {
        s_tok = bi;
        tokens[b] = bi;
        const int npos = positions[b] + 1;
        positions[b] = npos;
        s_pos = min(npos, max_seq - 1);
        if (step < log_cap) token_log[(size_t)step * log_width + b] = bi;
        if (b == 0 && step < log_cap && clk_log) {  // shader-clock / 100 MHz wall-clock stamps (diagnostic only)
            clk_log[2 * (size_t)step] = __builtin_amdgcn_s_memtime();
            clk_log[2 * (size_t)step + 1] = __builtin_amdgcn_s_memrealtime();
        }
    }
    __syncthreads();
    // next step's inputs of this sequence: its embedding row (8 bf16 per lane) and the RoPE row of its next position
    const ET* erow = embed + (size_t)s_tok * H;
    float* hrow = h + (size_t)b * ld_h;
    if (pos_embed) {          // learned positions: one row per position, added in fp32
        const ET* prow = pos_embed + (size_t)s_pos * H;
        for (int i = threadIdx.x; i < H; i += 256) hrow[i] = to_f(erow[i]) + to_f(prow[i]);
    } else if (std::is_same<ET, bf16>::value && (H & 7) == 0) {
        for (int v = threadIdx.x; v < (H >> 3); v += 256) {
            const uint4 raw = *reinterpret_cast<const uint4*>(erow + v * 8);
            float f[8];
            WTraits<bf16>::decode(raw, f);
            *reinterpret_cast<float4*>(hrow + v * 8) = make_float4(f[0], f[1], f[2], f[3]);
            *reinterpret_cast<float4*>(hrow + v * 8 + 4) = make_float4(f[4], f[5], f[6], f[7]);
        }
    } else {
        for (int i = threadIdx.x; i < H; i += 256) hrow[i] = to_f(erow[i]);
    }
    for (int i = threadIdx.x; i < half; i += 256) {
        cur_cos[(size_t)b * half + i] = rope_cos[(size_t)s_pos * half + i];
        cur_sin[(size_t)b * half + i] = rope_sin[(size_t)s_pos * half + i];
    }
    if (bump && threadIdx.x == 0) {
        if (M == 1) {
            step_counter[0] = step + 1;
        } else if (atomicAdd(&step_counter[1], 1) == M - 1) {   // every workgroup has read `step` before its own ticket
            atomicExch(&step_counter[1], 0);
            step_counter[0] = step + 1;
        }
    }
    tls.end();
}

struct Engine;

// The launch sequences of one kind of model.  Everything else an engine has - decode state, token log, sampling, graph capture
// and replay, timing - is shared (engine_api.hip), so a kind registers its functions here when it creates an engine.
struct EngineKind {
    pgk_status (*decode_step)(Engine* e, int batch, hipStream_t st, int* launches, bool short_ctx);
    // n_seqs sequences in one call, tokens concatenated; fp32 logits of the `want` rows (indices into the concatenation)
    pgk_status (*prefill)(Engine* e, int n_seqs, const int32_t* h_slots, const int32_t* h_lens, const int32_t* h_starts, const int32_t* h_tokens,
                          int n_want, const int32_t* h_want, float* h_logits, hipStream_t st);
    // one sequence; bf16 logits of every row and / or fp32 logits of the last one (null: only `prefill` exists)
    pgk_status (*prefill_one)(Engine* e, int seq, const int32_t* h_tokens, int n, int start_pos, void* all_logits, float* h_last_logits, hipStream_t st);
    pgk_status (*embed_state)(Engine* e, int batch, hipStream_t st);     // the residual stream of the state tokens (step entry)
    // may a step run at these positions? (host side; null: any position inside the cache)
    pgk_status (*check_state)(Engine* e, const int32_t* h_positions, int batch);
    void (*advance)(Engine* e, int batch, int steps);                    // the device state moved on by `steps` (null: nothing to note)
    pgk_status (*kv_ptr)(Engine* e, int layer, void** k, void** v);
    void (*destroy)(Engine* e);                                          // null: nothing beyond Engine itself
};

struct Engine {
    const EngineKind* kind = nullptr;
    void* kind_state = nullptr;
    pgk_model_config_t cfg;
    const bf16 *embed, *lm_head, *final_norm;
    std::vector<pgk_layer_weights_t> layers;
    int nsplit = 1, lm_blocks = 1, lm_cap = 1, log_cap = 4096;
    bool batched_mfma = true;   // chunks of 3 and 5..16 sequences use engine_batched.hip.h (PGK_BATCHED_MFMA=0: GEMV kernels only, =2: from 3 up)
    int batched_min = 5, batched_max = 64;   // PGK_BATCHED_MAX=16: chunks of at most 16 sequences (one weight pass per chunk), the A/B switch of the tiled kernels
    int cu_count = 256;
    bool short_path = true;     // contexts <= SHORT_CTX take the whole-context attention kernels (PGK_FUSED_ATTN=0: the split-KV sequence at every context)
    int pos_hi = -1;            // host-side upper bound of the largest position the next step sees (-1: unknown); selects the sequence, see step_is_short
    // in-graph stochastic sampling (pgk_engine_set_sampling): temperature <= 0 keeps greedy argmax
    float sample_temperature = 0.f, sample_top_p = 1.f;
    int sample_top_k = 0, u_cap = 0, u_alloc_rows = 0;   // u_cap: rows in use (ring length); u_alloc_rows: rows allocated
    float* u_ring = nullptr;       // [u_cap][max_batch] uniforms, row = step counter % u_cap
    void* sample_scratch = nullptr;   // top-k candidate keys (ops_sampling.hip), sized for max_batch rows
    size_t sample_scratch_cap = 0;
    int32_t* sampled = nullptr;    // [max_batch]
    bool fused_attn = false;   // one sequence at short context: attn + o_proj in one kernel (bf16 W_o, shapes that tile)
    bool attn_mfma = false;    // ... with Q.K^T and P.V on the matrix pipe from LDS-staged K/V (head_dim 128; PGK_ATTN_MFMA=0: the dot2 kernels); also the whole-context
                               // batch attention while its workgroups (96 KB of LDS: one per CU) fit one round - batch x Hkv <= CUs (beyond: attn_decode_kernel, batch 64 1.258 vs 1.316 ms)
    bool merged_oproj = false; // long contexts / fp8 W_o, one or two sequences: split-KV merge + o_proj in one kernel (PGK_MERGED_OPROJ=0: merge kernel + GEMV)
    int moproj_rows = 32;
    int oproj_rows = 32;       // W_o rows per workgroup on the fused path
    // device state
    bf16 *kcache = nullptr, *vcache = nullptr;
    float *rope_cos = nullptr, *rope_sin = nullptr, *cur_cos = nullptr, *cur_sin = nullptr;
    int32_t *tokens = nullptr, *positions = nullptr, *token_log = nullptr, *step_counter = nullptr;
    bf16 *act16 = nullptr, *attnv16 = nullptr;   // batched MFMA path: bf16 hand-off of SwiGLU output and attention output
    bf16* x16 = nullptr;                         // 17..64 sequences: the next RMSNorm's input rows in bf16 (layer 0: normalised by norm_rows_bf16; then un-normalised, written by o_proj / down)
    float* ss_part = nullptr;                    // ... and its statistic: per-workgroup sums of squares [64][1024]
    float *h = nullptr, *h2 = nullptr, *qkv = nullptr, *part = nullptr, *opart = nullptr, *attnv = nullptr, *act = nullptr, *logits = nullptr,
          *amax_val = nullptr;
    int* amax_idx = nullptr;
    unsigned long long* clk_log = nullptr;
    size_t kv_bytes = 0, ws_bytes = 0;
    // fragment-major copies of the layer weights for prompts of <= 128 tokens (ops_pkgemm.hip); PGK_PACKED_PREFILL=0: none
    struct PackedLayer { bf16 *qkv = nullptr, *o = nullptr, *gate_up = nullptr, *down = nullptr; };
    std::vector<PackedLayer> packed;
    bool packed_ok = false;     // the skinny-GEMM kernels of ops_pkgemm.hip can use the copy (their shape limits)
    bool packed_have = false;   // the copy exists (w8a16 engines: also for shapes beyond those kernels - the long-prompt GEMMs read it)
    size_t packed_bytes = 0;
    bool packed_resid = false;      // o_proj / down_proj without K split, carrying the next RMSNorm (pkgemm_resid_nt); PGK_PACKED_RESID=0: split-K slabs + norm launches
    float* pk_ss = nullptr;         // its sum-of-squares table [128][PK_SS_LD]
    bf16* packed_lm = nullptr;      // fragment-major lm_head for the batched (3..64 sequences) lm_head kernels; PGK_PACKED_LMHEAD=0: none
    float* dec_slabs = nullptr;     // 17..64 sequences on the packed kernels: split-K slabs of o_proj / down_proj [splits][M][H] (PGK_PACKED_DECODE=0: engine_batched kernels)
    bool packed_decode = false;
    // prefill workspace (grown on demand, outside capture)
    void* pf = nullptr;
    size_t pf_bytes = 0;
    int32_t* pf_tokens = nullptr;
    int pf_tokens_cap = 0;
    // captured step: [0] the long-context launch sequence, [1] the short-context one (when the engine has both)
    // captured steps: tier 0 = the short-context sequence (span 0); the others = the split-KV sequence with its slices cut for
    // contexts up to `span` positions (1024, 2048, ... and the cache length).  pgk_engine_replay picks per step (pick_tier).
    struct Tier { int span = 0; hipGraph_t graph = nullptr; hipGraphExec_t exec = nullptr; int launches = 0; };
    std::vector<Tier> tiers;
    int graph_batch = 0;
    bool one_sequence = false;  // the kind has ONE launch sequence, right and fast at every context: a single captured tier
    int step_span = 0;          // the split-KV slicing of the step being enqueued (launch_attn); 0: the whole cache
    int launches_per_step = 0;
    std::vector<void*> allocs;

    size_t kv_layer_elems() const { return (size_t)cfg.max_batch * cfg.num_kv_heads * cfg.max_seq_len * cfg.head_dim; }
    int qkv_dim() const { return (cfg.num_heads + 2 * cfg.num_kv_heads) * cfg.head_dim; }
};

inline pgk_status dev_alloc(Engine* e, void** p, size_t bytes, size_t* acct) {
    pgk_status r = pgk_malloc(p, bytes);
    if (r != PGK_OK) return r;
    e->allocs.push_back(*p);
    if (acct) *acct += bytes;
    return PGK_OK;
}

pgk_status sample_rows_ring(const float* logits, int rows, int vocab, float temperature, int top_k, float top_p, const float* u_ring,
                            int u_cap, int u_stride, const int32_t* step_counter, int32_t* out, void* scratch, hipStream_t st);
size_t sample_scratch_bytes(int rows, int vocab, int top_k, float top_p);

// one draw per sequence of the chunk from the fp32 logits the lm_head kernel just wrote; the uniform numbers come from
// the device ring row (step counter % u_cap), so a captured graph replays with fresh randomness the host queued up
inline pgk_status engine_sample(Engine* e, int b0, int M, hipStream_t st) {
    return sample_rows_ring(e->logits + (size_t)b0 * e->cfg.vocab_size, M, e->cfg.vocab_size, e->sample_temperature, e->sample_top_k,
                            e->sample_top_p, e->u_ring + b0, e->u_cap, e->cfg.max_batch, e->step_counter, e->sampled + b0, e->sample_scratch, st);
}

// Which launch sequence the NEXT step takes: the short-context one while the host-side bound on the step's largest
// position (set by pgk_engine_set_state, advanced by every step this library enqueues) stays below SHORT_CTX.  The bound
// is a speed hint only - both sequences are correct at any context - so a caller that rewrites the device-resident
// positions behind the library's back loses speed, never correctness; an unknown bound selects the long sequence.
inline int short_limit(int batch) { return batch == 1 ? SHORT_CTX_B1 : SHORT_CTX; }
inline bool step_is_short(const Engine* e, int batch) { return e->short_path && e->pos_hi >= 0 && e->pos_hi + 1 <= short_limit(batch); }

inline void drop_graphs(Engine* e) {
    for (auto& t : e->tiers) {
        if (t.exec) (void)hipGraphExecDestroy(t.exec);
        if (t.graph) (void)hipGraphDestroy(t.graph);
    }
    e->tiers.clear();
    e->graph_batch = 0;
}

// The split-KV slicing a step at the host-side position bound needs: the smallest of 1024, 2048, ... that covers the context, capped at
// the cache length (an unknown bound: the cache length).
inline int span_for(const Engine* e) {
    const int cap = e->cfg.max_seq_len;
    if (e->pos_hi < 0) return cap;
    int span = 1024;
    while (span < e->pos_hi + 1 && span < cap) span *= 2;
    return span < cap ? span : cap;
}

// The captured step the next replay takes: the short-context sequence while the position bound allows it (and it was captured),
// otherwise the split-KV tier whose slices cover the context; both kinds are correct at any context they cover.
inline size_t pick_tier(const Engine* e) {
    const bool has_short = !e->tiers.empty() && e->tiers[0].span == 0;
    if (has_short && (e->tiers.size() == 1 || step_is_short(e, e->graph_batch))) return 0;
    const int want = span_for(e);
    for (size_t i = has_short ? 1 : 0; i < e->tiers.size(); ++i)
        if (e->tiers[i].span >= want) return i;
    return e->tiers.size() - 1;
}

}  // namespace pgk
