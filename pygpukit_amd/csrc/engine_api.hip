// Engine entry points shared by every kind of model: lifetime, decode state, graph capture / replay, sampling, token log and
// the measurement hooks.  What a step or a prompt launches comes from Engine::kind (engine.hip, engine_stack.hip).

#include "engine_state.hip.h"

namespace pgk {

thread_local Probe* g_probe = nullptr;   // measurement hooks: engine_common.hip.h

}  // namespace pgk

using namespace pgk;

extern "C" {

pgk_status pgk_engine_destroy(pgk_engine eh) {
    if (!eh) return PGK_OK;
    Engine* e = (Engine*)eh;
    drop_graphs(e);
    if (e->kind && e->kind->destroy) e->kind->destroy(e);
    for (void* p : e->allocs) (void)pgk_free(p);
    if (e->pf) (void)pgk_free(e->pf);
    if (e->pf_tokens) (void)pgk_free(e->pf_tokens);
    if (e->u_ring) (void)pgk_free(e->u_ring);
    if (e->sampled) (void)pgk_free(e->sampled);
    if (e->sample_scratch) (void)pgk_free(e->sample_scratch);
    delete e;
    return PGK_OK;
}

pgk_status pgk_engine_bytes(pgk_engine eh, size_t* kv_bytes, size_t* workspace_bytes) {
    PGK_REQUIRE(eh, "pgk_engine_bytes: null engine");
    Engine* e = (Engine*)eh;
    if (kv_bytes) *kv_bytes = e->kv_bytes;
    if (workspace_bytes) *workspace_bytes = e->ws_bytes + e->pf_bytes + e->packed_bytes;
    return PGK_OK;
}

pgk_status pgk_engine_prefill_batch(pgk_engine eh, int n_seqs, const int32_t* h_slots, const int32_t* h_lens, const int32_t* h_starts,
                                    const int32_t* h_tokens, int n_want, const int32_t* h_want, float* h_logits, pgk_stream s) {
    PGK_REQUIRE(eh && h_slots && h_lens && h_starts && h_tokens && n_seqs >= 1, "pgk_engine_prefill_batch: null argument");
    PGK_REQUIRE(n_want == 0 || (n_want > 0 && h_want && h_logits), "pgk_engine_prefill_batch: wanted rows without an output");
    Engine* e = (Engine*)eh;
    const auto& c = e->cfg;
    long long total = 0;
    std::vector<char> used(c.max_batch, 0);
    for (int i = 0; i < n_seqs; ++i) {
        PGK_REQUIRE(h_slots[i] >= 0 && h_slots[i] < c.max_batch, "pgk_engine_prefill: sequence slot %d outside [0,%d)", h_slots[i], c.max_batch);
        PGK_REQUIRE(!used[h_slots[i]], "pgk_engine_prefill_batch: slot %d twice in one call", h_slots[i]);
        used[h_slots[i]] = 1;
        PGK_REQUIRE(h_lens[i] >= 1 && h_starts[i] >= 0 && (long long)h_starts[i] + h_lens[i] <= c.max_seq_len,
                    "pgk_engine_prefill: positions %d..%lld outside cache of %d", h_starts[i], (long long)h_starts[i] + h_lens[i], c.max_seq_len);
        total += h_lens[i];
    }
    PGK_REQUIRE(total < (1ll << 30), "pgk_engine_prefill_batch: %lld tokens in one call", total);
    for (long long i = 0; i < total; ++i)
        PGK_REQUIRE(h_tokens[i] >= 0 && h_tokens[i] < c.vocab_size, "pgk_engine_prefill: token %d out of range", h_tokens[i]);
    for (int i = 0; i < n_want; ++i) PGK_REQUIRE(h_want[i] >= 0 && h_want[i] < total, "pgk_engine_prefill_batch: wanted row %d outside [0,%lld)", h_want[i], total);
    return e->kind->prefill(e, n_seqs, h_slots, h_lens, h_starts, h_tokens, n_want, h_want, h_logits, resolve_stream(s));
}

pgk_status pgk_engine_prefill(pgk_engine eh, int seq, const int32_t* h_tokens, int n, int start_pos, void* all_logits,
                              float* h_last_logits, pgk_stream s) {
    PGK_REQUIRE(eh && h_tokens, "pgk_engine_prefill: null argument");
    Engine* e = (Engine*)eh;
    if (e->kind->prefill_one) return e->kind->prefill_one(e, seq, h_tokens, n, start_pos, all_logits, h_last_logits, resolve_stream(s));
    PGK_REQUIRE(!all_logits, "pgk_engine_prefill: this model's logits come from pgk_engine_prefill_batch (any rows, fp32)");
    const int32_t last = n - 1;
    return pgk_engine_prefill_batch(eh, 1, &seq, &n, &start_pos, h_tokens, h_last_logits ? 1 : 0, &last, h_last_logits, s);
}

pgk_status pgk_engine_set_state(pgk_engine eh, const int32_t* h_tokens, const int32_t* h_positions, int batch, pgk_stream s) {
    PGK_REQUIRE(eh && h_tokens && h_positions, "pgk_engine_set_state: null argument");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch, "pgk_engine_set_state: batch %d outside [1,%d]", batch, e->cfg.max_batch);
    for (int b = 0; b < batch; ++b) {
        PGK_REQUIRE(h_tokens[b] >= 0 && h_tokens[b] < e->cfg.vocab_size, "pgk_engine_set_state: token %d out of range", h_tokens[b]);
        PGK_REQUIRE(h_positions[b] >= 0 && h_positions[b] < e->cfg.max_seq_len, "pgk_engine_set_state: position %d outside cache of %d",
                    h_positions[b], e->cfg.max_seq_len);
    }
    if (e->kind->check_state)
        if (pgk_status r = e->kind->check_state(e, h_positions, batch)) return r;
    hipStream_t st = resolve_stream(s);
    e->pos_hi = 0;
    for (int b = 0; b < batch; ++b) e->pos_hi = h_positions[b] > e->pos_hi ? h_positions[b] : e->pos_hi;
    PGK_CHECK_HIP(hipMemcpyAsync(e->tokens, h_tokens, (size_t)batch * 4, hipMemcpyHostToDevice, st));
    PGK_CHECK_HIP(hipMemcpyAsync(e->positions, h_positions, (size_t)batch * 4, hipMemcpyHostToDevice, st));
    // the residual stream enters a step already holding the embeddings of the state tokens
    if (pgk_status r = e->kind->embed_state(e, batch, st)) return r;
    PGK_CHECK_HIP(hipStreamSynchronize(st));
    return PGK_OK;
}

pgk_status pgk_engine_decode_step(pgk_engine eh, int batch, pgk_stream s) {
    PGK_REQUIRE(eh, "pgk_engine_decode_step: null engine");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch, "pgk_engine_decode_step: batch %d outside [1,%d]", batch, e->cfg.max_batch);
    int launches = 0;
    e->step_span = span_for(e);
    pgk_status r = e->kind->decode_step(e, batch, resolve_stream(s), &launches, step_is_short(e, batch));
    e->launches_per_step = launches;
    if (e->pos_hi >= 0) ++e->pos_hi;
    if (r == PGK_OK && e->kind->advance) e->kind->advance(e, batch, 1);
    return r;
}

pgk_status pgk_engine_profile_step(pgk_engine eh, int batch, int n_iters, float* h_ms_sum, int* h_count, pgk_stream s) {
    PGK_REQUIRE(eh && h_ms_sum && h_count, "pgk_engine_profile_step: null argument");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch && n_iters >= 1, "pgk_engine_profile_step: bad arguments");
    hipStream_t st = resolve_stream(s);
    for (int i = 0; i < KC_COUNT; ++i) { h_ms_sum[i] = 0.f; h_count[i] = 0; }
    // Eager steps whose every launch carries its own start / stop event (hipExtLaunchKernelGGL): the elapsed time of a
    // pair is the dispatch's begin -> end interval, the quantity rocprofv3 --kernel-trace reports - no launch gap, nothing
    // subtracted.
    Probe probe;
    probe.timing = true;
    pgk_status r = PGK_OK;
    for (int it = 0; it < n_iters && r == PGK_OK; ++it) {
        probe.used = 0;
        probe.info.clear();
        g_probe = &probe;
        int launches = 0;
        e->step_span = span_for(e);
        r = e->kind->decode_step(e, batch, st, &launches, step_is_short(e, batch));
        g_probe = nullptr;
        if (e->pos_hi >= 0) ++e->pos_hi;
        if (r != PGK_OK) break;
        if (e->kind->advance) e->kind->advance(e, batch, 1);
        hipError_t he = hipStreamSynchronize(st);
        if (he != hipSuccess) { r = set_error(PGK_ERR_HIP, "pgk_engine_profile_step: %s", hipGetErrorString(he)); break; }
        for (size_t i = 0; i < probe.used; ++i) {
            float ms = 0.f;
            const int cls = probe.cls[i];
            if (cls >= 0 && cls < KC_COUNT && hipEventElapsedTime(&ms, probe.ev[2 * i], probe.ev[2 * i + 1]) == hipSuccess) {
                h_ms_sum[cls] += ms;
                h_count[cls] += 1;
            }
        }
    }
    for (hipEvent_t ev : probe.ev) (void)hipEventDestroy(ev);
    return r;
}

// Timeline of ONE replayed step (diagnostic): the step is captured into a temporary graph with every kernel's `tl` slot
// set, replayed `warm` times and then once more; per launch the host gets
//   h_out[6 i .. 6 i + 5] = { kernel class (KC_*), workgroups, first start, last start, first end, last end }
// with the four times in ticks of the 100 MHz s_memrealtime counter relative to the step's first start.  The engine's
// own captured graph is left alone; the sequence state advances by warm + 1 real steps.
pgk_status pgk_engine_timeline(pgk_engine eh, int batch, int warm, uint64_t* h_out, int max_launches, int* n_launches, pgk_stream s) {
    PGK_REQUIRE(eh && h_out && n_launches && max_launches >= 1 && warm >= 0, "pgk_engine_timeline: bad arguments");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch, "pgk_engine_timeline: batch %d outside [1,%d]", batch, e->cfg.max_batch);
    hipStream_t st = resolve_stream(s);
    const int cap = 16 * e->cfg.num_layers + 64;
    Probe probe;
    probe.tl_cap = cap;
    const size_t bytes = (size_t)cap * TL_MAXWG * 2 * sizeof(unsigned long long);
    if (pgk_status r = pgk_malloc((void**)&probe.tl, bytes)) return r;
    pgk_status r = PGK_OK;
    hipGraph_t g = nullptr;
    hipGraphExec_t ex = nullptr;
    hipError_t he = hipMemsetAsync(probe.tl, 0, bytes, st);
    if (he == hipSuccess) he = hipStreamSynchronize(st);
    if (he == hipSuccess) he = hipStreamBeginCapture(st, hipStreamCaptureModeRelaxed);
    if (he == hipSuccess) {
        g_probe = &probe;
        int launches = 0;
        e->step_span = span_for(e);
        r = e->kind->decode_step(e, batch, st, &launches, step_is_short(e, batch));
        g_probe = nullptr;
        he = hipStreamEndCapture(st, &g);
    }
    if (r == PGK_OK && he == hipSuccess) he = hipGraphInstantiate(&ex, g, nullptr, nullptr, 0);
    for (int i = 0; r == PGK_OK && he == hipSuccess && i <= warm; ++i) he = hipGraphLaunch(ex, st);
    if (e->pos_hi >= 0) e->pos_hi += warm + 1;
    if (e->kind->advance) e->kind->advance(e, batch, warm + 1);
    if (r == PGK_OK && he == hipSuccess) he = hipStreamSynchronize(st);
    const int n = (int)probe.info.size() < cap ? (int)probe.info.size() : cap;
    if (r == PGK_OK && he == hipSuccess) {
        std::vector<unsigned long long> host((size_t)n * TL_MAXWG * 2);
        he = hipMemcpy(host.data(), probe.tl, host.size() * sizeof(unsigned long long), hipMemcpyDeviceToHost);
        if (he == hipSuccess) {
            unsigned long long origin = ~0ull;
            std::vector<unsigned long long> agg((size_t)n * 4);
            for (int i = 0; i < n; ++i) {
                const int nwg = probe.info[i].nwg < TL_MAXWG ? probe.info[i].nwg : TL_MAXWG;
                unsigned long long s0 = ~0ull, s1 = 0, e0 = ~0ull, e1 = 0;
                for (int w = 0; w < nwg; ++w) {
                    const unsigned long long a = host[((size_t)i * TL_MAXWG + w) * 2], b = host[((size_t)i * TL_MAXWG + w) * 2 + 1];
                    if (a == 0 && b == 0) continue;   // slot never written
                    s0 = a < s0 ? a : s0; s1 = a > s1 ? a : s1; e0 = b < e0 ? b : e0; e1 = b > e1 ? b : e1;
                }
                agg[4 * i] = s0; agg[4 * i + 1] = s1; agg[4 * i + 2] = e0; agg[4 * i + 3] = e1;
                if (s0 < origin) origin = s0;
            }
#ifdef PGK_PHASE_STAMPS
            {
                double sum[KC_COUNT][8] = {}, cnt[KC_COUNT][8] = {}, dur[KC_COUNT] = {};
                for (int i = 0; i < n; ++i) {
                    const int cls = probe.info[i].cls, nwg = probe.info[i].nwg;
                    if (cls < 0 || cls >= KC_COUNT || nwg > 256) continue;
                    for (int w = 0; w < nwg; ++w) {
                        const unsigned long long t0 = host[((size_t)i * TL_MAXWG + w) * 2], t1 = host[((size_t)i * TL_MAXWG + w) * 2 + 1];
                        dur[cls] += (double)(t1 - t0);
                        for (int k = 0; k < 8; ++k) {
                            const unsigned long long v = host[((size_t)i * TL_MAXWG + 256 + 4 * w) * 2 + k];
                            if (v) { sum[cls][k] += (double)(v - t0); cnt[cls][k] += 1; }
                        }
                    }
                }
                for (int cls = 0; cls < KC_COUNT; ++cls)
                    for (int k = 0; k < 8; ++k)
                        if (cnt[cls][k] > 0) fprintf(stderr, "phase stamps: class %d phase %d at %.2f us after its workgroup's start (n=%.0f)\n", cls, k, sum[cls][k] / cnt[cls][k] / 100.0, cnt[cls][k]);
            }
#endif
            *n_launches = n < max_launches ? n : max_launches;
            for (int i = 0; i < *n_launches; ++i) {
                h_out[6 * i] = (uint64_t)probe.info[i].cls;
                h_out[6 * i + 1] = (uint64_t)probe.info[i].nwg;
                for (int k = 0; k < 4; ++k) h_out[6 * i + 2 + k] = agg[4 * i] == ~0ull ? 0 : agg[4 * i + k] - origin;
            }
        }
    }
    if (ex) (void)hipGraphExecDestroy(ex);
    if (g) (void)hipGraphDestroy(g);
    (void)pgk_free(probe.tl);
    if (r != PGK_OK) return r;
    if (he != hipSuccess) return set_error(PGK_ERR_HIP, "pgk_engine_timeline: %s", hipGetErrorString(he));
    return PGK_OK;
}

pgk_status pgk_engine_capture(pgk_engine eh, int batch, pgk_stream s) {
    PGK_REQUIRE(eh, "pgk_engine_capture: null engine");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch, "pgk_engine_capture: batch %d outside [1,%d]", batch, e->cfg.max_batch);
    hipStream_t st = resolve_stream(s);
    drop_graphs(e);
    // tier 0: the short-context sequence; then the split-KV sequence once per context tier (1024, 2048, ... positions and the
    // cache length) - needed whenever a context can exceed the short limit (or the short sequences are switched off)
    std::vector<int> spans;
    if (e->short_path) spans.push_back(0);
    if (!e->one_sequence && (!e->short_path || e->cfg.max_seq_len > short_limit(batch))) {
        for (int sp = 1024; sp < e->cfg.max_seq_len; sp *= 2) spans.push_back(sp);
        spans.push_back(e->cfg.max_seq_len);
    }
    for (int span : spans) {
        PGK_CHECK_HIP(hipStreamBeginCapture(st, hipStreamCaptureModeRelaxed));
        int launches = 0;
        e->step_span = span;
        pgk_status r = e->kind->decode_step(e, batch, st, &launches, span == 0);
        hipGraph_t g = nullptr;
        hipError_t he = hipStreamEndCapture(st, &g);
        if (r != PGK_OK) { if (g) (void)hipGraphDestroy(g); drop_graphs(e); return r; }
        if (he != hipSuccess || !g) { drop_graphs(e); return set_error(PGK_ERR_HIP, "pgk_engine_capture: hipStreamEndCapture: %s", hipGetErrorString(he)); }
        Engine::Tier t;
        t.span = span; t.graph = g; t.launches = launches;
        he = hipGraphInstantiate(&t.exec, g, nullptr, nullptr, 0);
        e->tiers.push_back(t);      // owned from here on (drop_graphs)
        if (he != hipSuccess) { drop_graphs(e); return set_error(PGK_ERR_HIP, "pgk_engine_capture: hipGraphInstantiate: %s", hipGetErrorString(he)); }
    }
    e->graph_batch = batch;
    e->launches_per_step = e->tiers[pick_tier(e)].launches;
    return PGK_OK;
}

pgk_status pgk_engine_replay(pgk_engine eh, int n_steps, pgk_stream s) {
    PGK_REQUIRE(eh, "pgk_engine_replay: null engine");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(!e->tiers.empty(), "pgk_engine_replay: no captured graph (call pgk_engine_capture first)");
    hipStream_t st = resolve_stream(s);
    for (int i = 0; i < n_steps; ++i) {
        const auto& t = e->tiers[pick_tier(e)];
        PGK_CHECK_HIP(hipGraphLaunch(t.exec, st));
        e->launches_per_step = t.launches;
        if (e->pos_hi >= 0) ++e->pos_hi;
        if (e->kind->advance) e->kind->advance(e, e->graph_batch, 1);
    }
    return PGK_OK;
}

pgk_status pgk_engine_logits_ptr(pgk_engine eh, void** logits_f32) {
    PGK_REQUIRE(eh && logits_f32, "pgk_engine_logits_ptr: null argument");
    *logits_f32 = ((Engine*)eh)->logits;
    return PGK_OK;
}

pgk_status pgk_engine_read_tokens(pgk_engine eh, int32_t* h_out, int batch, int n_steps, pgk_stream s) {
    PGK_REQUIRE(eh && h_out, "pgk_engine_read_tokens: null argument");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(n_steps >= 0 && n_steps <= e->log_cap, "pgk_engine_read_tokens: %d steps exceed the log capacity %d", n_steps, e->log_cap);
    PGK_REQUIRE(batch >= 1 && batch <= e->cfg.max_batch, "pgk_engine_read_tokens: bad batch %d", batch);
    hipStream_t st = resolve_stream(s);
    // log rows are max_batch wide; return the first `batch` columns, step-major
    std::vector<int32_t> tmp((size_t)n_steps * e->cfg.max_batch);
    if (n_steps) PGK_CHECK_HIP(hipMemcpyAsync(tmp.data(), e->token_log, tmp.size() * 4, hipMemcpyDeviceToHost, st));
    PGK_CHECK_HIP(hipStreamSynchronize(st));
    for (int t = 0; t < n_steps; ++t)
        for (int b = 0; b < batch; ++b) h_out[(size_t)t * batch + b] = tmp[(size_t)t * e->cfg.max_batch + b];
    return PGK_OK;
}

pgk_status pgk_engine_read_clock(pgk_engine eh, uint64_t* h_out, int n_steps, pgk_stream s) {
    PGK_REQUIRE(eh && h_out, "pgk_engine_read_clock: null argument");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(n_steps >= 0 && n_steps <= e->log_cap, "pgk_engine_read_clock: %d steps exceed the log capacity %d", n_steps, e->log_cap);
    hipStream_t st = resolve_stream(s);
    if (n_steps) {
        PGK_CHECK_HIP(hipMemcpyAsync(h_out, e->clk_log, (size_t)n_steps * 16, hipMemcpyDeviceToHost, st));
        PGK_CHECK_HIP(hipStreamSynchronize(st));
    }
    return PGK_OK;
}

// In-graph stochastic sampling.  temperature <= 0 restores greedy argmax.  `h_uniforms` [n_rows][max_batch] floats in
// [0,1) are copied into the device ring: step s of the log uses row s % n_rows.  The sampling node and its arguments
// (ring pointer and length, scratch pointer, temperature, top-k, top-p) are baked into a captured graph, so ANY change
// of them - switching sampling on or off, another temperature / top-k / top-p, another n_rows, a scratch buffer that had
// to grow - drops the engine's captured graph: pgk_engine_replay then fails with "no captured graph" until
// pgk_engine_capture is called again.  A refill with the same n_rows and the same parameters only overwrites the ring's
// contents and keeps the graph.
pgk_status pgk_engine_set_sampling(pgk_engine eh, float temperature, int top_k, float top_p, const float* h_uniforms, int n_rows,
                                   pgk_stream s) {
    PGK_REQUIRE(eh, "pgk_engine_set_sampling: null engine");
    Engine* e = (Engine*)eh;
    hipStream_t st = resolve_stream(s);
    auto drop_graph = [&]() {
        if (!e->tiers.empty()) (void)hipStreamSynchronize(st);
        drop_graphs(e);
    };
    if (temperature <= 0.f) {
        if (e->sample_temperature > 0.f) drop_graph();          // a captured sampling node must not be replayed as "greedy"
        e->sample_temperature = 0.f;
        return PGK_OK;
    }
    PGK_REQUIRE(top_k >= 0 && top_p > 0.f && top_p <= 1.f, "pgk_engine_set_sampling: need top_k >= 0 and 0 < top_p <= 1");
    PGK_REQUIRE(h_uniforms && n_rows >= 1, "pgk_engine_set_sampling: uniforms missing");
    const int B = e->cfg.max_batch;
    bool changed = e->sample_temperature != temperature || e->sample_top_k != top_k || e->sample_top_p != top_p || n_rows != e->u_cap;
    if (n_rows > e->u_alloc_rows) {
        drop_graph();                                           // its nodes hold the old ring pointer
        PGK_CHECK_HIP(hipStreamSynchronize(st));
        if (e->u_ring) pgk_free(e->u_ring);
        e->u_ring = nullptr;
        e->u_alloc_rows = 0;
        if (pgk_status r = pgk_malloc((void**)&e->u_ring, (size_t)n_rows * B * 4)) return r;
        e->u_alloc_rows = n_rows;
    }
    if (!e->sampled) {
        if (pgk_status r = pgk_malloc((void**)&e->sampled, (size_t)B * 4)) return r;
    }
    if (const size_t need = sample_scratch_bytes(B, e->cfg.vocab_size, top_k, top_p); need > e->sample_scratch_cap) {
        drop_graph();
        PGK_CHECK_HIP(hipStreamSynchronize(st));
        if (e->sample_scratch) pgk_free(e->sample_scratch);
        e->sample_scratch = nullptr;
        e->sample_scratch_cap = 0;
        if (pgk_status r = pgk_malloc(&e->sample_scratch, need)) return r;
        e->sample_scratch_cap = need;
    }
    if (changed) drop_graph();
    PGK_CHECK_HIP(hipMemcpyAsync(e->u_ring, h_uniforms, (size_t)n_rows * B * 4, hipMemcpyHostToDevice, st));
    PGK_CHECK_HIP(hipStreamSynchronize(st));
    e->u_cap = n_rows;                                          // ring length = rows queued: row index is step % n_rows
    e->sample_temperature = temperature;
    e->sample_top_k = top_k;
    e->sample_top_p = top_p;
    return PGK_OK;
}

pgk_status pgk_engine_reset_log(pgk_engine eh, pgk_stream s) {
    PGK_REQUIRE(eh, "pgk_engine_reset_log: null engine");
    PGK_CHECK_HIP(hipMemsetAsync(((Engine*)eh)->step_counter, 0, 16, resolve_stream(s)));
    return PGK_OK;
}

pgk_status pgk_engine_kv_ptr(pgk_engine eh, int layer, void** k, void** v) {
    PGK_REQUIRE(eh && k && v, "pgk_engine_kv_ptr: null argument");
    Engine* e = (Engine*)eh;
    PGK_REQUIRE(layer >= 0 && layer < e->cfg.num_layers, "pgk_engine_kv_ptr: layer %d", layer);
    return e->kind->kv_ptr(e, layer, k, v);
}

pgk_status pgk_engine_state_ptr(pgk_engine eh, void** tokens, void** positions) {
    PGK_REQUIRE(eh && tokens && positions, "pgk_engine_state_ptr: null argument");
    *tokens = ((Engine*)eh)->tokens;
    *positions = ((Engine*)eh)->positions;
    return PGK_OK;
}

pgk_status pgk_engine_launches_per_step(pgk_engine eh, int* n) {
    PGK_REQUIRE(eh && n, "pgk_engine_launches_per_step: null argument");
    *n = ((Engine*)eh)->launches_per_step;
    return PGK_OK;
}

}  // extern "C"
