"""Python handle on the native decode/prefill engine (pgk_engine_* in include/pgk_hip.h).

One C call enqueues a whole token step (5 fused kernels per layer); `capture()` records it into ONE
hipGraph whose token id / position live in device memory, so `replay(n)` runs n greedy steps with no
host round trip.  This is what DecodeM1Graph / DecodeBatch drive; the reference's counterpart is the
2L+2-graph replay loop of src/pygpukit/llm/decode/m1_graph.py:463-589."""

from __future__ import annotations

import ctypes as C

import numpy as np

from pygpukit_amd import _hip
from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32, int32
from pygpukit_amd.core.factory import from_numpy, zeros
from pygpukit_amd.llm.config import LoopConfig
from pygpukit_amd.ops.tensor import concat_axis0, pad_2d


class Engine:
    def __init__(self, config: dict, embed: GPUArray, layers: list[dict], final_norm: GPUArray, lm_head: GPUArray | None = None,
                 *, max_seq_len: int = 512, max_batch: int = 1, weight_format: str = "bf16", use_qk_norm: bool = True):
        """config: vocab_size, hidden_size, num_layers, num_heads, num_kv_heads, head_dim, intermediate_size,
        norm_eps, rope_theta.  layers[i]: GPUArrays attn_norm, w_qkv [(Hq+2Hkv)D, H], q_norm, k_norm, w_o,
        mlp_norm, w_gate_up [2I, H], w_down (+ s_qkv, s_o, s_gate_up, s_down for fp8)."""
        _hip.require_device()
        self.config = dict(config)
        self.max_seq_len, self.max_batch = max_seq_len, max_batch
        self.weight_format = weight_format
        self._keep = [embed, final_norm, lm_head, layers]  # keep the weights alive
        mc = _hip.ModelConfig(config["vocab_size"], config["hidden_size"], config["num_layers"], config["num_heads"],
                              config["num_kv_heads"], config["head_dim"], config["intermediate_size"], max_seq_len, max_batch,
                              float(config["norm_eps"]), float(config["rope_theta"]), {"bf16": 0, "fp8": 1, "fp8a8": 2}[weight_format],
                              1 if use_qk_norm else 0)
        for a in (embed, final_norm):
            if a.dtype != bfloat16:
                raise ValueError("Engine: embedding / norm weights must be bfloat16")
        arr = (_hip.LayerWeights * len(layers))()
        for i, lw in enumerate(layers):
            for name, _ in _hip.LayerWeights._fields_:
                t = lw.get(name)
                setattr(arr[i], name, t.data_ptr() if t is not None else None)
        h = C.c_void_p()
        _hip.call("pgk_engine_create", C.byref(mc), embed._p, lm_head._p if lm_head is not None else None, final_norm._p,
                  arr, C.byref(h))
        self._h = h.value
        self._captured_batch = 0
        self.last_prefill_logits: np.ndarray | None = None

    def __del__(self):
        try:
            if getattr(self, "_h", 0):
                _hip.call("pgk_engine_destroy", C.c_void_p(self._h))
        except Exception:
            pass
        self._h = 0

    @property
    def handle(self) -> C.c_void_p:
        return C.c_void_p(self._h)

    def bytes(self) -> tuple[int, int]:
        kv, ws = C.c_size_t(), C.c_size_t()
        _hip.call("pgk_engine_bytes", self.handle, C.byref(kv), C.byref(ws))
        return kv.value, ws.value

    # ------------------------------------------------------------------ prefill
    def prefill(self, tokens, seq: int = 0, start_pos: int = 0, *, want_last_logits: bool = True,
                all_logits: GPUArray | None = None) -> np.ndarray | None:
        """Run the prompt through the MFMA path, filling sequence slot `seq`'s KV rows; returns the last
        row's logits (fp32 [V]) when asked.  all_logits: optional bf16 [n, V] device buffer."""
        toks = np.ascontiguousarray(tokens, dtype=np.int32)
        out = np.empty(self.config["vocab_size"], np.float32) if want_last_logits else None
        _hip.call("pgk_engine_prefill", self.handle, seq, toks.ctypes.data_as(_hip.c_i32_p), len(toks), start_pos,
                  all_logits._p if all_logits is not None else None,
                  out.ctypes.data_as(C.POINTER(C.c_float)) if out is not None else None, None)
        if out is not None:
            self.last_prefill_logits = out
        return out

    def prefill_batch(self, prompts, slots=None, starts=None, *, want=None) -> np.ndarray:
        """Several sequences in one call: prompts[i] goes to slot slots[i] (default i) from position starts[i] (default 0).  Returns the
        fp32 logits [n, V] of every sequence's last row, or with `want` (one ascending list of row indices per sequence; layer-list
        engines only) of exactly those rows, sequence by sequence."""
        lens = np.asarray([len(p) for p in prompts], np.int32)
        if lens.size == 0 or (lens < 1).any():
            raise ValueError("prefill_batch: every prompt needs at least one token")
        slots = np.asarray(range(len(prompts)) if slots is None else slots, np.int32)
        starts = np.zeros(len(prompts), np.int32) if starts is None else np.asarray(starts, np.int32)
        if len(slots) != len(prompts) or len(starts) != len(prompts) or (want is not None and len(want) != len(prompts)):
            raise ValueError("prefill_batch: prompts, slots, starts and want must have the same length")
        first = np.concatenate([[0], np.cumsum(lens)[:-1]])
        rows = [[n - 1] for n in lens] if want is None else want
        for n, r in zip(lens, rows):
            if any(not 0 <= i < n for i in r):
                raise ValueError("prefill_batch: wanted row outside its prompt")
        w = np.asarray([f + i for f, r in zip(first, rows) for i in r], np.int32)
        toks = np.ascontiguousarray(np.concatenate([np.asarray(p, np.int32) for p in prompts]))
        out = np.empty((len(w), self.config["vocab_size"]), np.float32)
        i32 = lambda a: a.ctypes.data_as(_hip.c_i32_p)  # noqa: E731
        _hip.call("pgk_engine_prefill_batch", self.handle, len(prompts), i32(slots), i32(lens), i32(starts), i32(toks), len(w),
                  i32(w) if len(w) else None, out.ctypes.data_as(C.POINTER(C.c_float)) if len(w) else None, None)
        return out

    # ------------------------------------------------------------------ decode
    def set_state(self, tokens, positions) -> None:
        t = np.ascontiguousarray(tokens, dtype=np.int32)
        p = np.ascontiguousarray(positions, dtype=np.int32)
        if len(t) != len(p):
            raise ValueError("set_state: tokens and positions must have the same length")
        _hip.call("pgk_engine_set_state", self.handle, t.ctypes.data_as(_hip.c_i32_p), p.ctypes.data_as(_hip.c_i32_p), len(t), None)

    def set_sampling(self, temperature: float, top_k: int = 0, top_p: float = 1.0, uniforms: np.ndarray | None = None,
                     n_steps: int = 256, seed: int | None = None) -> np.ndarray | None:
        """Switch the decode step from greedy argmax to a temperature / top-k / top-p draw made inside the step (and so
        inside a captured graph).  `uniforms` [n_steps, max_batch] float32 in [0,1) (drawn from `seed` when omitted) are
        queued on the device: step s uses row s % n_steps.  Returns the uniforms used (None when switching back to
        greedy with temperature <= 0).  Call before capture().  Calling again with the same parameters and the same
        number of rows only queues fresh uniforms; any other change (on/off, temperature, top_k, top_p, row count)
        drops the captured graph - capture() again before replay()."""
        key = (0.0,) if temperature <= 0 else (float(temperature), int(top_k), float(top_p),
                                                int(uniforms.shape[0]) if uniforms is not None else int(n_steps))
        if key != getattr(self, "_sampling_key", (0.0,)):
            self._captured_batch = 0
        self._sampling_key = key
        if temperature <= 0:
            _hip.call("pgk_engine_set_sampling", self.handle, C.c_float(0.0), 0, C.c_float(1.0), None, 0, None)
            return None
        if uniforms is None:
            uniforms = np.random.default_rng(seed).random((n_steps, self.max_batch), dtype=np.float32)
        u = np.ascontiguousarray(uniforms, dtype=np.float32)
        if u.ndim != 2 or u.shape[1] != self.max_batch:
            raise ValueError(f"set_sampling: uniforms must be [n_steps, {self.max_batch}]")
        _hip.call("pgk_engine_set_sampling", self.handle, C.c_float(temperature), int(top_k), C.c_float(top_p),
                  u.ctypes.data_as(C.POINTER(C.c_float)), u.shape[0], None)
        return u

    def decode_step(self, batch: int = 1) -> None:
        """Enqueue one eager (un-captured) step."""
        _hip.call("pgk_engine_decode_step", self.handle, batch, None)

    KERNEL_CLASSES = ("embed", "norm_qkv", "attn", "oproj", "gateup", "down", "lmhead", "argmax", "recur")

    def profile_step(self, batch: int = 1, n_iters: int = 8) -> dict:
        """Eager steps, every launch bracketed by its own start/stop event (the dispatch's begin -> end interval, what
        rocprofv3 --kernel-trace reports) -> {class: (avg_us_per_launch, launches_per_step)}."""
        ms = (C.c_float * len(self.KERNEL_CLASSES))()
        cnt = (C.c_int * len(self.KERNEL_CLASSES))()
        _hip.call("pgk_engine_profile_step", self.handle, batch, n_iters, ms, cnt, None)
        return {name: ((ms[i] * 1e3 / cnt[i]) if cnt[i] else 0.0, cnt[i] // n_iters) for i, name in enumerate(self.KERNEL_CLASSES)
                if cnt[i] or name != "recur"}      # (recur: layer-list models only)

    def timeline(self, batch: int = 1, warm: int = 2) -> list[dict]:
        """One graph-replayed step as a list of launches in order: kernel class, workgroups, and the first/last start and
        first/last end over the launch's workgroups in microseconds from the step's first start (in-kernel
        s_memrealtime stamps; diagnostic capture, the engine's own graph is untouched)."""
        cap = 16 * self.config["num_layers"] + 64
        buf = (C.c_uint64 * (6 * cap))()
        n = C.c_int()
        _hip.call("pgk_engine_timeline", self.handle, batch, warm, buf, cap, C.byref(n), None)
        out = []
        for i in range(n.value):
            cls, nwg, s0, s1, e0, e1 = (int(buf[6 * i + k]) for k in range(6))
            out.append({"kernel": self.KERNEL_CLASSES[cls] if 0 <= cls < len(self.KERNEL_CLASSES) else str(cls), "workgroups": nwg,
                        "first_start_us": s0 / 100.0, "last_start_us": s1 / 100.0, "first_end_us": e0 / 100.0, "last_end_us": e1 / 100.0})
        return out

    def capture(self, batch: int = 1) -> None:
        _hip.call("pgk_engine_capture", self.handle, batch, None)
        self._captured_batch = batch

    def replay(self, n_steps: int = 1) -> None:
        _hip.call("pgk_engine_replay", self.handle, n_steps, None)

    def synchronize(self) -> None:
        _hip.call("pgk_stream_sync", None)

    def reset_log(self) -> None:
        _hip.call("pgk_engine_reset_log", self.handle, None)

    def read_tokens(self, batch: int, n_steps: int) -> np.ndarray:
        out = np.empty((n_steps, batch), np.int32)
        _hip.call("pgk_engine_read_tokens", self.handle, out.ctypes.data_as(_hip.c_i32_p), batch, n_steps, None)
        return out

    def shader_clock_mhz(self, n_steps: int) -> float:
        """In-kernel shader clock over the last n_steps logged steps: d(s_memtime)/d(s_memrealtime) x 100 MHz."""
        buf = np.zeros(2 * n_steps, np.uint64)
        _hip.call("pgk_engine_read_clock", self.handle, buf.ctypes.data_as(C.POINTER(C.c_uint64)), n_steps, None)
        t, r = buf[0::2].astype(np.float64), buf[1::2].astype(np.float64)
        if n_steps < 2 or r[-1] == r[0]:
            return 0.0
        return float((t[-1] - t[0]) / (r[-1] - r[0]) * 100.0)

    def logits(self, batch: int = 1) -> GPUArray:
        """fp32 [batch, V] view of the last step's logits (owned by the engine)."""
        p = C.c_void_p()
        _hip.call("pgk_engine_logits_ptr", self.handle, C.byref(p))
        a = GPUArray((batch, self.config["vocab_size"]), float32, p.value, owns_memory=False)
        a._source_ref = self
        return a

    def kv_cache(self, layer: int) -> tuple[GPUArray, GPUArray]:
        """bf16 [max_batch, Hkv, max_seq, D] views of layer `layer`'s K and V caches."""
        k, v = C.c_void_p(), C.c_void_p()
        _hip.call("pgk_engine_kv_ptr", self.handle, layer, C.byref(k), C.byref(v))
        shape = (self.max_batch, self.config["num_kv_heads"], self.max_seq_len, self.config["head_dim"])
        ka, va = GPUArray(shape, bfloat16, k.value, owns_memory=False), GPUArray(shape, bfloat16, v.value, owns_memory=False)
        ka._source_ref = va._source_ref = self
        return ka, va

    def state_arrays(self, batch: int) -> tuple[GPUArray, GPUArray]:
        """int32 [batch] views of the device-resident (token, position) state."""
        from pygpukit_amd.core.dtypes import int32

        t, p = C.c_void_p(), C.c_void_p()
        _hip.call("pgk_engine_state_ptr", self.handle, C.byref(t), C.byref(p))
        ta, pa = GPUArray((batch,), int32, t.value, owns_memory=False), GPUArray((batch,), int32, p.value, owns_memory=False)
        ta._source_ref = pa._source_ref = self
        return ta, pa

    def launches_per_step(self) -> int:
        n = C.c_int()
        _hip.call("pgk_engine_launches_per_step", self.handle, C.byref(n))
        return n.value

    # ------------------------------------------------------------------ convenience
    def generate_greedy(self, prompt, max_new_tokens: int, *, use_graph: bool = True) -> list[int]:
        """Prompt + max_new_tokens greedy tokens for one sequence (slot 0): prefill, argmax of the last
        row (lowest index on ties), then max_new_tokens-1 device-resident decode steps."""
        prompt = [int(t) for t in prompt]
        logits = self.prefill(prompt, seq=0, start_pos=0)
        first = int(np.argmax(logits))
        out = prompt + [first]
        n = max_new_tokens - 1
        if n <= 0:
            return out[: len(prompt) + max_new_tokens]
        self.set_state([first], [len(prompt)])
        self.reset_log()
        if use_graph:
            if self._captured_batch != 1:
                self.capture(1)
            self.replay(n)
        else:
            for _ in range(n):
                self.decode_step(1)
        self.synchronize()
        return out + [int(t) for t in self.read_tokens(1, n)[:, 0]]

    def generate(self, prompt, max_new_tokens: int, temperature: float = 1.0, top_k: int = 50, top_p: float = 0.9, *,
                 seed: int | None = None) -> list[int]:
        """CausalTransformerModel.generate's sampling semantics (causal.py:179-255) with every draw made on the device:
        the first token from the prefill logits (ops.sample_token_gpu semantics via the oracle-restated sampler), the
        rest inside the captured decode graph (set_sampling).  temperature == 0 is generate_greedy."""
        if temperature == 0:
            return self.generate_greedy(prompt, max_new_tokens)
        from pygpukit_amd.core.factory import from_numpy
        from pygpukit_amd.ops.sampling import sample_token_gpu

        prompt = [int(t) for t in prompt]
        rng = np.random.default_rng(seed)
        logits = self.prefill(prompt, seq=0, start_pos=0)
        first = sample_token_gpu(from_numpy(np.ascontiguousarray(logits, dtype=np.float32)), temperature, top_k, top_p,
                                 u=float(rng.random(dtype=np.float32)))
        out = prompt + [first]
        n = max_new_tokens - 1
        if n <= 0:
            return out[: len(prompt) + max_new_tokens]
        self.reset_log()
        u = np.zeros((n, self.max_batch), np.float32)
        u[:, 0] = rng.random(n, dtype=np.float32)
        self.set_sampling(temperature, top_k, top_p, uniforms=u)
        self.set_state([first], [len(prompt)])
        self.capture(1)            # the sampling node is part of the graph
        self.replay(n)
        self.synchronize()
        toks = [int(t) for t in self.read_tokens(1, n)[:, 0]]
        self.set_sampling(0.0)
        self._captured_batch = None
        return out + toks


NO_WINDOW = 2**30


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def _up64(n: int) -> int:
    return _up(n, 64)


def _attention_pad(dim: int, vdim: int) -> int:
    """Head width the attention kernels run at: 64, 128 or a larger multiple of 64."""
    m = max(dim, vdim)
    return 64 if m <= 64 else 128 if m <= 128 else _up64(m)


def _head_rows(w: GPUArray, heads: int, per_head: int, pad: int, cols: int) -> GPUArray:
    """[heads * per_head, c] -> [heads * pad, cols]"""
    c = w.shape[1]
    return pad_2d(pad_2d(w.view((heads, per_head * c)), heads, pad * c).view((heads * pad, c)), heads * pad, cols)


def _head_cols(w: GPUArray, heads: int, per_head: int, pad: int, rows: int, cols: int) -> GPUArray:
    """[r, heads * per_head] -> [rows, cols], heads pad columns apart"""
    r = w.shape[0]
    return pad_2d(pad_2d(w.view((r * heads, per_head)), r * heads, pad).view((r, heads * pad)), rows, cols)


def _stack_rows(parts: list[GPUArray]) -> GPUArray:
    """Matrices of one width below each other, zero rows up to a multiple of 64."""
    cols = parts[0].shape[1]
    out = zeros((_up64(sum(w.shape[0] for w in parts)), cols), parts[0].dtype)
    at = 0
    for w in parts:
        _hip.call("pgk_memcpy_d2d", C.c_void_p(out.data_ptr() + at * cols * w.itemsize), w._p, w.nbytes, None)
        at += w.shape[0]
    return out


def _row(w: GPUArray, n: int) -> GPUArray:
    return pad_2d(w.view((1, w.size)), 1, n)


def _host_f32(a: GPUArray) -> np.ndarray:
    h = a.to_numpy()
    return (h.astype(np.uint32) << 16).view(np.float32) if a.dtype == bfloat16 else h.astype(np.float32)


def _pad_heads(v: np.ndarray, heads: int, pad: int, fill: float = 0.0) -> np.ndarray:
    """[..., heads * d] -> [..., heads * pad]"""
    d = v.shape[-1] // heads
    out = np.full((*v.shape[:-1], heads, pad), fill, np.float32)
    out[..., :d] = v.reshape(*v.shape[:-1], heads, d)
    return out.reshape(*v.shape[:-1], heads * pad)


def _pad_taps(taps: tuple[GPUArray, ...], heads: tuple[tuple[int, int], ...]) -> GPUArray:
    """[taps, heads * d] each -> one [taps, all padded channels]"""
    c = np.ascontiguousarray(np.concatenate([_pad_heads(_host_f32(t), h, p) for t, (h, p) in zip(taps, heads)], axis=1))
    return from_numpy((c.view(np.uint32) >> 16).astype(np.uint16) if taps[0].dtype == bfloat16 else c)      # (bfloat16 values: the upper halves are exact)


class StackEngine(Engine):
    """The native engine for layer-list models (csrc/engine_stack.hip): fp32 residual stream, sandwich layers (a norm after each sublayer
    and optionally before it) parallel ones (one norm, mixer beside experts) or hyper-connected ones (several streams), a mixer per layer (latent attention, attention
    over a K/V ring, with mixed scores or without, linear recurrences, gated delta rule), every layer with its own sizes, possibly a stretch of layers that runs several
    times.  State, graphs, sampling and generation are Engine's.

    The cache of an attention layer is a ring of min(window or chunk, max_seq_len) rows per sequence slot, that of a recurrent one a state: a
    sequence goes on where it stopped (or starts again at position 0); a position whose window or state has been overwritten is refused."""

    _SIZES = ("mixer", "ff", "heads", "kv_heads", "dim", "vdim", "rank", "window", "taps", "kv_from", "head_pad", "vhead_pad", "rank_pad", "n_att", "ff_pad")
    _MORE = dict(gated=0, rot=0, norm_parts=1, rank_a=0, rank_g=0, experts=0, top=0, groups=0, keep=0, chunked=0, ff_dim=0, shared_pad=0)       # sizes of some layers, and their defaults

    def __init__(self, config: dict, embed: GPUArray, position_embed: GPUArray | None, head: GPUArray, final_norm: GPUArray, layers: list[dict], *,
                 max_seq_len: int = 512, max_batch: int = 1):
        """config: vocab_size, width, max_positions, norm_eps, residual_mult; for parallel layers block and layer_norm, with a loop `loop`
        (start, stop, times) and its arrays loop_in [wp, 2 wp], loop_step [times, wp]; for hyper-connected ones block, streams, norm_groups,
        logit_cap.  layers[i]: the sizes and packed arrays of pack_layer(), pack_attention(), pack_recurrence(), pack_delta(),
        pack_state_space() or pack_talking()."""
        _hip.require_device()
        dt = embed.dtype
        if dt not in (bfloat16, float32):
            raise NotImplementedError("the layer-list engine runs in bfloat16 or float32")
        self.config = dict(config, num_layers=len(layers))
        self.layers = layers
        self.max_seq_len, self.max_batch, self.dtype = max_seq_len, max_batch, dt
        self.weight_format = str(dt)
        self._keep = [embed, position_embed, head, final_norm, layers]
        wp = _up64(config["width"])
        if head.shape != (config["vocab_size"], wp) or final_norm.shape != (1, wp) or final_norm.dtype != float32 or embed.shape != (config["vocab_size"], config["width"]):
            raise ValueError("StackEngine: embedding / head / final norm shapes do not match the configuration")
        if position_embed is not None and position_embed.shape != (config["max_positions"], config["width"]):
            raise ValueError(f"StackEngine: position table {position_embed.shape}")
        block, loop = config.get("block", _hip.BLOCK_SANDWICH), config.get("loop")
        parallel, hyper, streams = block == _hip.BLOCK_PARALLEL, block == _hip.BLOCK_HYPER, config.get("streams", 1)
        self._runs = [i for i, _ in LoopConfig(*loop).runs(len(layers))] if loop else list(range(len(layers)))
        arr = (_hip.StackLayer * len(layers))()
        for i, lw in enumerate(layers):
            hd, gd = lw["heads"] * lw["head_pad"], 0 if lw["kv_from"] >= 0 else lw["kv_heads"] * lw["head_pad"]
            moe, E = lw["ff_pad"] and lw["ff"] == _hip.FF_MOE, lw.get("experts", 0)
            ff, rp, n_att, n_in = lw["ff_pad"], lw["rank_pad"], lw["n_att"], lw["w_in"].shape[0] - (_up64(E) if moe else 0)
            up, table = 2 * ff if lw["ff"] == _hip.FF_SWIGLU else ff, ff and lw["ff"] == _hip.FF_TABLE
            # name -> (shape, dtype, may be absent)
            want = {"norm1": ((1, wp), float32, not parallel and not hyper), "norm1b": ((1, wp), float32, parallel or hyper), "w_in": ((n_in + (_up64(E) if moe else 0), wp), dt, False),
                    "w_o": ((wp, n_att), dt, False), "b_in": ((1, n_in), float32, True)}
            if moe:
                want.update(w_gate_up=((E, 2 * ff, wp), dt, False), w_down=((E, wp, ff), dt, False), correction=((E,), float32, False))
            elif table:
                sp = lw["shared_pad"]
                want.update(w_gate_up=((E, ff, wp), dt, False), w_down=((E, wp, ff), dt, False), table=((config["vocab_size"], lw["top"]), int32, False),
                            w_shared_up=((sp, wp), dt, not sp), w_shared_down=((wp, sp), dt, not sp), w_shared_gate=((1, wp), dt, not sp))
            elif ff and hyper:
                want.update(w_gate_up=((ff, wp), dt, False), w_down=((wp, ff), dt, False), act=((4,), float32, False))
            elif ff:
                want.update(norm2=((1, wp), float32, True), norm2b=((1, wp), float32, False), w_gate_up=((up, wp), dt, False), w_down=((wp, ff), dt, False))
            if hyper:
                want.update(hyper1=((streams * (streams + 2),), float32, False), hyper2=((streams * (streams + 2),), float32, not ff), norm2=((1, wp), float32, not ff))
            if lw["mixer"] == _hip.MIX_TALK:
                hp = lw["head_pad"]
                want.update(q_norm=((1, hp), float32, False), k_norm=((1, hp), float32, lw["kv_from"] >= 0), rot_freq=((lw["rot"] // 2,), float32, not lw["rot"]),
                            talk=((lw["heads"], lw["heads"]), float32, True), sink=((lw["heads"],), float32, True), b_o=((1, wp), float32, True))
            elif lw["mixer"] == _hip.MIX_LATENT:
                want.update(c_norm=((1, rp), float32, False), w_ukv=((2 * hd, rp), dt, False), rot_freq=((lw.get("rot", 0) // 2,), float32, not lw.get("rot", 0)))
            elif lw["mixer"] in (_hip.MIX_DELTA, _hip.MIX_SSD):
                delta, hv = lw["mixer"] == _hip.MIX_DELTA, lw["heads"] * lw["vhead_pad"]
                want.update(conv=((lw["taps"], hv + 2 * gd), dt, False), conv_bias=((1, hv + 2 * gd), float32, delta), decay=((lw["heads"],), float32, False),
                            dt_bias=((1, hd if delta else lw["heads"]), float32, False), skip=((1, lw["heads"]), float32, delta),
                            o_norm=((1, lw["vhead_pad"] if delta else hv), float32, False), w_a2=((hd, lw.get("rank_a", 0)), dt, not delta),
                            w_g2=((hv, lw.get("rank_g", 0)), dt, not delta))
            elif lw["mixer"] == _hip.MIX_ATTENTION:
                want.update(conv=((lw["taps"], hd + 2 * gd), dt, True), q_norm=((1, hd), float32, True), k_norm=((1, gd), float32, True),
                            slopes=((1, lw["heads"]), float32, True))
            else:
                want.update(lower=((1, hd), float32, False), o_norm=((1, lw["vhead_pad"]), float32, False))
            for name, (shape, dtype, optional) in want.items():
                t = lw.get(name)
                if t is None and optional:
                    continue
                if t is None or t.shape != shape or t.dtype != dtype:
                    raise ValueError(f"StackEngine: layer {i}: {name} must be {dtype} {shape}, got {None if t is None else (t.dtype, t.shape)}")
                setattr(arr[i], name, t.data_ptr())
            for name in self._SIZES:
                setattr(arr[i], name, lw[name])
            for name, default in self._MORE.items():
                setattr(arr[i], name, lw.get(name, default))
            arr[i].n_in, arr[i].scale, arr[i].router_scale = n_in, lw["scale"], lw.get("router_scale", 1.0)
            arr[i].act_pos, arr[i].act_neg = lw.get("act_params", (0.0, 0.0))
        sc = _hip.StackConfig(config["vocab_size"], config["width"], len(layers), config["max_positions"], max_seq_len, max_batch, config["norm_eps"],
                              config["residual_mult"], dt.code, block, int(config.get("layer_norm", 0)))
        sc.streams, sc.norm_groups, sc.logit_cap = streams, config.get("norm_groups", 1), config.get("logit_cap") or 0.0
        if loop:
            lin, step = config["loop_in"], config["loop_step"]
            if lin.shape != (wp, 2 * wp) or lin.dtype != dt or step.shape != (loop[2], wp) or step.dtype != float32:
                raise ValueError(f"StackEngine: loop input {lin.shape}, steps {step.shape}")
            self._keep += [lin, step]
            sc.loop_start, sc.loop_stop, sc.loop_times, sc.loop_in, sc.loop_step = *loop, lin.data_ptr(), step.data_ptr()
        h = C.c_void_p()
        _hip.call("pgk_engine_create_stack", C.byref(sc), embed._p, position_embed._p if position_embed is not None else None, head._p, final_norm._p,
                  arr, C.byref(h))
        self._h = h.value
        self._captured_batch = 0
        self.last_prefill_logits = None

    @staticmethod
    def _pack_common(width: int, norm1: GPUArray | None, norm1b: GPUArray | None, gate_up: GPUArray | None, down: GPUArray | None, norm2: GPUArray | None,
                     norm2b: GPUArray | None, act_params: tuple[float, float] | None) -> dict:
        """Norms and feed-forward of a layer.  gate_up: the SwiGLU matrix [2 ff, width], or with act_params (xIELU's two factors)
        the up-projection [ff, width]."""
        wp = _up64(width)
        out = dict(norm1=None if norm1 is None else _row(norm1, wp), norm1b=None if norm1b is None else _row(norm1b, wp), ff_pad=0, ff=_hip.FF_SWIGLU if act_params is None else _hip.FF_XIELU,
                   rank=0, rank_pad=0, kv_from=-1, taps=1, window=NO_WINDOW, scale=1.0)
        if act_params is not None:
            out["act_params"] = act_params
        if gate_up is not None:
            ff = down.shape[1]
            fp = _up64(ff)
            if act_params is not None:
                gate_up = pad_2d(gate_up, fp, wp)
            elif (ff, width) != (fp, wp):
                gate_up = concat_axis0(pad_2d(gate_up._view(0, (ff, width)), fp, wp), pad_2d(gate_up._view(ff * width, (ff, width)), fp, wp))
            out.update(ff_pad=fp, w_gate_up=gate_up, w_down=pad_2d(down, wp, fp), norm2=None if norm2 is None else _row(norm2, wp), norm2b=_row(norm2b, wp))
        return out

    @classmethod
    def pack_layer(cls, q: GPUArray, kv_down: GPUArray, head_gate: GPUArray | None, kv_norm: GPUArray, k_up: GPUArray, v_up: GPUArray, o: GPUArray, norm1: GPUArray,
                   norm1b: GPUArray | None, *, rot_freq: GPUArray | None = None, heads: int, dim: int, vdim: int, window: int, scale: float, gate_up: GPUArray | None = None,
                   down: GPUArray | None = None, norm2: GPUArray | None = None, norm2b: GPUArray | None = None,
                   act_params: tuple[float, float] | None = None) -> dict:
        """One latent-attention layer's matrices ([out, in]; norms fp32 with offsets applied) -> the engine's padded layout: head widths to
        64 / 128 / a multiple of 64, every other width to a multiple of 64.  Arrays that already fit are used as they are.  rot_freq [rot / 2]:
        the last rot of the dim query columns, and of kv_down's rows, are the rotated part (k_up and v_up take all of a cached row)."""
        rot = 0 if rot_freq is None else 2 * rot_freq.size
        width, rank = q.shape[1], kv_down.shape[0] - rot
        wp, rp, hp = _up64(width), _up64(rank + rot), _attention_pad(dim, vdim)
        hd = heads * hp
        out = cls._pack_common(width, norm1, norm1b, gate_up, down, norm2, norm2b, act_params)
        out.update(mixer=_hip.MIX_LATENT, heads=heads, kv_heads=heads, dim=dim, vdim=vdim, rank=rank, window=window, scale=scale, head_pad=hp, vhead_pad=hp, rank_pad=rp,
                   gated=int(head_gate is not None), rot=rot, rot_freq=rot_freq, n_att=hd,
                   w_in=_stack_rows([_head_rows(q, heads, dim, hp, wp), pad_2d(kv_down, rp, wp)] + ([] if head_gate is None else [pad_2d(head_gate, heads, wp)])), c_norm=_row(kv_norm, rp),
                   w_ukv=concat_axis0(_head_rows(k_up, heads, dim, hp, rp), _head_rows(v_up, heads, vdim, hp, rp)), w_o=_head_cols(o, heads, vdim, hp, wp, hd))
        return out

    @classmethod
    def pack_attention(cls, q: GPUArray, k: GPUArray | None, v: GPUArray | None, gate: GPUArray, o: GPUArray, norm1: GPUArray | None, norm1b: GPUArray, *, heads: int,
                       kv_heads: int, dim: int, vdim: int, window: int, scale: float, biases: tuple = (None, None, None), convs: tuple = (None, None, None),
                       q_norm: GPUArray | None = None, k_norm: GPUArray | None = None, slopes: GPUArray | None = None, kv_from: int | None = None,
                       gate_up: GPUArray | None = None, down: GPUArray | None = None, norm2: GPUArray | None = None, norm2b: GPUArray | None = None,
                       act_params: tuple[float, float] | None = None) -> dict:
        """One layer of attention over a K/V ring: q, k, v, gate, o [out, in]; biases and convs ([channels, taps]) of q, k, v; norms of the
        whole q and k rows; slopes [heads]; kv_from: the layer whose keys and values it takes (k, v are None then)."""
        width = q.shape[1]
        wp, hp = _up64(width), _attention_pad(dim, vdim)
        parts = [(q, heads, dim)] + ([] if kv_from is not None else [(k, kv_heads, dim), (v, kv_heads, vdim)])
        mats = [_head_rows(w, n, d, hp, wp) for w, n, d in parts] + [_head_rows(gate, heads, vdim, hp, wp)]
        w_in = _stack_rows(mats)
        out = cls._pack_common(width, norm1, norm1b, gate_up, down, norm2, norm2b, act_params)
        rows = sum(m.shape[0] for m in mats[:-1])

        def channels(arrays: tuple) -> np.ndarray:        # [..., channels] of q (, k, v) -> padded heads side by side
            return np.concatenate([_pad_heads(_host_f32(a).T, n, hp) for a, (_, n, _) in zip(arrays, parts)], axis=-1)

        b_in = conv = None
        if biases[0] is not None:
            b = np.zeros((1, w_in.shape[0]), np.float32)
            b[0, :rows] = channels(biases)
            b_in = from_numpy(b)
        if convs[0] is not None:
            c = np.ascontiguousarray(channels(convs))          # (bfloat16 values: the upper halves are exact)
            conv = from_numpy((c.view(np.uint32) >> 16).astype(np.uint16) if q.dtype == bfloat16 else c)
        vec = lambda a, n: None if a is None else from_numpy(_pad_heads(_host_f32(a).reshape(1, -1), n, hp))  # noqa: E731
        out.update(mixer=_hip.MIX_ATTENTION, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=window, scale=scale, head_pad=hp, vhead_pad=hp, n_att=heads * hp,
                   kv_from=-1 if kv_from is None else kv_from, taps=1 if conv is None else conv.shape[0], w_in=w_in, b_in=b_in, conv=conv, q_norm=vec(q_norm, heads),
                   k_norm=None if kv_from is not None else vec(k_norm, kv_heads), slopes=None if slopes is None else slopes.view((1, heads)),
                   w_o=_head_cols(o, heads, vdim, hp, wp, heads * hp))
        return out

    @classmethod
    def pack_recurrence(cls, q: GPUArray, forget: GPUArray, v: GPUArray, o: GPUArray, forget_bias: GPUArray, lower: GPUArray, head_norm: GPUArray,
                        norm1: GPUArray | None, norm1b: GPUArray, *, heads: int, dim: int, vdim: int, gate_up: GPUArray | None = None, down: GPUArray | None = None,
                        norm2: GPUArray | None = None, norm2b: GPUArray | None = None, act_params: tuple[float, float] | None = None) -> dict:
        """One gated-recurrence layer: q, forget, v, o [out, in]; forget_bias, lower and head_norm fp32.  Padding channels keep an empty
        state: their lower bound is 1, so nothing is written."""
        width = q.shape[1]
        wp, dp, vp = _up64(width), _up(dim, 16), _up(vdim, 16)
        w_in = _stack_rows([_head_rows(q, heads, dim, dp, wp), _head_rows(forget, heads, dim, dp, wp), _head_rows(v, heads, vdim, vp, wp)])
        n_att = _up64(heads * vp)
        b = np.zeros((1, w_in.shape[0]), np.float32)
        b[0, heads * dp:2 * heads * dp] = _pad_heads(_host_f32(forget_bias).reshape(1, -1), heads, dp)
        out = cls._pack_common(width, norm1, norm1b, gate_up, down, norm2, norm2b, act_params)
        out.update(mixer=_hip.MIX_HGRN2, heads=heads, kv_heads=heads, dim=dim, vdim=vdim, head_pad=dp, vhead_pad=vp, n_att=n_att, w_in=w_in, b_in=from_numpy(b),
                   lower=from_numpy(_pad_heads(_host_f32(lower).reshape(1, -1), heads, dp, 1.0)), o_norm=_row(head_norm, vp),
                   w_o=_head_cols(o, heads, vdim, vp, wp, n_att))
        return out

    @classmethod
    def pack_delta(cls, q: GPUArray, k: GPUArray, v: GPUArray, strength: GPUArray, decay_maps: tuple[GPUArray, GPUArray], gate_maps: tuple[GPUArray, GPUArray], o: GPUArray,
                   taps: tuple[GPUArray, GPUArray, GPUArray], decay: GPUArray, step_bias: GPUArray, head_norm: GPUArray, norm1: GPUArray | None,
                   norm1b: GPUArray | None = None, *, heads: int, kv_heads: int, dim: int, vdim: int) -> dict:
        """One layer of the gated delta rule: matrices [out, in], taps of q, k, v [taps, channels]; fp32 decay [heads], step_bias [heads * dim],
        head_norm [vdim].  Head widths up to 32 / 64 / 128 / a multiple of 16 (keys) and of 16 (values); padding channels stay zero."""
        width = q.shape[1]
        wp, vp = _up64(width), _up(vdim, 16)
        dp = next((p for p in (32, 64, 128) if dim <= p), _up(dim, 16))
        ra, rg = (_up64(m[0].shape[0]) for m in (decay_maps, gate_maps))
        channels = 2 * kv_heads * dp + heads * vp
        w_in = _stack_rows([_head_rows(q, kv_heads, dim, dp, wp), _head_rows(k, kv_heads, dim, dp, wp), _head_rows(v, heads, vdim, vp, wp),
                            pad_2d(strength, _up64(channels + heads) - channels, wp), pad_2d(decay_maps[0], ra, wp), pad_2d(gate_maps[0], rg, wp)])
        n_att = _up64(heads * vp)
        out = cls._pack_common(width, norm1, norm1b, None, None, None, None, None)
        out.update(mixer=_hip.MIX_DELTA, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, head_pad=dp, vhead_pad=vp, rank_a=ra, rank_g=rg, n_att=n_att, w_in=w_in,
                   taps=taps[0].shape[0], conv=_pad_taps(taps, ((kv_heads, dp), (kv_heads, dp), (heads, vp))), decay=decay,
                   dt_bias=from_numpy(_pad_heads(_host_f32(step_bias).reshape(1, -1), heads, dp)), o_norm=_row(head_norm, vp),
                   w_a2=_head_rows(decay_maps[1], heads, dim, dp, ra), w_g2=_head_rows(gate_maps[1], heads, vdim, vp, rg), w_o=_head_cols(o, heads, vdim, vp, wp, n_att))
        return out

    @classmethod
    def pack_state_space(cls, z: GPUArray, xbc: GPUArray, t: GPUArray, o: GPUArray, taps: GPUArray, taps_bias: GPUArray, decay: GPUArray, step_bias: GPUArray, skip: GPUArray,
                         out_norm: GPUArray, norm1: GPUArray | None, norm1b: GPUArray | None = None, *, heads: int, groups: int, dim: int, vdim: int, norm_parts: int) -> dict:
        """One state-space layer: rows of z [heads * vdim, width], x | B | C and t [heads, width]; taps [taps, channels of x | B | C]; fp32 taps_bias,
        decay, step_bias, skip [heads], out_norm [heads * vdim]."""
        width = z.shape[1]
        wp, dp, vp = _up64(width), _up(dim, 16), _up(vdim, 16)
        v, g = heads * vdim, groups * dim
        sizes, heads_of = (v, g, g), ((heads, vp), (groups, dp), (groups, dp))
        at = (0, v, v + g)
        cut = lambda i: xbc._view(at[i] * width, (sizes[i], width))  # noqa: E731
        w_in = _stack_rows([_head_rows(cut(0), heads, vdim, vp, wp), _head_rows(cut(1), groups, dim, dp, wp), _head_rows(cut(2), groups, dim, dp, wp),
                            _head_rows(z, heads, vdim, vp, wp), pad_2d(t, heads, wp)])
        n_att = _up64(heads * vp)
        host = taps.to_numpy()
        parts = tuple(from_numpy(host[:, a:a + n]) for a, n in zip(at, sizes))
        bias = _host_f32(taps_bias).reshape(1, -1)
        out = cls._pack_common(width, norm1, norm1b, None, None, None, None, None)
        out.update(mixer=_hip.MIX_SSD, heads=heads, kv_heads=groups, dim=dim, vdim=vdim, head_pad=dp, vhead_pad=vp, n_att=n_att, w_in=w_in, norm_parts=norm_parts,
                   taps=taps.shape[0], conv=_pad_taps(parts, heads_of), decay=decay, dt_bias=step_bias.view((1, heads)), skip=skip.view((1, heads)),
                   conv_bias=from_numpy(np.concatenate([_pad_heads(bias[:, a:a + n], h, p) for a, n, (h, p) in zip(at, sizes, heads_of)], axis=1)),
                   o_norm=from_numpy(_pad_heads(_host_f32(out_norm).reshape(1, -1), heads, vp)), w_o=_head_cols(o, heads, vdim, vp, wp, n_att))
        return out

    @classmethod
    def pack_talking(cls, q: GPUArray, k: GPUArray | None, v: GPUArray | None, o: GPUArray, norm1: GPUArray, *, heads: int, kv_heads: int, dim: int, vdim: int, window: int,
                     chunked: bool, scale: float, biases: tuple, o_bias: GPUArray | None, q_norm: GPUArray, k_norm: GPUArray | None, rot_freq: GPUArray | None = None,
                     talk: GPUArray | None = None, sink: GPUArray | None = None, kv_from: int | None = None) -> dict:
        """The mixer of one hyper-connected layer: q, k, v, o [out, in] (k, v None with kv_from) and their biases; fp32 norms over a head's dim,
        rot_freq [rot / 2], talk [heads, heads], sink [heads]."""
        width = q.shape[1]
        wp, hp = _up64(width), _attention_pad(dim, vdim)
        parts = [(q, heads, dim)] + ([] if kv_from is not None else [(k, kv_heads, dim), (v, kv_heads, vdim)])
        w_in = _stack_rows([_head_rows(w, n, d, hp, wp) for w, n, d in parts])
        b = np.zeros((1, w_in.shape[0]), np.float32)
        flat = np.concatenate([_pad_heads(_host_f32(a).reshape(-1), n, hp) for a, (_, n, _) in zip(biases, parts)])
        b[0, :flat.size] = flat
        out = cls._pack_common(width, norm1, None, None, None, None, None, None)
        out.update(mixer=_hip.MIX_TALK, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, window=window, chunked=int(chunked), scale=scale, head_pad=hp, vhead_pad=hp, n_att=heads * hp,
                   kv_from=-1 if kv_from is None else kv_from, w_in=w_in, b_in=from_numpy(b), q_norm=_row(q_norm, hp), k_norm=None if k_norm is None else _row(k_norm, hp),
                   rot=0 if rot_freq is None else 2 * rot_freq.size, rot_freq=rot_freq, talk=talk, sink=sink,
                   b_o=None if o_bias is None else _row(from_numpy(_host_f32(o_bias)), wp), w_o=_head_cols(o, heads, vdim, hp, wp, heads * hp))
        return out

    @staticmethod
    def pack_hyper(read: GPUArray, write: GPUArray, mix: GPUArray) -> GPUArray:
        """A sublayer's numbers as the kernels read them: read | write | mix [from][to]"""
        return from_numpy(np.concatenate([a.to_numpy().reshape(-1) for a in (read, write, mix)]))

    @staticmethod
    def add_poly_mlp(layer: dict, width: int, up: GPUArray, down: GPUArray, act: GPUArray) -> dict:
        """A packed mixer plus a dense feed-forward with a polynomial-norm activation: up [ff, width], down [width, ff], act fp32 [4]."""
        ff, wp = up.shape[0], _up64(width)
        fp = _up64(ff)
        layer.update(ff=_hip.FF_POLY, ff_pad=fp, ff_dim=ff, w_gate_up=pad_2d(up, fp, wp), w_down=pad_2d(down, wp, fp), act=act)
        return layer

    @staticmethod
    def add_table_experts(layer: dict, width: int, table: GPUArray, up: GPUArray, down: GPUArray, shared: tuple[GPUArray, GPUArray, GPUArray] | None) -> dict:
        """A packed mixer plus experts that a table chooses: table int32 [vocab, top], up [E, ff, width], down [E, width, ff]; shared: the shared
        expert's up [ff', width], down [width, ff'] and gate [1, width]."""
        E, ff, _ = up.shape
        wp, fp = _up64(width), _up64(ff)
        layer.update(ff=_hip.FF_TABLE, ff_pad=fp, experts=E, top=table.shape[1], table=table, shared_pad=0,
                     w_gate_up=_head_rows(up.view((E * ff, width)), E, ff, fp, wp).view((E, fp, wp)), w_down=_head_rows(down.view((E * width, ff)), E, width, wp, fp).view((E, wp, fp)))
        if shared is not None:
            sp = _up64(shared[0].shape[0])
            layer.update(shared_pad=sp, w_shared_up=pad_2d(shared[0], sp, wp), w_shared_down=pad_2d(shared[1], wp, sp), w_shared_gate=pad_2d(shared[2], 1, wp))
        return layer

    @classmethod
    def _pack_hyper_block(cls, b, c) -> dict:
        from pygpukit_amd.llm.layers import TableExperts, TalkingAttention

        a = b.attn
        if not isinstance(a, TalkingAttention):
            raise NotImplementedError(f"the layer-list engine has no hyper-connected layer of {type(a).__name__}")
        norms = [n for n in (b.attn_norm, b.mlp_norm, a.q_norm, a.k_norm) if n is not None]
        if any(n.eps != c.norm_eps for n in norms) or any(n.groups != c.norm_groups for n in norms[:1 if b.mlp_norm is None else 2]):
            raise NotImplementedError("the layer-list engine takes one epsilon and one number of norm groups for all layers")
        own = a.source is None
        out = cls.pack_talking(a.q_proj.weight, a.k_proj.weight if own else None, a.v_proj.weight if own else None, a.o_proj.weight, b.attn_norm.weight, heads=a.num_heads,
                               kv_heads=a.num_kv_heads, dim=a.head_dim, vdim=a.v_head_dim, window=a.window, chunked=a.chunked, scale=a.scale,
                               biases=tuple(p.bias for p in ((a.q_proj, a.k_proj, a.v_proj) if own else (a.q_proj,))), o_bias=a.o_proj.bias, q_norm=a.q_norm.weight,
                               k_norm=a.k_norm.weight if own else None, rot_freq=a.rot_freq, talk=a.talk, sink=a.sink, kv_from=a.kv_from)
        h, m, width = b.attn_hyper, b.mlp, a.q_proj.weight.shape[1]
        out["hyper1"] = cls.pack_hyper(h.read, h.write, h.mix)
        if m is None:
            return out
        h = b.mlp_hyper
        out.update(hyper2=cls.pack_hyper(h.read, h.write, h.mix), norm2=_row(b.mlp_norm.weight, _up64(width)))
        if isinstance(m, TableExperts):
            shared = None if m.shared_up is None else (m.shared_up.weight, m.shared_down.weight, m.shared_gate.weight)
            return cls.add_table_experts(out, width, m.table, m.up, m.down, shared)
        if m.activation != "poly_norm" or m.act_eps != c.norm_eps:
            raise NotImplementedError("hyper-connected layers have polynomial-norm feed-forwards or experts chosen by a table")
        return cls.add_poly_mlp(out, width, m.fc1.weight, m.fc2.weight, m.act_params)

    @staticmethod
    def add_experts(layer: dict, width: int, router: GPUArray, correction: GPUArray, gate_up: GPUArray, down: GPUArray, *, top: int, groups: int = 0, keep: int = 0,
                    scale: float = 1.0) -> dict:
        """A packed mixer plus its layer's experts: router [E, width], gate_up [E, 2 ff, width], down [E, width, ff], correction fp32 [E].  The
        router's rows go behind the mixer's in w_in."""
        E, two_ff, _ = gate_up.shape
        ff, wp = two_ff // 2, _up64(width)
        fp = _up64(ff)
        layer.update(ff=_hip.FF_MOE, ff_pad=fp, experts=E, top=top, groups=groups, keep=keep, router_scale=scale, correction=correction,
                     w_in=concat_axis0(layer["w_in"], pad_2d(router, _up64(E), wp)),
                     w_gate_up=_head_rows(gate_up.view((2 * E * ff, width)), 2 * E, ff, fp, wp).view((E, 2 * fp, wp)),
                     w_down=_head_rows(down.view((E * width, ff)), E, width, wp, fp).view((E, wp, fp)))
        return layer

    @classmethod
    def _pack_parallel(cls, b) -> dict:
        from pygpukit_amd.llm.layers import ChannelDelta, LatentAttention, StateSpace

        a, norm = b.attn, b.attn_norm.weight
        if isinstance(a, LatentAttention):
            out = cls.pack_layer(a.q_proj.weight, a.kv_down.weight, None if a.head_gate is None else a.head_gate.weight, a.kv_norm.weight, a.k_up.weight, a.v_up.weight,
                                 a.o_proj.weight, norm, None, heads=a.num_heads, dim=a.head_dim + a.rot_dim, vdim=a.v_head_dim, window=a.window, scale=a.scale, rot_freq=a.rot_freq)
        elif isinstance(a, ChannelDelta):
            w = lambda maps: tuple(m.weight for m in maps)  # noqa: E731
            out = cls.pack_delta(a.q_proj.weight, a.k_proj.weight, a.v_proj.weight, a.strength.weight, w(a.decay_maps), w(a.gate_maps), a.o_proj.weight, a.taps, a.decay, a.step_bias,
                                 a.head_norm, norm, heads=a.num_heads, kv_heads=a.num_kv_heads, dim=a.head_dim, vdim=a.v_head_dim)
        elif isinstance(a, StateSpace):
            out = cls.pack_state_space(a.z_proj.weight, a.xbc_proj.weight, a.t_proj.weight, a.o_proj.weight, a.taps, a.taps_bias, a.decay, a.step_bias, a.skip, a.out_norm, norm,
                                       heads=a.num_heads, groups=a.num_groups, dim=a.head_dim, vdim=a.v_head_dim, norm_parts=a.norm_groups)
        else:
            raise NotImplementedError(f"the layer-list engine has no parallel layer of {type(a).__name__}")
        m = b.mlp
        if m is not None:
            cls.add_experts(out, m.router.shape[1], m.router, m.correction, m.gate_up, m.down, top=m.top, groups=m.groups, keep=m.keep, scale=m.scale)
        return out

    @classmethod
    def _pack_block(cls, b, c) -> dict:
        from pygpukit_amd.llm.layers import GatedRecurrence, GatedWindowAttention, HyperBlock, LatentAttention, ParallelBlock

        if isinstance(b, HyperBlock):
            return cls._pack_hyper_block(b, c)
        if isinstance(b, ParallelBlock):
            if b.attn_norm.eps != c.norm_eps or b.attn_norm.norm_type != c.norm_type:
                raise NotImplementedError("the layer-list engine takes one kind of norm and one epsilon for all layers")
            return cls._pack_parallel(b)
        a = b.attn
        if b.post_attn_norm is None or (b.mlp is not None and b.post_mlp_norm is None):
            raise NotImplementedError("the layer-list engine needs a norm after each sublayer")
        if b.residual_mult != c.residual_mult or b.post_attn_norm.eps != c.norm_eps:
            raise NotImplementedError("the layer-list engine takes one residual factor and one norm epsilon for all layers")
        weight = lambda n: None if n is None else n.weight  # noqa: E731
        common = {}
        if b.mlp is not None:
            xielu = b.mlp.activation == "xielu"
            if not xielu and b.mlp.gate_up_proj is None:
                raise NotImplementedError("the layer-list engine needs a fused gate / up weight")
            common = dict(gate_up=b.mlp.fc1.weight if xielu else b.mlp.gate_up_proj.weight, down=b.mlp.fc2.weight if xielu else b.mlp.down_proj.weight,
                          norm2=weight(b.mlp_norm), norm2b=b.post_mlp_norm.weight, act_params=b.mlp.act_params if xielu else None)
        norms = (weight(b.attn_norm), b.post_attn_norm.weight)
        if isinstance(a, LatentAttention):
            if a.head_gate is None or b.attn_norm is None:
                raise NotImplementedError("the layer-list engine needs a norm before gated latent attention")
            return cls.pack_layer(a.q_proj.weight, a.kv_down.weight, a.head_gate.weight, a.kv_norm.weight, a.k_up.weight, a.v_up.weight, a.o_proj.weight, *norms,
                                  rot_freq=a.rot_freq, heads=a.num_heads, dim=a.head_dim + a.rot_dim, vdim=a.v_head_dim, window=a.window, scale=a.scale, **common)
        if isinstance(a, GatedWindowAttention):
            own = a.source is None
            return cls.pack_attention(a.q_proj.weight, a.k_proj.weight if own else None, a.v_proj.weight if own else None, a.out_gate.weight, a.o_proj.weight, *norms,
                                      heads=a.num_heads, kv_heads=a.num_kv_heads, dim=a.head_dim, vdim=a.v_head_dim, window=a.window, scale=a.scale,
                                      biases=(a.q_proj.bias, a.k_proj.bias, a.v_proj.bias) if own else (a.q_proj.bias,),
                                      convs=(a.q_conv, a.k_conv, a.v_conv) if own else (a.q_conv,), q_norm=weight(a.q_norm), k_norm=weight(a.k_norm), slopes=a.slopes,
                                      kv_from=a.kv_from, **common)
        if isinstance(a, GatedRecurrence):
            return cls.pack_recurrence(a.q_proj.weight, a.forget_proj.weight, a.v_proj.weight, a.o_proj.weight, a.forget_bias, a.lower, a.head_norm, *norms,
                                       heads=a.num_heads, dim=a.head_dim, vdim=a.v_head_dim, **common)
        raise NotImplementedError(f"the layer-list engine has no {type(a).__name__}")

    @classmethod
    def from_model(cls, model, *, max_seq_len: int = 512, max_batch: int = 1) -> "StackEngine":
        c = model.config
        width = model.embed_tokens.shape[1]
        packed = model.__dict__.get("_stack_layers")       # packed once, shared by every engine of this model
        if packed is None:
            packed = [cls._pack_block(b, c) for b in model.blocks]
            head = model._lm_head if model._lm_head is not None else model.embed_tokens
            wp = _up64(width)
            model._stack_layers = packed
            model._stack_head = (pad_2d(head, head.shape[0], wp), _row(model.final_norm.weight, wp))
            model._stack_more = cls._pack_more(model, width)
        head, fnorm = model._stack_head
        cfg = dict(vocab_size=model.embed_tokens.shape[0], width=width, hidden_size=width, max_positions=c.max_position_embeddings, norm_eps=c.norm_eps,
                   residual_mult=c.residual_mult, **model._stack_more)
        return cls(cfg, model.embed_tokens, model.position_embed, head, fnorm, packed, max_seq_len=max_seq_len, max_batch=max_batch)

    @staticmethod
    def _pack_more(model, width: int) -> dict:
        """What parallel or hyper-connected layers and a loop add to the engine's configuration."""
        from pygpukit_amd.llm.layers import HyperBlock, ParallelBlock

        c, hyper = model.config, [isinstance(b, HyperBlock) for b in model.blocks]
        if any(hyper):
            if not all(hyper):
                raise NotImplementedError("the layer-list engine takes hyper-connected layers or others, not both")
            return dict(block=_hip.BLOCK_HYPER, streams=c.streams, norm_groups=c.norm_groups, logit_cap=c.logit_softcap)

        parallel = [isinstance(b, ParallelBlock) for b in model.blocks]
        if not any(parallel):
            return {}
        if not all(parallel):
            raise NotImplementedError("the layer-list engine takes parallel or sandwich layers, not both")
        out: dict = dict(block=_hip.BLOCK_PARALLEL, layer_norm=int(model.final_norm.norm_type == "layernorm"))
        if model.loop is not None:
            l, wp = model.config.loop, _up64(width)
            out.update(loop=(l.start, l.stop, l.times), loop_in=_head_cols(model.loop.weight, 2, width, wp, wp, 2 * wp), loop_step=pad_2d(model.loop.step, l.times, wp))
        return out

    def _layer_memory(self, layer: int, shape: tuple[int, ...], dtype) -> GPUArray:
        p, none = C.c_void_p(), C.c_void_p()
        _hip.call("pgk_engine_kv_ptr", self.handle, layer, C.byref(p), C.byref(none))
        a = GPUArray(shape, dtype, p.value, owns_memory=False)
        a._source_ref = self
        return a

    def latent_cache(self, layer: int) -> GPUArray:
        """[max_batch, R, rank_pad] view of layer `layer`'s latent rings: position p of a sequence is row p % R, R = min(window, max_seq_len).
        (With a loop, here and below: of run `layer`, one pass of one layer in the order they run.)"""
        lw = self.layers[self._runs[layer]]
        if lw["mixer"] != _hip.MIX_LATENT:
            raise ValueError(f"layer {layer} caches no latents")
        return self._layer_memory(layer, (self.max_batch, min(lw["window"], self.max_seq_len), lw["rank_pad"]), self.dtype)

    def recurrent_state(self, layer: int) -> GPUArray:
        """float32 [max_batch, heads, dim, vdim] (widths padded) view of layer `layer`'s states."""
        lw = self.layers[self._runs[layer]]
        if lw["mixer"] not in (_hip.MIX_HGRN2, _hip.MIX_DELTA, _hip.MIX_SSD):
            raise ValueError(f"layer {layer} has no recurrent state")
        return self._layer_memory(layer, (self.max_batch, lw["heads"], lw["head_pad"], lw["vhead_pad"]), float32)

    def kv_cache(self, layer: int):
        raise NotImplementedError("a layer-list engine's caches are rings and states: latent_cache(), recurrent_state()")
