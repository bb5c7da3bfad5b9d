"""Grouped-head attention over a sliding window, with taps over time, norms over whole projections, a distance bias and an elementwise gate.

    u = W x + b for q, k, v;   y_t = sum_j w_j u_(t - taps + 1 + j) per channel;   q, k: y / rms(y) * weight over the whole row
    s_a(i, j) = scale * q_a(i) . k(j) - slope_a * (i - j)  for 0 <= i - j < window;   out = O (sigmoid(G x) * [softmax(s_a) v])

A layer may take the keys and values of an earlier one (`source`) and then has only q, the gate and O of its own.  This is the
operator-surface form; the native engine's is csrc/engine_stack.hip with the kernels of csrc/ops_gated_attn.hip."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float16
from pygpukit_amd.core.factory import zeros
from pygpukit_amd.ops._common import call
from pygpukit_amd.ops.basic import cast_bf16_to_f32, cast_f16_to_f32, concat_axis0, rmsnorm_f32, short_conv, window_attention

from .linear import LinearBF16
from .norm import Norm

NO_WINDOW = 2**30


class GatedWindowAttention:
    def __init__(self, q_proj: LinearBF16, k_proj: LinearBF16 | None, v_proj: LinearBF16 | None, o_proj: GPUArray, out_gate: GPUArray, *, num_heads: int,
                 num_kv_heads: int, head_dim: int, v_head_dim: int, scale: float, window: int | None = None, q_norm: Norm | None = None, k_norm: Norm | None = None,
                 q_conv: GPUArray | None = None, k_conv: GPUArray | None = None, v_conv: GPUArray | None = None, slopes: GPUArray | None = None,
                 source: "GatedWindowAttention | None" = None, kv_from: int | None = None):
        """q_proj [heads * head_dim, hidden], k_proj / v_proj over the kv heads (None with `source`), o_proj [hidden, heads * v_head_dim],
        out_gate [heads * v_head_dim, hidden], *_conv [channels, taps], slopes float32 [heads]; kv_from: the source's layer index."""
        if (source is None) != (k_proj is not None and v_proj is not None) or (source is None) != (kv_from is None):
            raise ValueError("GatedWindowAttention: key and value projections, or a source layer")
        self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim = num_heads, num_kv_heads, head_dim, v_head_dim
        self.scale, self.window = float(scale), NO_WINDOW if window is None else int(window)
        self.q_proj, self.k_proj, self.v_proj = q_proj, k_proj, v_proj
        self.o_proj, self.out_gate = LinearBF16(o_proj), LinearBF16(out_gate)
        self.q_norm, self.k_norm, self.q_conv, self.k_conv, self.v_conv = q_norm, k_norm, q_conv, k_conv, v_conv
        self.slopes, self.source, self.kv_from = slopes, source, kv_from
        self.cache_rows = source is None          # past[0] has a row per position
        self._k_cache: GPUArray | None = None
        self._v_cache: GPUArray | None = None
        self._tails: list[GPUArray] = []
        self._max_cache_len = 0

    # ------------------------------------------------------------------ projections
    def _branches(self) -> list[tuple[LinearBF16, GPUArray | None, Norm | None]]:
        q = [(self.q_proj, self.q_conv, self.q_norm)]
        return q if self.source is not None else q + [(self.k_proj, self.k_conv, self.k_norm), (self.v_proj, self.v_conv, None)]

    def _empty_tails(self) -> list[GPUArray]:
        return [zeros((max(c.shape[1] - 1, 1), p.out_features), p.weight.dtype) for p, c, _ in self._branches() if c is not None]

    def _project(self, x: GPUArray, tails: list[GPUArray]) -> tuple[list[GPUArray], list[GPUArray]]:
        """q (k, v) rows of x and the tails after it."""
        out, new, at = [], [], 0
        for proj, conv, norm in self._branches():
            y = proj(x)
            if conv is not None:
                taps, u = conv.shape[1], y
                y = short_conv(u, conv, tails[at] if taps > 1 else None)
                both = concat_axis0(tails[at], u)
                keep = max(taps - 1, 1)
                new.append(both._view((both.shape[0] - keep) * u.shape[1], (keep, u.shape[1])))
                at += 1
            if norm is not None:
                f = cast_bf16_to_f32(y) if y.dtype == bfloat16 else cast_f16_to_f32(y) if y.dtype == float16 else y
                y = rmsnorm_f32(f, norm.weight, norm.eps, dtype=y.dtype)
            out.append(y)
        return out, new

    def attend(self, x: GPUArray, q: GPUArray, k: GPUArray, v: GPUArray) -> GPUArray:
        """x [S, hidden] and q: the newest S of the positions whose k, v [kv_len, ...] are given."""
        S, H, G, d, dv = x.shape[0], self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim
        n = k.shape[0]
        seen = min(n, self.window - 1 + S)                       # rows before that are outside every query's window
        k, v = k._view((n - seen) * G * d, (seen, G, d)), v._view((n - seen) * G * dv, (seen, G, dv))
        y = window_attention(q.view((S, H, d)), k, v, self.scale, self.window, gate=self.out_gate(x).view((S, H, dv)), slopes=self.slopes)
        return self.o_proj(y.view((S, H * dv)))

    # ------------------------------------------------------------------ dynamic cache
    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None, use_cache: bool = False,
                 source_kv: tuple | None = None) -> tuple[GPUArray, tuple | None]:
        """past / present: (keys [kv_len, ...], values, tails ...); with a source layer (tails ...) only, and source_kv its present."""
        tails = self._empty_tails() if past_kv is None else list(past_kv if self.source is not None else past_kv[2:])
        rows, tails = self._project(x, tails)
        if self.source is not None:
            k, v = source_kv[:2]
            present = tuple(tails)
        else:
            k, v = rows[1:] if past_kv is None else (concat_axis0(past_kv[0], rows[1]), concat_axis0(past_kv[1], rows[2]))
            present = (k, v, *tails)
        return self.attend(x, rows[0], k, v), (present if use_cache else None)

    # ------------------------------------------------------------------ fixed cache
    def init_fixed_cache(self, max_seq_len: int, dtype: str = "bfloat16") -> None:
        if self.source is None:
            self._k_cache = zeros((max_seq_len, self.num_kv_heads * self.head_dim), dtype)
            self._v_cache = zeros((max_seq_len, self.num_kv_heads * self.v_head_dim), dtype)
        self._tails = self._empty_tails()
        self._max_cache_len = max_seq_len

    def fill_fixed_cache(self, present: tuple) -> None:
        tails = present
        if self.source is None:
            self._store(present[0], present[1], 0)
            tails = present[2:]
        self._keep(list(tails))

    def cache_arrays(self) -> tuple[GPUArray, ...]:
        return (*(() if self.source is not None else (self._k_cache, self._v_cache)), *self._tails)

    def _keep(self, tails: list[GPUArray]) -> None:
        for dst, src in zip(self._tails, tails):
            call("pgk_memcpy_d2d", dst._p, src._p, src.nbytes, None)

    def _store(self, k: GPUArray, v: GPUArray, position: int) -> None:
        if self._k_cache is None:
            raise RuntimeError("Call init_fixed_cache first")
        if position < 0 or position + k.shape[0] > self._max_cache_len or k.dtype != self._k_cache.dtype:
            raise ValueError(f"rows {position}..{position + k.shape[0]} ({k.dtype}) outside the cache [{self._max_cache_len}] ({self._k_cache.dtype})")
        for dst, src in ((self._k_cache, k), (self._v_cache, v)):
            call("pgk_memcpy_d2d", dst.data_ptr() + position * dst.shape[1] * dst.itemsize, src._p, src.nbytes, None)

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int, *, out: GPUArray | None = None) -> GPUArray:
        return self.forward_fixed_cache_batch(x, position, context_len)

    def forward_fixed_cache_batch(self, x: GPUArray, start_position: int, context_len: int) -> GPUArray:
        """The tails are those of the last token run: positions go on from there or start at 0."""
        if context_len != start_position + x.shape[0]:
            raise ValueError(f"context_len {context_len} must end with the {x.shape[0]} tokens at position {start_position}")
        rows, tails = self._project(x, self._empty_tails() if start_position == 0 else self._tails)
        self._keep(tails)
        if self.source is None:
            self._store(rows[1], rows[2], start_position)
        kv = self.source if self.source is not None else self
        return self.attend(x, rows[0], kv._k_cache.slice_rows(context_len), kv._v_cache.slice_rows(context_len))


__all__ = ["GatedWindowAttention"]
