"""Grouped-head attention whose heads mix their scores before the softmax, with a sink per head, over a sliding window or in chunks of
positions.

    q, k, v = W h + b per head;   q, k <- turn(norm(.)): RMS norm over the head, then columns i and i + rot / 2 turned by the position
    raw_h(i, j) = scale * q_h(i) . k(j);   s_h = sum_g talk[h, g] raw_g;   p_h = exp(s_h) / (sum_j exp(s_h) + exp(sink_h));   out = O p v + b_o

A layer may take the keys and values of an earlier one (`source`) and then has only q and O of its own.  This is the operator-surface
form; the native engine's is csrc/engine_stack.hip with the kernels of csrc/ops_talk.hip."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.factory import zeros
from pygpukit_amd.ops._common import call
from pygpukit_amd.ops.basic import concat_axis0, head_norm_rope, talk_attention

from .linear import LinearBF16
from .norm import Norm

NO_WINDOW = 2**30


class TalkingAttention:
    def __init__(self, q_proj: LinearBF16, k_proj: LinearBF16 | None, v_proj: LinearBF16 | None, o_proj: LinearBF16, *, num_heads: int, num_kv_heads: int, head_dim: int,
                 v_head_dim: int, scale: float, window: int | None = None, chunked: bool = False, q_norm: Norm, k_norm: Norm | None = None, rot_freq: GPUArray | None = None,
                 talk: GPUArray | None = None, sink: GPUArray | None = None, source: "TalkingAttention | None" = None, kv_from: int | None = None):
        """Projections with their biases (k_proj, v_proj None with `source`); q_norm, k_norm over head_dim; rot_freq float32 [rot / 2]; talk
        float32 [heads, heads]; sink float32 [heads]; kv_from: the source's layer index."""
        if (source is None) != (k_proj is not None and v_proj is not None and k_norm is not None) or (source is None) != (kv_from is None):
            raise ValueError("TalkingAttention: key and value projections with the keys' norm, or a source layer")
        self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim = num_heads, num_kv_heads, head_dim, v_head_dim
        self.scale, self.window, self.chunked = float(scale), NO_WINDOW if window is None else int(window), bool(chunked)
        self.q_proj, self.k_proj, self.v_proj, self.o_proj = q_proj, k_proj, v_proj, o_proj
        self.q_norm, self.k_norm, self.rot_freq, self.talk, self.sink = q_norm, k_norm, rot_freq, talk, sink
        self.source, self.kv_from = source, kv_from
        self.cache_rows = source is None          # past[0] has a row per position
        self._k_cache: GPUArray | None = None
        self._v_cache: GPUArray | None = None
        self._max_cache_len = 0

    def _heads(self, x: GPUArray, proj: LinearBF16, norm: Norm, heads: int, first: int) -> GPUArray:
        return head_norm_rope(proj(x).view((x.shape[0], heads, self.head_dim)), norm.weight, self.rot_freq, first, norm.eps)

    def _keys_values(self, x: GPUArray, first: int) -> tuple[GPUArray, GPUArray]:
        """[S, kv heads * width] each"""
        return self._heads(x, self.k_proj, self.k_norm, self.num_kv_heads, first).view((x.shape[0], self.num_kv_heads * self.head_dim)), self.v_proj(x)

    def seen_from(self, position: int) -> int:
        """The first position that a query at `position` sees."""
        return position - position % self.window if self.chunked else max(0, position - self.window + 1)

    def attend(self, x: GPUArray, k: GPUArray, v: GPUArray) -> GPUArray:
        """x [S, hidden]: the newest S of the positions whose k, v [positions, ...] are given."""
        S, H, G, d, dv = x.shape[0], self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim
        n = k.shape[0]
        q = self._heads(x, self.q_proj, self.q_norm, H, n - S)
        lo = self.seen_from(n - S)
        k, v = k._view(lo * G * d, (n - lo, G, d)), v._view(lo * G * dv, (n - lo, G, dv))
        y = talk_attention(q, k, v, self.scale, self.window, chunked=self.chunked, first=lo, talk=self.talk, sink=self.sink)
        return self.o_proj(y.view((S, H * dv)))

    # ------------------------------------------------------------------ dynamic cache
    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None, use_cache: bool = False,
                 source_kv: tuple | None = None) -> tuple[GPUArray, tuple | None]:
        """past / present: (keys [kv_len, ...], values); with a source layer () and source_kv its present."""
        if self.source is not None:
            return self.attend(x, *source_kv), (() if use_cache else None)
        k, v = self._keys_values(x, 0 if past_kv is None else past_kv[0].shape[0])
        if past_kv is not None:
            k, v = concat_axis0(past_kv[0], k), concat_axis0(past_kv[1], v)
        return self.attend(x, k, v), ((k, v) if use_cache else None)

    # ------------------------------------------------------------------ fixed cache
    def init_fixed_cache(self, max_seq_len: int, dtype: str = "bfloat16") -> None:
        if self.source is None:
            self._k_cache = zeros((max_seq_len, self.num_kv_heads * self.head_dim), dtype)
            self._v_cache = zeros((max_seq_len, self.num_kv_heads * self.v_head_dim), dtype)
        self._max_cache_len = max_seq_len

    def fill_fixed_cache(self, present: tuple) -> None:
        if self.source is None:
            self._store(present[0], present[1], 0)

    def cache_arrays(self) -> tuple[GPUArray, ...]:
        return () if self.source is not None else (self._k_cache, self._v_cache)

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
        if context_len != start_position + x.shape[0]:
            raise ValueError(f"context_len {context_len} must end with the {x.shape[0]} tokens at position {start_position}")
        if self.source is None:
            self._store(*self._keys_values(x, start_position), start_position)
        kv = self.source if self.source is not None else self
        return self.attend(x, kv._k_cache.slice_rows(context_len), kv._v_cache.slice_rows(context_len))


__all__ = ["TalkingAttention"]
