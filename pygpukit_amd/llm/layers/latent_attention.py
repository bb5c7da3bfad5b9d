"""Latent attention: keys and values are linear maps of one small normalised vector per token, and only that vector is cached.

    c = rmsnorm(D h) * w_c        [kv_rank]         k_a = U_k,a c,  v_a = U_v,a c
    y_a = sigmoid((G h)_a) * softmax_window(scale * q_a . k_a) v_a,   q = Q h        out = O [y_0 .. y_H-1]

With rot_dim > 0 the last rot_dim columns of every q_a and the last rot_dim rows of D h (not normed, one vector for all heads, appended
to every k_a) are turned by the position: pair (2i, 2i + 1) by position * rot_base^(-2i / rot_dim).  The cached row is [c | that vector].

This is the operator-surface form (one op call per step, any float dtype): dynamic past (the latents of every position so far) and
fixed cache [max_seq, kv_rank].  The native engine's form - latents in a ring of `window` rows, U_k folded into the query while
decoding - is csrc/engine_stack.hip, which takes the same weights (StackEngine)."""

from __future__ import annotations

import numpy as np

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float16, float32
from pygpukit_amd.core.factory import from_numpy, zeros
from pygpukit_amd.ops._common import call
from pygpukit_amd.ops.basic import cast_bf16_to_f32, cast_f16_to_f32, concat_axis0, latent_rows, rmsnorm_f32, rotate_pairs, window_attention

from .linear import LinearBF16
from .norm import Norm

NO_WINDOW = 2**30


class LatentAttention:
    def __init__(self, q_proj: GPUArray, kv_down: GPUArray, kv_norm: Norm, k_up: GPUArray, v_up: GPUArray, o_proj: GPUArray, *, num_heads: int,
                 head_dim: int, v_head_dim: int, scale: float, window: int | None = None, head_gate: GPUArray | None = None, rot_dim: int = 0,
                 rot_freq: GPUArray | None = None):
        """q_proj [heads * head_dim, hidden], kv_down [rank, hidden], k_up [heads * head_dim, rank], v_up [heads * v_head_dim, rank],
        o_proj [hidden, heads * v_head_dim], head_gate [heads, hidden]; kv_norm: fp32-stream norm of width rank.  With rot_dim: q_proj
        [heads * (head_dim + rot_dim), hidden], kv_down [rank + rot_dim, hidden], rot_freq float32 [rot_dim / 2]."""
        self.num_heads, self.head_dim, self.v_head_dim = num_heads, head_dim, v_head_dim
        self.rot_dim, self.rot_freq = rot_dim, rot_freq
        self.kv_rank, self.scale = kv_down.shape[0] - rot_dim, float(scale)
        self.cache_width = self.kv_rank + rot_dim
        self.window = NO_WINDOW if window is None else int(window)
        hidden = q_proj.shape[1]
        want = {"q_proj": (q_proj, (num_heads * (head_dim + rot_dim), hidden)), "kv_down": (kv_down, (self.cache_width, hidden)),
                "k_up": (k_up, (num_heads * head_dim, self.kv_rank)), "v_up": (v_up, (num_heads * v_head_dim, self.kv_rank)),
                "o_proj": (o_proj, (hidden, num_heads * v_head_dim))}
        if head_gate is not None:
            want["head_gate"] = (head_gate, (num_heads, hidden))
        for name, (w, shape) in want.items():
            if w.shape != shape:
                raise ValueError(f"LatentAttention: {name} is {w.shape}, expected {shape}")
        if rot_dim:                       # the maps take whole cached rows: the rotated part passes into every head's key and no value
            k, v = k_up.to_numpy(), v_up.to_numpy()
            one = 0x3F80 if k_up.dtype == bfloat16 else 1
            kx = np.zeros((num_heads, head_dim + rot_dim, self.cache_width), k.dtype)
            kx[:, :head_dim, :self.kv_rank] = k.reshape(num_heads, head_dim, self.kv_rank)
            kx[:, head_dim + np.arange(rot_dim), self.kv_rank + np.arange(rot_dim)] = one
            vx = np.zeros((v.shape[0], self.cache_width), v.dtype)
            vx[:, :self.kv_rank] = v
            k_up, v_up = from_numpy(kx.reshape(-1, self.cache_width)), from_numpy(vx)
        if kv_norm.weight.shape != (self.kv_rank,):
            raise ValueError(f"LatentAttention: kv_norm is {kv_norm.weight.shape}, expected {(self.kv_rank,)}")
        self.q_proj, self.kv_down, self.k_up, self.v_up, self.o_proj = (LinearBF16(w) for w in (q_proj, kv_down, k_up, v_up, o_proj))
        self.head_gate = LinearBF16(head_gate) if head_gate is not None else None
        self.kv_norm = kv_norm
        self._c_cache: GPUArray | None = None
        self._max_cache_len = 0

    # ------------------------------------------------------------------ cache
    def init_fixed_cache(self, max_seq_len: int, dtype: str = "bfloat16") -> None:
        self._c_cache = zeros((max_seq_len, self.cache_width), dtype)
        self._max_cache_len = max_seq_len

    def fill_fixed_cache(self, present: tuple) -> None:
        self._store(present[0], 0)

    def cache_arrays(self) -> tuple[GPUArray, ...]:
        return (self._c_cache,)

    def _store(self, c: GPUArray, position: int) -> None:
        if self._c_cache is None:
            raise RuntimeError("Call init_fixed_cache first")
        if position < 0 or position + c.shape[0] > self._max_cache_len or c.dtype != self._c_cache.dtype:
            raise ValueError(f"latent rows {position}..{position + c.shape[0]} ({c.dtype}) outside the cache [{self._max_cache_len}] ({self._c_cache.dtype})")
        call("pgk_memcpy_d2d", self._c_cache.data_ptr() + position * self.cache_width * c.itemsize, c._p, c.nbytes, None)

    # ------------------------------------------------------------------ steps
    def latents(self, x: GPUArray, first: int) -> GPUArray:
        """Cache rows of positions first, first + 1, ..."""
        d = self.kv_down(x)
        if self.rot_dim:
            return latent_rows(d, self.kv_norm.weight, self.rot_freq, first, eps=self.kv_norm.eps)
        if d.dtype == bfloat16:
            d = cast_bf16_to_f32(d)
        elif d.dtype == float16:
            d = cast_f16_to_f32(d)
        assert d.dtype == float32
        return rmsnorm_f32(d, self.kv_norm.weight, self.kv_norm.eps, dtype=x.dtype)

    def attend(self, x: GPUArray, c: GPUArray) -> GPUArray:
        """x [S, hidden]: the newest S of the positions whose latents c [kv_len, rank] holds."""
        S, H = x.shape[0], self.num_heads
        seen = min(c.shape[0], self.window - 1 + S)              # rows before that are outside every query's window
        first, d = c.shape[0] - S, self.head_dim + self.rot_dim
        c = c._view((c.shape[0] - seen) * self.cache_width, (seen, self.cache_width))
        q = self.q_proj(x).view((S, H, d))
        if self.rot_dim:
            rotate_pairs(q, self.rot_freq, first)
        k, v = self.k_up(c).view((seen, H, d)), self.v_up(c).view((seen, H, self.v_head_dim))
        gate = self.head_gate(x) if self.head_gate is not None else None
        y = window_attention(q, k, v, self.scale, self.window, gate=gate)
        return self.o_proj(y.view((S, H * self.v_head_dim)))

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False) -> tuple[GPUArray, tuple | None]:
        """past / present: (latents [kv_len, cache_width],)."""
        c = self.latents(x, 0 if past_kv is None else past_kv[0].shape[0])
        if past_kv is not None:
            c = concat_axis0(past_kv[0], c)
        return self.attend(x, c), ((c,) if use_cache else None)

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int, *, out: GPUArray | None = None) -> GPUArray:
        return self.forward_fixed_cache_batch(x, position, context_len)

    def forward_fixed_cache_batch(self, x: GPUArray, start_position: int, context_len: int) -> GPUArray:
        if context_len != start_position + x.shape[0]:
            raise ValueError(f"context_len {context_len} must end with the {x.shape[0]} tokens at position {start_position}")
        self._store(self.latents(x, start_position), start_position)
        return self.attend(x, self._c_cache.slice_rows(context_len))


__all__ = ["LatentAttention"]
