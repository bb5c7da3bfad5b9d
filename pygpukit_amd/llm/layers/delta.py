"""Gated delta rule with a decay per key channel.

    q, k, v = silu(taps over time of Q x, K x, V x);  q, k of unit length per head, q also times head_dim^-1/2;  b = sigmoid(B x)
    g = exp(-decay * softplus(A_2 A_1 x + step_bias))            one per head and key channel
    per head: S <- diag(g) S,  u = b (v - S^T k),  S <- S + k u^T,  o = S^T q;   out = O [o / rms(o) * w * sigmoid(G_2 G_1 x)]

A sequence keeps the state, [heads, head_dim, v_head_dim] in fp32, and the last taps - 1 projected rows.  Kernels: csrc/ops_delta.hip;
the native engine runs the same weights (csrc/engine_stack.hip)."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.factory import zeros
from pygpukit_amd.ops._common import call
from pygpukit_amd.ops.basic import concat_axis0, conv_silu, delta_rule

from .linear import LinearBF16


class TapState:
    """What every mixer with taps over time and an fp32 state keeps of a sequence, dynamic or in the fixed cache."""

    cache_rows = False                    # the cache has no row per position
    kv_from = None
    _cache: tuple[GPUArray, ...] | None = None

    def _fresh(self, dtype) -> tuple[GPUArray, ...]:
        """The fp32 state, then the rows before the next token of every convolved projection."""
        raise NotImplementedError

    def _run(self, x: GPUArray, cache: tuple[GPUArray, ...], fresh: bool) -> GPUArray:
        raise NotImplementedError

    @staticmethod
    def _convolve(u: GPUArray, past: GPUArray, taps: GPUArray, bias: GPUArray | None = None) -> GPUArray:
        """silu of the convolved rows; `past` [taps - 1 (at least 1), channels] takes the last rows."""
        keep = taps.shape[0] - 1
        y = conv_silu(u, taps, past if keep else None, bias=bias)
        if keep:
            rows = u if u.shape[0] >= keep else concat_axis0(past, u)
            row = rows.nbytes // rows.shape[0]
            call("pgk_memcpy_d2d", past._p, rows.data_ptr() + (rows.shape[0] - keep) * row, keep * row, None)
        return y

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False) -> tuple[GPUArray, tuple | None]:
        """past / present: (state, rows before the next token ...)."""
        cache = self._fresh(x.dtype)
        if past_kv is not None:
            for a, b in zip(cache, past_kv):
                call("pgk_memcpy_d2d", a._p, b._p, a.nbytes, None)
        y = self._run(x, cache, past_kv is None)
        return y, (cache if use_cache else None)

    # ------------------------------------------------------------------ fixed cache
    def init_fixed_cache(self, max_seq_len: int, dtype: str = "bfloat16") -> None:
        self._cache = self._fresh(dtype)

    def fill_fixed_cache(self, present: tuple) -> None:
        for a, b in zip(self._cache, present):
            call("pgk_memcpy_d2d", a._p, b._p, a.nbytes, None)

    def cache_arrays(self) -> tuple[GPUArray, ...]:
        return self._cache

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int, *, out: GPUArray | None = None) -> GPUArray:
        return self.forward_fixed_cache_batch(x, position, context_len)

    def forward_fixed_cache_batch(self, x: GPUArray, start_position: int, context_len: int) -> GPUArray:
        """The state is that of the last token run: positions go on from there or start at 0."""
        if self._cache is None:
            raise RuntimeError("Call init_fixed_cache first")
        if context_len != start_position + x.shape[0]:
            raise ValueError(f"context_len {context_len} must end with the {x.shape[0]} tokens at position {start_position}")
        if start_position == 0:
            for a in self._cache[1:]:
                call("pgk_memcpy_d2d", a._p, zeros(a.shape, a.dtype)._p, a.nbytes, None)
        return self._run(x, self._cache, start_position == 0)


class ChannelDelta(TapState):
    def __init__(self, q_proj: GPUArray, k_proj: GPUArray, v_proj: GPUArray, o_proj: GPUArray, strength: GPUArray, decay_maps: tuple[GPUArray, GPUArray],
                 gate_maps: tuple[GPUArray, GPUArray], taps: tuple[GPUArray, GPUArray, GPUArray], decay: GPUArray, step_bias: GPUArray, head_norm: GPUArray, *,
                 num_heads: int, num_kv_heads: int, head_dim: int, v_head_dim: int, eps: float):
        """q_proj, k_proj [kv_heads * head_dim, hidden], v_proj [heads * v_head_dim, hidden], strength [heads, hidden]; maps: [rank, hidden] and
        [heads * (head_dim or v_head_dim), rank]; taps of q, k, v [taps, channels], the last for the token itself; float32: decay [heads]
        (rates), step_bias [heads * head_dim], head_norm [v_head_dim]."""
        self.num_heads, self.num_kv_heads, self.head_dim, self.v_head_dim, self.eps = num_heads, num_kv_heads, head_dim, v_head_dim, eps
        self.q_proj, self.k_proj, self.v_proj, self.o_proj, self.strength = (LinearBF16(w) for w in (q_proj, k_proj, v_proj, o_proj, strength))
        self.decay_maps, self.gate_maps = tuple(LinearBF16(w) for w in decay_maps), tuple(LinearBF16(w) for w in gate_maps)
        self.taps, self.decay, self.step_bias, self.head_norm = taps, decay, step_bias, head_norm

    def _fresh(self, dtype) -> tuple[GPUArray, ...]:
        keep = max(1, self.taps[0].shape[0] - 1)
        return (zeros((self.num_heads, self.head_dim, self.v_head_dim), "float32"), *(zeros((keep, t.shape[1]), dtype) for t in self.taps))

    def _run(self, x: GPUArray, cache: tuple[GPUArray, ...], fresh: bool) -> GPUArray:
        q, k, v = (self._convolve(p(x), past, t) for p, past, t in zip((self.q_proj, self.k_proj, self.v_proj), cache[1:], self.taps))
        y = delta_rule(q, k, v, self.decay_maps[1](self.decay_maps[0](x)), self.strength(x), self.gate_maps[1](self.gate_maps[0](x)), cache[0], decay=self.decay,
                       step_bias=self.step_bias, norm=self.head_norm, eps=self.eps, fresh=fresh)
        return self.o_proj(y)


__all__ = ["ChannelDelta", "TapState"]
