"""Gated linear recurrence (HGRN2): linear attention whose forget gate also decides what is written.

    q = silu(Q x),  v = V x,  f = l + (1 - l) sigmoid(F x + b)      per head: S <- diag(f) S + (1 - f) v^T,  o = S^T q
    out = O [o_a / rms(o_a) * w]

The state, [heads, head_dim, v_head_dim] in fp32, is all that a sequence keeps.  This is the operator-surface form; the native engine's
is csrc/engine_stack.hip with the kernels of csrc/ops_recurrence.hip."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.factory import zeros
from pygpukit_amd.ops._common import call
from pygpukit_amd.ops.basic import gated_recurrence

from .linear import LinearBF16


class GatedRecurrence:
    cache_rows = False                    # the cache has no row per position
    kv_from = None

    def __init__(self, q_proj: GPUArray, forget_proj: GPUArray, v_proj: GPUArray, o_proj: GPUArray, forget_bias: GPUArray, lower: GPUArray, head_norm: GPUArray, *,
                 num_heads: int, head_dim: int, v_head_dim: int, eps: float):
        """q_proj, forget_proj [heads * head_dim, hidden], v_proj [heads * v_head_dim, hidden], o_proj [hidden, heads * v_head_dim];
        float32: forget_bias and lower [heads * head_dim], head_norm [v_head_dim]."""
        self.num_heads, self.head_dim, self.v_head_dim, self.eps = num_heads, head_dim, v_head_dim, eps
        self.q_proj, self.forget_proj, self.v_proj, self.o_proj = (LinearBF16(w) for w in (q_proj, forget_proj, v_proj, o_proj))
        self.forget_bias, self.lower, self.head_norm = forget_bias, lower, head_norm
        self._state: GPUArray | None = None

    def _new_state(self) -> GPUArray:
        return zeros((self.num_heads, self.head_dim, self.v_head_dim), "float32")

    def _run(self, x: GPUArray, state: GPUArray, fresh: bool) -> GPUArray:
        y = gated_recurrence(self.q_proj(x), self.forget_proj(x), self.v_proj(x), self.lower, state, f_bias=self.forget_bias, norm=self.head_norm, eps=self.eps,
                             fresh=fresh)
        return self.o_proj(y)

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False) -> tuple[GPUArray, tuple | None]:
        """past / present: (state,)."""
        state = self._new_state()
        if past_kv is not None:
            call("pgk_memcpy_d2d", state._p, past_kv[0]._p, state.nbytes, None)
        y = self._run(x, state, past_kv is None)
        return y, ((state,) if use_cache else None)

    # ------------------------------------------------------------------ fixed cache
    def init_fixed_cache(self, max_seq_len: int, dtype: str = "bfloat16") -> None:
        self._state = self._new_state()

    def fill_fixed_cache(self, present: tuple) -> None:
        call("pgk_memcpy_d2d", self._state._p, present[0]._p, self._state.nbytes, None)

    def cache_arrays(self) -> tuple[GPUArray, ...]:
        return (self._state,)

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int, *, out: GPUArray | None = None) -> GPUArray:
        return self.forward_fixed_cache_batch(x, position, context_len)

    def forward_fixed_cache_batch(self, x: GPUArray, start_position: int, context_len: int) -> GPUArray:
        """The state is that of the last token run: positions go on from there or start at 0."""
        if self._state is None:
            raise RuntimeError("Call init_fixed_cache first")
        if context_len != start_position + x.shape[0]:
            raise ValueError(f"context_len {context_len} must end with the {x.shape[0]} tokens at position {start_position}")
        return self._run(x, self._state, start_position == 0)


__all__ = ["GatedRecurrence"]
