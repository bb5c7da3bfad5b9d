"""State-space duality (Mamba-2): a linear recurrence with one decay per head and row.

    z | x | B | C | t = W_in h;   x, B, C = silu(taps over time + bias);   t <- softplus(t + step_bias)
    per head: S <- exp(-decay t) S + t B x^T,  y = S^T C + skip x;   out = O [rms in norm_groups parts of (y * silu(z)) * w]

A sequence keeps the state, [heads, state, v_head_dim] in fp32, and the last taps - 1 rows before the taps.  Kernels:
csrc/ops_recurrence.hip; the native engine runs the same weights (csrc/engine_stack.hip)."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.factory import zeros
from pygpukit_amd.ops.basic import state_space

from .delta import TapState
from .linear import LinearBF16


class StateSpace(TapState):
    def __init__(self, in_proj: tuple[GPUArray, GPUArray, GPUArray], o_proj: GPUArray, taps: GPUArray, taps_bias: GPUArray, decay: GPUArray, step_bias: GPUArray,
                 skip: GPUArray, out_norm: GPUArray, *, num_heads: int, num_groups: int, state_dim: int, v_head_dim: int, norm_groups: int, eps: float):
        """in_proj: rows of z [heads * v_head_dim, hidden], of x | B | C [heads * v_head_dim + 2 groups * state_dim, hidden] and of t [heads, hidden];
        taps [taps, channels of x | B | C]; float32: taps_bias [channels], decay (rates), step_bias, skip [heads], out_norm [heads * v_head_dim]."""
        self.num_heads, self.num_groups, self.head_dim, self.v_head_dim, self.norm_groups, self.eps = num_heads, num_groups, state_dim, v_head_dim, norm_groups, eps
        self.z_proj, self.xbc_proj, self.t_proj = (LinearBF16(w) for w in in_proj)
        self.o_proj = LinearBF16(o_proj)
        self.taps, self.taps_bias, self.decay, self.step_bias, self.skip, self.out_norm = taps, taps_bias, decay, step_bias, skip, out_norm

    def _fresh(self, dtype) -> tuple[GPUArray, ...]:
        return zeros((self.num_heads, self.head_dim, self.v_head_dim), "float32"), zeros((max(1, self.taps.shape[0] - 1), self.taps.shape[1]), dtype)

    def _run(self, x: GPUArray, cache: tuple[GPUArray, ...], fresh: bool) -> GPUArray:
        xbc = self._convolve(self.xbc_proj(x), cache[1], self.taps, self.taps_bias)
        y = state_space(xbc, self.z_proj(x), self.t_proj(x), cache[0], groups=self.num_groups, decay=self.decay, step_bias=self.step_bias, skip=self.skip, norm=self.out_norm,
                        norm_groups=self.norm_groups, eps=self.eps, fresh=fresh)
        return self.o_proj(y)


__all__ = ["StateSpace"]
