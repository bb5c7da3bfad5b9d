"""Mixtures of experts.  MixtureOfExperts: a router picks `top` of the layer's SwiGLU feed-forwards for every token (csrc/moe.hip.h).

    s = sigmoid(R x);  chosen: the `top` largest s + correction (among the experts of the best `keep` groups, a group's value being the sum
    of its two largest);  out = sum over the chosen of  scale * s / (sum of the chosen s) * W_d (silu(W_g x) * W_u x)

TableExperts: a table of token ids names the experts, and a gated shared one runs for every token.

    out = 1 / top * sum over table[token] of W_d gelu(W_u x)  +  sigmoid(w . x) * W_d' gelu(W_u' x)"""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, int32
from pygpukit_amd.ops.basic import add_inplace, cast_bf16_to_f32, gelu_erf, head_gate, mixture_of_experts, table_experts

from .linear import LinearBF16


class MixtureOfExperts:
    def __init__(self, router: GPUArray, correction: GPUArray, gate_up: GPUArray, down: GPUArray, *, top: int, groups: int = 0, keep: int = 0, scale: float = 1.0):
        """router [experts, hidden]; correction float32 [experts]; gate_up [experts, 2 ff, hidden] (gate rows, then up rows of an expert);
        down [experts, hidden, ff]."""
        n, two_ff, hidden = gate_up.shape
        ff = two_ff // 2
        if router.shape != (n, hidden) or correction.shape != (n,) or down.shape != (n, hidden, ff):
            raise ValueError(f"MixtureOfExperts: router {router.shape}, correction {correction.shape}, gate_up {gate_up.shape}, down {down.shape}")
        self.router, self.correction, self.gate_up, self.down = router, correction, gate_up, down
        self.num_experts, self.intermediate_size, self.top, self.groups, self.keep, self.scale = n, ff, top, groups, keep, scale

    def __call__(self, x: GPUArray) -> GPUArray:
        """-> float32 [rows, hidden]"""
        return mixture_of_experts(x, self.router, self.correction, self.gate_up, self.down, top=self.top, groups=self.groups, keep=self.keep, scale=self.scale)


class TableExperts:
    needs_tokens = True

    def __init__(self, table: GPUArray, up: GPUArray, down: GPUArray, *, shared_up: GPUArray | None = None, shared_down: GPUArray | None = None, shared_gate: GPUArray | None = None):
        """table int32 [vocab, top]; up [experts, ff, hidden]; down [experts, hidden, ff]; the shared expert's up [ff', hidden], down
        [hidden, ff'] and gate [1, hidden], or none of them."""
        n, ff, hidden = up.shape
        if table.ndim != 2 or table.dtype != int32 or down.shape != (n, hidden, ff):
            raise ValueError(f"TableExperts: table {table.shape}, up {up.shape}, down {down.shape}")
        if shared_up is not None and (shared_up.shape[1] != hidden or shared_down.shape != (hidden, shared_up.shape[0]) or shared_gate.shape != (1, hidden)):
            raise ValueError(f"TableExperts: shared expert {shared_up.shape}, {shared_down.shape}, gate {shared_gate.shape}")
        self.table, self.up, self.down = table, up, down
        self.num_experts, self.intermediate_size, self.top = n, ff, table.shape[1]
        self.shared_up, self.shared_down, self.shared_gate = (None if w is None else LinearBF16(w) for w in (shared_up, shared_down, shared_gate))

    def __call__(self, x: GPUArray, tokens: GPUArray) -> GPUArray:
        """-> float32 [rows, hidden]; tokens int32 [rows]"""
        y = table_experts(x, tokens, self.table, self.up, self.down)
        if self.shared_up is not None:
            h = self.shared_up(x)
            z = self.shared_down(gelu_erf(h, out=h))
            head_gate(z.view((z.shape[0], 1, z.shape[1])), self.shared_gate(x))
            add_inplace(y, cast_bf16_to_f32(z) if z.dtype == bfloat16 else z)
        return y


__all__ = ["MixtureOfExperts", "TableExperts"]
