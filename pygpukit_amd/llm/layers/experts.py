"""Mixture of experts: a router picks `top` of the layer's SwiGLU feed-forwards for every token (csrc/moe.hip.h).

    s = sigmoid(R x);  chosen: the `top` largest s + correction (among the experts of the best `keep` groups, a group's value being the sum
    of its two largest);  out = sum over the chosen of  scale * s / (sum of the chosen s) * W_d (silu(W_g x) * W_u x)"""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.ops.basic import mixture_of_experts


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


__all__ = ["MixtureOfExperts"]
