"""Transformer block (reference: src/pygpukit/llm/layers/block.py:18-57): pre-norm attention and MLP with
residual adds.  Layer-list models add a norm on each sublayer's output, a factor on its contribution and layers without MLP."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.ops.basic import add

from .attention import Attention
from .latent_attention import LatentAttention
from .mlp import MLP
from .norm import Norm


class TransformerBlock:
    def __init__(self, attn_norm: Norm, attn: "Attention | LatentAttention", mlp_norm: Norm | None, mlp: MLP | None,
                 post_attn_norm: Norm | None = None, post_mlp_norm: Norm | None = None, residual_mult: float = 1.0):
        self.attn_norm, self.attn, self.mlp_norm, self.mlp = attn_norm, attn, mlp_norm, mlp
        self.post_attn_norm, self.post_mlp_norm, self.residual_mult = post_attn_norm, post_mlp_norm, residual_mult

    def add_attn(self, x: GPUArray, y: GPUArray) -> GPUArray:
        return add(x, y) if self.post_attn_norm is None else self.post_attn_norm.add_to(x, y, self.residual_mult)

    def add_mlp(self, x: GPUArray) -> GPUArray:
        if self.mlp is None:
            return x
        y = self.mlp(self.mlp_norm(x))
        return add(x, y) if self.post_mlp_norm is None else self.post_mlp_norm.add_to(x, y, self.residual_mult)

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False) -> tuple[GPUArray, tuple | None]:
        attn_out, present_kv = self.attn(self.attn_norm(x), position_ids, past_kv, use_cache)
        return self.add_mlp(self.add_attn(x, attn_out)), present_kv

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int) -> GPUArray:
        """x [M, hidden] at positions position .. position + M - 1 against the layer's fixed cache."""
        attn = self.attn.forward_fixed_cache if x.shape[0] == 1 else self.attn.forward_fixed_cache_batch
        return self.add_mlp(self.add_attn(x, attn(self.attn_norm(x), position, context_len)))


__all__ = ["TransformerBlock"]
