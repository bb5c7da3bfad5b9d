"""Transformer block (reference: src/pygpukit/llm/layers/block.py:18-57): pre-norm attention and MLP with
residual adds.  Layer-list models add a norm on each sublayer's output (with or without one on its input), a factor on its
contribution and layers without MLP."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import float16, float32
from pygpukit_amd.ops.basic import add, cast_f32_to_bf16, cast_f32_to_f16

from .attention import Attention
from .latent_attention import LatentAttention
from .mlp import MLP
from .norm import Norm
from .recurrence import GatedRecurrence
from .window_attention import GatedWindowAttention

Mixer = Attention | LatentAttention | GatedWindowAttention | GatedRecurrence


class TransformerBlock:
    def __init__(self, attn_norm: Norm | None, attn: Mixer, mlp_norm: Norm | None, mlp: MLP | None,
                 post_attn_norm: Norm | None = None, post_mlp_norm: Norm | None = None, residual_mult: float = 1.0):
        self.attn_norm, self.attn, self.mlp_norm, self.mlp = attn_norm, attn, mlp_norm, mlp
        self.post_attn_norm, self.post_mlp_norm, self.residual_mult = post_attn_norm, post_mlp_norm, residual_mult

    def _enter(self, norm: Norm | None, x: GPUArray, post: Norm | None) -> GPUArray:
        """What a sublayer reads: the norm of the stream, or without a norm the stream itself in the sublayer's element type."""
        if norm is not None:
            return norm(x)
        dt = post.stream_dtype
        return x if dt == float32 else cast_f32_to_f16(x) if dt == float16 else cast_f32_to_bf16(x)

    def add_attn(self, x: GPUArray, y: GPUArray) -> GPUArray:
        return add(x, y) if self.post_attn_norm is None else self.post_attn_norm.add_to(x, y, self.residual_mult)

    def add_mlp(self, x: GPUArray) -> GPUArray:
        if self.mlp is None:
            return x
        y = self.mlp(self._enter(self.mlp_norm, x, self.post_mlp_norm))
        return add(x, y) if self.post_mlp_norm is None else self.post_mlp_norm.add_to(x, y, self.residual_mult)

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False, source_kv: tuple | None = None) -> tuple[GPUArray, tuple | None]:
        """source_kv: what the layer this one takes its keys and values from has just returned."""
        h = self._enter(self.attn_norm, x, self.post_attn_norm)
        extra = {} if source_kv is None else {"source_kv": source_kv}
        attn_out, present_kv = self.attn(h, position_ids, past_kv, use_cache, **extra)
        return self.add_mlp(self.add_attn(x, attn_out)), present_kv

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int) -> GPUArray:
        """x [M, hidden] at positions position .. position + M - 1 against the layer's fixed cache."""
        attn = self.attn.forward_fixed_cache if x.shape[0] == 1 else self.attn.forward_fixed_cache_batch
        return self.add_mlp(self.add_attn(x, attn(self._enter(self.attn_norm, x, self.post_attn_norm), position, context_len)))


__all__ = ["TransformerBlock"]
