"""Transformer block (reference: src/pygpukit/llm/layers/block.py:18-57): pre-norm attention and MLP with
residual adds.  Layer-list models add a norm on each sublayer's output (with or without one on its input), a factor on its
contribution and layers without MLP, run mixer and experts side by side (ParallelBlock), or keep several residual streams (HyperBlock)."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import float16, float32
from pygpukit_amd.core.factory import from_numpy
from pygpukit_amd.ops.basic import add, add_inplace, bias_add_inplace, cast_bf16_to_f32, cast_f16_to_f32, cast_f32_to_bf16, cast_f32_to_f16, hyper_read, hyper_write

from .attention import Attention
from .delta import ChannelDelta
from .experts import MixtureOfExperts, TableExperts
from .latent_attention import LatentAttention
from .linear import LinearBF16
from .mlp import MLP
from .norm import Norm
from .recurrence import GatedRecurrence
from .state_space import StateSpace
from .talking_attention import TalkingAttention
from .window_attention import GatedWindowAttention

Mixer = Attention | LatentAttention | GatedWindowAttention | GatedRecurrence | ChannelDelta | StateSpace | TalkingAttention


def _narrow(x: GPUArray, dtype) -> GPUArray:
    return x if dtype == float32 else cast_f32_to_f16(x) if dtype == float16 else cast_f32_to_bf16(x)


def _wide(x: GPUArray) -> GPUArray:
    return x if x.dtype == float32 else cast_f16_to_f32(x) if x.dtype == float16 else cast_bf16_to_f32(x)


class TransformerBlock:
    def __init__(self, attn_norm: Norm | None, attn: Mixer, mlp_norm: Norm | None, mlp: MLP | None,
                 post_attn_norm: Norm | None = None, post_mlp_norm: Norm | None = None, residual_mult: float = 1.0):
        self.attn_norm, self.attn, self.mlp_norm, self.mlp = attn_norm, attn, mlp_norm, mlp
        self.post_attn_norm, self.post_mlp_norm, self.residual_mult = post_attn_norm, post_mlp_norm, residual_mult

    def _enter(self, norm: Norm | None, x: GPUArray, post: Norm | None) -> GPUArray:
        """What a sublayer reads: the norm of the stream, or without a norm the stream itself in the sublayer's element type."""
        if norm is not None:
            return norm(x)
        return _narrow(x, post.stream_dtype)

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


class ParallelBlock:
    """x += mixer(h) + experts(h) with h = norm(x): one norm, an fp32 stream, experts or none."""

    residual_mult = 1.0

    def __init__(self, norm: Norm, attn: Mixer, mlp: MixtureOfExperts | None):
        self.attn_norm, self.attn, self.mlp = norm, attn, mlp

    def _add(self, x: GPUArray, h: GPUArray, y: GPUArray) -> GPUArray:
        y = _wide(y)
        if self.mlp is not None:
            add_inplace(y, self.mlp(h))
        return add(x, y)

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None,
                 use_cache: bool = False, source_kv: tuple | None = None) -> tuple[GPUArray, tuple | None]:
        h = self.attn_norm(x)
        y, present_kv = self.attn(h, position_ids, past_kv, use_cache)
        return self._add(x, h, y), present_kv

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int) -> GPUArray:
        h = self.attn_norm(x)
        return self._add(x, h, self.attn.forward_fixed_cache_batch(h, position, context_len))


class HyperConnection:
    """How a sublayer is tied to the residual streams: reads sum_a read[a] x_a, writes x_b <- sum_a mix[a, b] x_a + write[b] y (float32)."""

    def __init__(self, read: GPUArray, write: GPUArray, mix: GPUArray):
        n = read.size
        if read.shape != (n,) or write.shape != (n,) or mix.shape != (n, n) or any(w.dtype != float32 for w in (read, write, mix)):
            raise ValueError(f"HyperConnection: {read.shape}, {write.shape}, {mix.shape}")
        self.read, self.write, self.mix = read, write, mix


class HyperBlock:
    """Mixer, then feed-forward (an MLP, experts chosen by token, or none), each with a norm of its own and a HyperConnection, on float32
    streams [n, streams, hidden]."""

    residual_mult = 1.0

    def __init__(self, attn_norm: Norm, attn: Mixer, attn_hyper: HyperConnection, mlp_norm: Norm | None, mlp: MLP | TableExperts | None, mlp_hyper: HyperConnection | None):
        self.attn_norm, self.attn, self.attn_hyper, self.mlp_norm, self.mlp, self.mlp_hyper = attn_norm, attn, attn_hyper, mlp_norm, mlp, mlp_hyper

    @property
    def needs_tokens(self) -> bool:
        return getattr(self.mlp, "needs_tokens", False)

    @staticmethod
    def _write(x: GPUArray, y: GPUArray, h: HyperConnection) -> GPUArray:
        return hyper_write(x, y, h.write, h.mix)

    def _feed_forward(self, x: GPUArray, tokens: GPUArray | None) -> GPUArray:
        if self.mlp is None:
            return x
        h = self.mlp_norm(hyper_read(x, self.mlp_hyper.read))
        return self._write(x, self.mlp(h, tokens) if self.needs_tokens else self.mlp(h), self.mlp_hyper)

    def __call__(self, x: GPUArray, position_ids: list[int] | None = None, past_kv: tuple | None = None, use_cache: bool = False,
                 source_kv: tuple | None = None, tokens: GPUArray | None = None) -> tuple[GPUArray, tuple | None]:
        extra = {} if source_kv is None else {"source_kv": source_kv}
        y, present_kv = self.attn(self.attn_norm(hyper_read(x, self.attn_hyper.read)), position_ids, past_kv, use_cache, **extra)
        return self._feed_forward(self._write(x, y, self.attn_hyper), tokens), present_kv

    def forward_fixed_cache(self, x: GPUArray, position: int, context_len: int, tokens: GPUArray | None = None) -> GPUArray:
        y = self.attn.forward_fixed_cache_batch(self.attn_norm(hyper_read(x, self.attn_hyper.read)), position, context_len)
        return self._feed_forward(self._write(x, y, self.attn_hyper), tokens)


class LoopInput:
    """What a pass of a looped stretch starts with: x <- W_x x + W_e e + step[pass], e the embedding rows."""

    def __init__(self, weight: GPUArray, step: GPUArray):
        """weight [hidden, 2 hidden]; step float32 [passes, hidden]."""
        hidden = weight.shape[0]
        if weight.shape != (hidden, 2 * hidden) or step.ndim != 2 or step.shape[1] != hidden or step.dtype != float32:
            raise ValueError(f"LoopInput: weight {weight.shape}, step {step.shape}")
        self.weight, self.step = weight, step
        self._halves: tuple[LinearBF16, LinearBF16] | None = None

    def __call__(self, x: GPUArray, e: GPUArray, t: int) -> GPUArray:
        hidden, dt = x.shape[1], self.weight.dtype
        if self._halves is None:
            w = self.weight.to_numpy()
            self._halves = tuple(LinearBF16(from_numpy(w[:, i * hidden:(i + 1) * hidden])) for i in (0, 1))
        y = _wide(self._halves[0](_narrow(x, dt)))
        add_inplace(y, _wide(self._halves[1](_narrow(e, dt))))
        bias_add_inplace(y, self.step._view(t * hidden, (hidden,)))
        return y


__all__ = ["TransformerBlock", "ParallelBlock", "HyperBlock", "HyperConnection", "LoopInput"]
