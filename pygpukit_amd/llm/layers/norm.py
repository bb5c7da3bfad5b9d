"""Norm layer (reference: src/pygpukit/llm/layers/norm.py:18-39)."""

from __future__ import annotations

from typing import Literal

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import DataType, float32
from pygpukit_amd.ops.basic import group_norm_f32, layernorm, layernorm_f32, rmsnorm, rmsnorm_add_f32, rmsnorm_f32


class Norm:
    """`stream_dtype` set: the norm of an fp32 residual stream - `weight` is fp32 with any offset already added, the result leaves in
    stream_dtype, and add_to() is the norm-then-residual-add of a sublayer's output.  `groups`: equal parts of the row, each over its
    own root mean square."""

    def __init__(self, weight: GPUArray, bias: GPUArray | None = None,
                 norm_type: Literal["rmsnorm", "layernorm"] = "rmsnorm", eps: float = 1e-5, stream_dtype: DataType | None = None,
                 groups: int = 1):
        self.weight, self.bias, self.norm_type, self.eps = weight, bias, norm_type, eps
        self.stream_dtype, self.groups = stream_dtype, groups
        if stream_dtype is not None and (bias is not None or weight.dtype != float32):
            raise ValueError("an fp32-stream norm has a float32 weight and no bias")
        if groups != 1 and (stream_dtype is None or norm_type != "rmsnorm"):
            raise ValueError("norms in groups are RMS norms of an fp32 stream")

    def add_to(self, stream: GPUArray, y: GPUArray, mult: float = 1.0) -> GPUArray:
        """stream += mult * norm(y), in place."""
        if self.norm_type != "rmsnorm" or self.groups != 1:
            raise NotImplementedError("a layer norm, or one in groups, of a sublayer's output")
        return rmsnorm_add_f32(stream, y, self.weight, self.eps, mult)

    def __call__(self, x: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
        if self.stream_dtype is not None:
            if self.norm_type == "layernorm":
                return layernorm_f32(x, self.weight, self.eps, dtype=self.stream_dtype, out=out)
            if self.groups != 1:
                return group_norm_f32(x, self.weight, self.groups, self.eps, dtype=self.stream_dtype, out=out)
            return rmsnorm_f32(x, self.weight, self.eps, dtype=self.stream_dtype, out=out)
        if self.norm_type == "rmsnorm":
            return rmsnorm(x, self.weight, self.eps, out=out)
        if self.bias is None:
            raise ValueError("LayerNorm requires bias")
        return layernorm(x, self.weight, self.bias, self.eps, out=out)


__all__ = ["Norm"]
