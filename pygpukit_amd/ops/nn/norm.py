"""Row normalisations (reference: src/pygpukit/ops/nn/norm.py:16-218 -> ops.cuh:143-155)."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import float32
from pygpukit_amd.ops._common import call, check_out, validate_float, validate_same_dtype


def _check(input: GPUArray, gamma: GPUArray, name: str) -> None:
    validate_float(input, name)
    if input.ndim != 2:
        raise ValueError(f"{name} expects 2D input [batch, features], got {input.ndim}D")
    if gamma.ndim != 1:
        raise ValueError(f"{name} expects 1D gamma")
    validate_same_dtype(input, gamma, name)
    if input.shape[1] != gamma.shape[0]:
        raise ValueError(f"{name}: input features ({input.shape[1]}) must match gamma size ({gamma.shape[0]})")


def rmsnorm(input: GPUArray, gamma: GPUArray, eps: float = 1e-5, *, out: GPUArray | None = None) -> GPUArray:
    _check(input, gamma, "rmsnorm")
    o = check_out(out, input.shape, input.dtype, "rmsnorm")
    call("pgk_rmsnorm", input._p, gamma._p, o._p, input.shape[0], input.shape[1], eps, input.dtype.code, None)
    return o


def rmsnorm_f32(input: GPUArray, weight: GPUArray, eps: float = 1e-5, *, dtype=float32, out: GPUArray | None = None) -> GPUArray:
    """RMSNorm of an fp32 stream with an fp32 weight; the result leaves in `dtype`."""
    _check(input, weight, "rmsnorm_f32")
    if input.dtype != float32:
        raise ValueError("rmsnorm_f32: input and weight must be float32")
    o = check_out(out, input.shape, dtype, "rmsnorm_f32")
    call("pgk_rmsnorm_f32", input._p, weight._p, o._p, input.shape[0], input.shape[1], eps, o.dtype.code, None)
    return o


def group_norm_f32(input: GPUArray, weight: GPUArray, groups: int, eps: float = 1e-5, *, dtype=float32, out: GPUArray | None = None) -> GPUArray:
    """RMS norm of an fp32 stream in `groups` equal consecutive parts, each over its own root mean square, with an fp32 weight."""
    _check(input, weight, "group_norm_f32")
    if input.dtype != float32 or groups < 1 or input.shape[1] % groups:
        raise ValueError(f"group_norm_f32: float32 rows of {input.shape[1]} in {groups} groups")
    o = check_out(out, input.shape, dtype, "group_norm_f32")
    call("pgk_group_norm_f32", input._p, weight._p, o._p, input.shape[0], input.shape[1], int(groups), eps, o.dtype.code, None)
    return o


def layernorm_f32(input: GPUArray, weight: GPUArray, eps: float = 1e-5, *, dtype=float32, out: GPUArray | None = None) -> GPUArray:
    """Layer norm (no bias) of an fp32 stream with an fp32 weight; the result leaves in `dtype`."""
    _check(input, weight, "layernorm_f32")
    if input.dtype != float32:
        raise ValueError("layernorm_f32: input and weight must be float32")
    o = check_out(out, input.shape, dtype, "layernorm_f32")
    call("pgk_layernorm_f32", input._p, weight._p, o._p, input.shape[0], input.shape[1], eps, o.dtype.code, None)
    return o


def rmsnorm_add_f32(stream: GPUArray, y: GPUArray, weight: GPUArray, eps: float = 1e-5, mult: float = 1.0) -> GPUArray:
    """stream += mult * rmsnorm(y) * weight in place (fp32 stream and weight, y in any float type)."""
    validate_float(y, "rmsnorm_add_f32")
    if stream.dtype != float32 or weight.dtype != float32:
        raise ValueError("rmsnorm_add_f32: stream and weight must be float32")
    if stream.ndim != 2 or stream.shape != y.shape or weight.shape != (stream.shape[1],):
        raise ValueError(f"rmsnorm_add_f32: shapes {stream.shape}, {y.shape}, {weight.shape} do not match")
    call("pgk_rmsnorm_add_f32", stream._p, y._p, weight._p, stream.shape[0], stream.shape[1], eps, mult, y.dtype.code, None)
    return stream


def layernorm(input: GPUArray, gamma: GPUArray, beta: GPUArray, eps: float = 1e-5, *, out: GPUArray | None = None) -> GPUArray:
    _check(input, gamma, "layernorm")
    if beta.shape != gamma.shape or beta.dtype != gamma.dtype:
        raise ValueError("layernorm: beta must match gamma")
    o = check_out(out, input.shape, input.dtype, "layernorm")
    call("pgk_layernorm", input._p, gamma._p, beta._p, o._p, input.shape[0], input.shape[1], eps, input.dtype.code, None)
    return o
