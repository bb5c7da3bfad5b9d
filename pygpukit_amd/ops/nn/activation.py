"""Activations (reference: src/pygpukit/ops/nn/activation.py:16-225 -> ops.cuh:136,176-191)."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32
from pygpukit_amd.ops._common import call, check_out, validate_float

_ACT = {"silu": 0, "gelu": 1, "sigmoid": 2, "tanh": 3, "relu2": 4}


def _act(a: GPUArray, name: str, out: GPUArray | None) -> GPUArray:
    validate_float(a, name)
    o = check_out(out, a.shape, a.dtype, name)
    call("pgk_activation", a._p, o._p, a.size, _ACT[name], a.dtype.code, None)
    return o


def silu(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    """x / (1 + exp(-x)); `out` may alias the input."""
    return _act(a, "silu", out)


def gelu(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    """tanh GELU with the reference's constants 0.7978845608 / 0.044715."""
    return _act(a, "gelu", out)


def sigmoid(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    return _act(a, "sigmoid", out)


def tanh(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    return _act(a, "tanh", out)


def relu2(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    return _act(a, "relu2", out)


def gelu_erf(a: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    """The exact gelu, z / 2 (1 + erf(z / sqrt 2)); `out` may alias the input."""
    validate_float(a, "gelu_erf")
    o = check_out(out, a.shape, a.dtype, "gelu_erf")
    call("pgk_gelu_erf", a._p, o._p, a.size, a.dtype.code, None)
    return o


def soft_cap(a: GPUArray, cap: float, *, out: GPUArray | None = None) -> GPUArray:
    """cap * tanh(a / cap); `out` may alias the input."""
    validate_float(a, "soft_cap")
    if not cap > 0:
        raise ValueError(f"soft_cap: cap {cap}")
    o = check_out(out, a.shape, a.dtype, "soft_cap")
    call("pgk_soft_cap", a._p, o._p, a.size, float(cap), a.dtype.code, None)
    return o


def poly_norm(z: GPUArray, act: GPUArray, eps: float, *, out: GPUArray | None = None) -> GPUArray:
    """Rows of a r(z) + b r(z^2) + c r(z^3) + e with r(x) = x / sqrt(mean(x^2) + eps) and act = float32 (a, b, c, e)."""
    if z.ndim != 2 or z.dtype not in (float32, bfloat16) or act.dtype != float32 or act.size != 4:
        raise ValueError("poly_norm: float32 or bfloat16 [rows, width] and four float32 numbers")
    o = check_out(out, z.shape, z.dtype, "poly_norm")
    call("pgk_poly_norm", z._p, o._p, z.shape[0], z.shape[1], act._p, float(eps), z.dtype.code, None)
    return o


def xielu(a: GPUArray, pos: float, neg: float, *, out: GPUArray | None = None) -> GPUArray:
    """z > 0: pos * z^2 + z / 2;  z <= 0: neg * (exp(z) - 1 - z) + z / 2.  `out` may alias the input."""
    validate_float(a, "xielu")
    o = check_out(out, a.shape, a.dtype, "xielu")
    call("pgk_xielu", a._p, o._p, a.size, float(pos), float(neg), a.dtype.code, None)
    return o
