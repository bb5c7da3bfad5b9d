"""Operators over time: short causal convolution, gated linear recurrence."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32
from pygpukit_amd.ops._common import call, check_out, validate_float


def short_conv(u: GPUArray, weight: GPUArray, past: GPUArray | None = None, *, out: GPUArray | None = None) -> GPUArray:
    """y_t = sum_j weight[:, j] * u_(t - taps + 1 + j) per channel: u [n, channels], weight [channels, taps], past [taps - 1, channels] =
    the rows before u (None: zeros)."""
    validate_float(u, "short_conv")
    if u.ndim != 2 or weight.ndim != 2 or weight.shape[0] != u.shape[1] or weight.dtype != u.dtype:
        raise ValueError(f"short_conv: u {u.shape} and weight {weight.shape} do not match")
    taps = weight.shape[1]
    if past is not None and (past.shape != (taps - 1, u.shape[1]) or past.dtype != u.dtype):
        raise ValueError(f"short_conv: past {past.shape}, expected {(taps - 1, u.shape[1])}")
    o = check_out(out, u.shape, u.dtype, "short_conv")
    call("pgk_short_conv", u._p, past._p if past is not None and taps > 1 else None, weight._p, o._p, u.shape[0], u.shape[1], taps, u.dtype.code, None)
    return o


def gated_recurrence(q: GPUArray, f: GPUArray, v: GPUArray, lower: GPUArray, state: GPUArray, *, f_bias: GPUArray | None = None, norm: GPUArray | None = None,
                     eps: float = 1e-5, fresh: bool = False, out: GPUArray | None = None) -> GPUArray:
    """n rows of one sequence: q, f [n, heads * dim] (before their activations), v [n, heads * vdim], state float32 [heads, dim, vdim],
    updated in place (fresh: it starts at zero).  With the gate g = lower + (1 - lower) sigmoid(f + f_bias):
    S <- diag(g) S + (1 - g) v^T, o = S^T silu(q), and with `norm` [vdim] o / rms(o) * norm per head.  -> [n, heads * vdim]."""
    if q.dtype not in (float32, bfloat16) or f.dtype != q.dtype or v.dtype != q.dtype:
        raise ValueError("gated_recurrence: q, f, v must be float32 or bfloat16 of one dtype")
    if state.ndim != 3 or state.dtype != float32:
        raise ValueError("gated_recurrence: state must be float32 [heads, dim, vdim]")
    heads, dim, vdim = state.shape
    n = q.shape[0]
    if q.shape != (n, heads * dim) or f.shape != q.shape or v.shape != (n, heads * vdim):
        raise ValueError(f"gated_recurrence: shapes {q.shape}, {f.shape}, {v.shape} do not match the state {state.shape}")
    for name, a, size in (("lower", lower, heads * dim), ("f_bias", f_bias, heads * dim), ("norm", norm, vdim)):
        if a is not None and (a.size != size or a.dtype != float32):
            raise ValueError(f"gated_recurrence: {name} must be float32 of {size} elements")
    o = check_out(out, (n, heads * vdim), q.dtype, "gated_recurrence")
    opt = lambda a: a._p if a is not None else None  # noqa: E731
    call("pgk_gated_recurrence", q._p, f._p, v._p, opt(f_bias), lower._p, opt(norm), state._p, o._p, n, int(fresh), heads, dim, vdim, float(eps), q.dtype.code, None)
    return o
