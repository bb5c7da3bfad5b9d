"""Operators over time: short causal convolution, linear recurrences, gated delta rule."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32
from pygpukit_amd.ops._common import call, check_out, validate_float
from pygpukit_amd.ops.tensor import cast_bf16_to_f32, pad_2d


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


def conv_silu(u: GPUArray, taps: GPUArray, past: GPUArray | None = None, *, bias: GPUArray | None = None, out: GPUArray | None = None) -> GPUArray:
    """silu of the short convolution of u [n, channels] with taps [taps, channels] (the last row multiplies the token itself) and bias (float32
    [channels]); past [taps - 1, channels]: the rows before u (None: zeros)."""
    if u.dtype not in (float32, bfloat16) or u.ndim != 2 or taps.ndim != 2 or taps.shape[1] != u.shape[1] or taps.dtype != u.dtype:
        raise ValueError(f"conv_silu: u {u.shape} ({u.dtype}) and taps {taps.shape} ({taps.dtype}) do not match")
    if past is not None and (past.shape != (taps.shape[0] - 1, u.shape[1]) or past.dtype != u.dtype):
        raise ValueError(f"conv_silu: past {past.shape}, expected {(taps.shape[0] - 1, u.shape[1])}")
    if bias is not None and (bias.size != u.shape[1] or bias.dtype != float32):
        raise ValueError(f"conv_silu: bias must be float32 of {u.shape[1]} elements")
    o = check_out(out, u.shape, u.dtype, "conv_silu")
    n, ch = u.shape
    if ch % 4:                                                 # the kernel takes four channels at a time
        p = -(-ch // 4) * 4
        y = conv_silu(pad_2d(u, n, p), pad_2d(taps, taps.shape[0], p), None if past is None else pad_2d(past, past.shape[0], p),
                      bias=None if bias is None else pad_2d(bias.view((1, ch)), 1, p))
        call("pgk_pad_2d", y._p, o._p, n, p, n, ch, u.dtype.code, None)
        return o
    call("pgk_conv_silu", u._p, _opt(past), taps._p, _opt(bias), o._p, u.shape[0], u.shape[1], taps.shape[0], u.dtype.code, None)
    return o


def _opt(a: GPUArray | None):
    return a._p if a is not None else None


def _check_f32(name: str, **sizes) -> None:
    for what, (a, size) in sizes.items():
        if a.size != size or a.dtype != float32:
            raise ValueError(f"{name}: {what} must be float32 of {size} elements")


def delta_rule(q: GPUArray, k: GPUArray, v: GPUArray, z: GPUArray, strength: GPUArray, gate: GPUArray, state: GPUArray, *, decay: GPUArray, step_bias: GPUArray,
               norm: GPUArray, eps: float = 1e-5, fresh: bool = False, out: GPUArray | None = None) -> GPUArray:
    """n rows of one sequence (pgk_delta_rule): q, k [n, kv_heads * dim], v [n, heads * vdim] after taps and activation, decay logits z [n, heads * dim],
    strength [n, heads] and gate [n, heads * vdim] before their sigmoid, state float32 [heads, dim, vdim], updated in place (fresh: it starts
    at zero).  q, k of unit length, g = exp(-decay softplus(z + step_bias)): S <- diag(g) S, u = b (v - S^T k), S <- S + k u^T, o = S^T q;
    -> o / rms(o) * norm * sigmoid(gate), [n, heads * vdim]."""
    if q.dtype not in (float32, bfloat16) or any(a.dtype != q.dtype for a in (k, v, strength, gate)):
        raise ValueError("delta_rule: q, k, v, strength, gate must be float32 or bfloat16 of one dtype")
    if state.ndim != 3 or state.dtype != float32:
        raise ValueError("delta_rule: state must be float32 [heads, dim, vdim]")
    heads, dim, vdim = state.shape
    n = q.shape[0]
    kv = q.shape[1] // dim
    if q.shape != (n, kv * dim) or kv < 1 or heads % kv or k.shape != q.shape or v.shape != (n, heads * vdim) or z.shape != (n, heads * dim) or strength.shape != (n, heads) or gate.shape != v.shape:
        raise ValueError(f"delta_rule: shapes {q.shape}, {k.shape}, {v.shape}, {z.shape}, {strength.shape}, {gate.shape} do not match the state {state.shape}")
    _check_f32("delta_rule", decay=(decay, heads), step_bias=(step_bias, heads * dim), norm=(norm, vdim))
    z = z if z.dtype == float32 else cast_bf16_to_f32(z)
    o = check_out(out, v.shape, q.dtype, "delta_rule")
    call("pgk_delta_rule", q._p, k._p, v._p, z._p, strength._p, gate._p, decay._p, step_bias._p, norm._p, state._p, o._p, n, int(fresh), heads, kv, dim, vdim, float(eps),
         q.dtype.code, None)
    return o


def state_space(xbc: GPUArray, z: GPUArray, t: GPUArray, state: GPUArray, *, groups: int, decay: GPUArray, step_bias: GPUArray, skip: GPUArray, norm: GPUArray,
                norm_groups: int = 1, eps: float = 1e-5, fresh: bool = False, out: GPUArray | None = None) -> GPUArray:
    """n rows of one sequence (pgk_state_space): xbc [n, heads * vdim | groups * dim | groups * dim] after taps and activation, z [n, heads * vdim],
    t [n, heads], state float32 [heads, dim, vdim], updated in place.  t <- softplus(t + step_bias): S <- exp(-decay t) S + t B x^T,
    y = S^T C + skip x; -> rms norm in norm_groups parts of y silu(z), times norm, [n, heads * vdim]."""
    if xbc.dtype not in (float32, bfloat16) or z.dtype != xbc.dtype or t.dtype != xbc.dtype:
        raise ValueError("state_space: xbc, z, t must be float32 or bfloat16 of one dtype")
    if state.ndim != 3 or state.dtype != float32:
        raise ValueError("state_space: state must be float32 [heads, dim, vdim]")
    heads, dim, vdim = state.shape
    n = xbc.shape[0]
    if groups < 1 or heads % groups or xbc.shape != (n, heads * vdim + 2 * groups * dim) or z.shape != (n, heads * vdim) or t.shape != (n, heads):
        raise ValueError(f"state_space: shapes {xbc.shape}, {z.shape}, {t.shape} do not match the state {state.shape} in {groups} groups")
    _check_f32("state_space", decay=(decay, heads), step_bias=(step_bias, heads), skip=(skip, heads), norm=(norm, heads * vdim))
    o = check_out(out, z.shape, xbc.dtype, "state_space")
    call("pgk_state_space", xbc._p, z._p, t._p, decay._p, step_bias._p, skip._p, norm._p, state._p, o._p, n, int(fresh), heads, int(groups), dim, vdim, int(norm_groups),
         float(eps), xbc.dtype.code, None)
    return o
