"""Hyper-connections: several fp32 residual streams instead of one."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import float32
from pygpukit_amd.ops._common import call, check_out, validate_float


def hyper_read(streams: GPUArray, weights: GPUArray | None = None, *, out: GPUArray | None = None) -> GPUArray:
    """streams float32 [n, streams, width] -> sum_a weights[a] x_a [n, width] (no weights: the plain sum)."""
    if streams.ndim != 3 or streams.dtype != float32 or (weights is not None and (weights.shape != (streams.shape[1],) or weights.dtype != float32)):
        raise ValueError(f"hyper_read: streams {streams.shape} and their weights are float32")
    n, s, w = streams.shape
    o = check_out(out, (n, w), float32, "hyper_read")
    call("pgk_hyper_read", streams._p, weights._p if weights is not None else None, o._p, n, s, w, None)
    return o


def hyper_write(streams: GPUArray, y: GPUArray, out_weights: GPUArray, mix: GPUArray) -> GPUArray:
    """x_b <- sum_a mix[a, b] x_a + out_weights[b] y, in place: streams float32 [n, streams, width], y [n, width] of any float type."""
    validate_float(y, "hyper_write")
    if streams.ndim != 3 or streams.dtype != float32 or y.shape != (streams.shape[0], streams.shape[2]):
        raise ValueError(f"hyper_write: streams {streams.shape}, rows {y.shape}")
    n, s, w = streams.shape
    if out_weights.shape != (s,) or mix.shape != (s, s) or out_weights.dtype != float32 or mix.dtype != float32:
        raise ValueError(f"hyper_write: weights {out_weights.shape}, {mix.shape} of {s} streams")
    call("pgk_hyper_write", streams._p, y._p, out_weights._p, mix._p, n, s, w, y.dtype.code, None)
    return streams


__all__ = ["hyper_read", "hyper_write"]
