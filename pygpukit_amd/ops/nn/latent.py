"""Operators of latent attention: cache rows with a rotated part, rotation of query columns."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import float32
from pygpukit_amd.ops._common import call, check_out, validate_float


def latent_rows(x: GPUArray, norm: GPUArray, freq: GPUArray, first: int, *, eps: float = 1e-5, out: GPUArray | None = None) -> GPUArray:
    """x [n, rank + rot] -> [rms norm of the first rank columns * norm | the last rot columns turned by their position]: row i is position
    first + i, columns (2j, 2j + 1) turn by position * freq[j].  norm float32 [rank], freq float32 [rot / 2]."""
    validate_float(x, "latent_rows")
    rank, rot = norm.size, 2 * freq.size
    if x.ndim != 2 or x.shape[1] != rank + rot or norm.dtype != float32 or freq.dtype != float32:
        raise ValueError(f"latent_rows: rows {x.shape}, norm of {rank}, {rot} turned columns")
    o = check_out(out, x.shape, x.dtype, "latent_rows")
    call("pgk_latent_rows", x._p, norm._p, freq._p, o._p, x.shape[0], rank, rot, int(first), float(eps), x.dtype.code, None)
    return o


def rotate_pairs(x: GPUArray, freq: GPUArray, first: int) -> GPUArray:
    """The last 2 * len(freq) columns of x [n, heads, dim], turned in place as in latent_rows."""
    validate_float(x, "rotate_pairs")
    if x.ndim != 3 or freq.dtype != float32 or 2 * freq.size > x.shape[2]:
        raise ValueError(f"rotate_pairs: x {x.shape}, {freq.size} pairs")
    call("pgk_rotate_pairs", x._p, freq._p, x.shape[0], x.shape[1], x.shape[2], 2 * freq.size, int(first), x.dtype.code, None)
    return x


__all__ = ["latent_rows", "rotate_pairs"]
