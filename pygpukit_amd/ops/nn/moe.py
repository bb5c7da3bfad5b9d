"""Mixture of experts."""

from __future__ import annotations

from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32, int32
from pygpukit_amd.ops._common import call, check_out
from pygpukit_amd.ops.tensor import pad_2d


def mixture_of_experts(x: GPUArray, router: GPUArray, correction: GPUArray, gate_up: GPUArray, down: GPUArray, *, top: int, groups: int = 0, keep: int = 0,
                       scale: float = 1.0, out: GPUArray | None = None) -> GPUArray:
    """x [n, hidden], router [experts, hidden], correction float32 [experts], gate_up [experts, 2 ff, hidden], down [experts, hidden, ff]
    -> float32 [n, hidden].  s = sigmoid(x router^T); the `top` largest s + correction are chosen (groups > 0: among the experts of the
    `keep` groups of neighbours with the largest sum of their two largest), weights scale * s / (sum of the chosen s)."""
    if x.dtype not in (float32, bfloat16) or any(a.dtype != x.dtype for a in (router, gate_up, down)) or correction.dtype != float32:
        raise ValueError("mixture_of_experts: float32 or bfloat16 of one dtype, correction float32")
    n, hidden = x.shape
    E, two_ff, _ = gate_up.shape
    ff = two_ff // 2
    if router.shape != (E, hidden) or correction.shape != (E,) or gate_up.shape != (E, 2 * ff, hidden) or down.shape != (E, hidden, ff):
        raise ValueError(f"mixture_of_experts: x {x.shape}, router {router.shape}, gate_up {gate_up.shape}, down {down.shape}")
    wp, fp, ep = (-(-v // 64) * 64 for v in (hidden, ff, E))
    if (wp, fp) != (hidden, ff):
        x = pad_2d(x, n, wp)
        gate_up = pad_2d(pad_2d(gate_up.view((2 * E, ff * hidden)), 2 * E, fp * hidden).view((2 * E * fp, hidden)), 2 * E * fp, wp)
        down = pad_2d(pad_2d(down.view((E, hidden * ff)), E, wp * ff).view((E * wp, ff)), E * wp, fp)
    o = check_out(out, (n, hidden), float32, "mixture_of_experts")
    full = o if wp == hidden else GPUArray((n, wp), float32)
    call("pgk_moe", x._p, pad_2d(router, ep, wp)._p, correction._p, gate_up._p, down._p, full._p, n, wp, fp, E, int(top), int(groups), int(keep), float(scale), x.dtype.code, None)
    if full is not o:
        call("pgk_pad_2d", full.view((n * wp,))._p, o._p, n, wp, n, hidden, float32.code, None)
    return o


def table_experts(x: GPUArray, tokens: GPUArray, table: GPUArray, up: GPUArray, down: GPUArray, *, out: GPUArray | None = None) -> GPUArray:
    """x [n, hidden], tokens int32 [n], table int32 [vocab, top], up [experts, ff, hidden], down [experts, hidden, ff] -> float32 [n, hidden]:
    the mean over the experts that the token's row of the table names (entries below `experts`) of down gelu(up x), exact gelu."""
    if x.dtype not in (float32, bfloat16) or up.dtype != x.dtype or down.dtype != x.dtype or table.dtype != int32 or tokens.dtype != int32:
        raise ValueError("table_experts: float32 or bfloat16 of one dtype, table and tokens int32")
    n, hidden = x.shape
    E, ff, _ = up.shape
    if table.ndim != 2 or tokens.shape != (n,) or up.shape != (E, ff, hidden) or down.shape != (E, hidden, ff):
        raise ValueError(f"table_experts: x {x.shape}, tokens {tokens.shape}, table {table.shape}, up {up.shape}, down {down.shape}")
    wp, fp = (-(-v // 64) * 64 for v in (hidden, ff))
    if (wp, fp) != (hidden, ff):
        x = pad_2d(x, n, wp)
        up = pad_2d(pad_2d(up.view((E, ff * hidden)), E, fp * hidden).view((E * fp, hidden)), E * fp, wp)
        down = pad_2d(pad_2d(down.view((E, hidden * ff)), E, wp * ff).view((E * wp, ff)), E * wp, fp)
    o = check_out(out, (n, hidden), float32, "table_experts")
    full = o if wp == hidden else GPUArray((n, wp), float32)
    call("pgk_table_moe", x._p, table._p, tokens._p, up._p, down._p, full._p, n, wp, fp, E, table.shape[1], x.dtype.code, None)
    if full is not o:
        call("pgk_pad_2d", full._p, o._p, n, wp, n, hidden, float32.code, None)
    return o


__all__ = ["mixture_of_experts", "table_experts"]
