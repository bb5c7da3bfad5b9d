"""Causal scaled-dot-product attention (reference: src/pygpukit/ops/nn/attention.py:16-235 ->
ops.cuh:287-300).  K/V may carry fewer heads than Q (un-expanded GQA): kv head = q head // (Hq/Hkv)."""

from __future__ import annotations

import ctypes as C

from pygpukit_amd import _hip
from pygpukit_amd.core.array import GPUArray
from pygpukit_amd.core.dtypes import bfloat16, float32, int32
from pygpukit_amd.ops._common import call, check_out, validate_float

_ws_cache: dict[tuple[int, int, int], GPUArray] = {}


def _check_qkv(Q: GPUArray, K: GPUArray, V: GPUArray, name: str):
    validate_float(Q, name)
    if Q.ndim != 3 or K.ndim != 3 or V.ndim != 3:
        raise ValueError(f"{name} expects 3D inputs [n_heads, seq_len, head_dim]")
    if Q.dtype != K.dtype or Q.dtype != V.dtype:
        raise ValueError(f"{name}: Q, K, V must have same dtype")
    hq, q_len, d = Q.shape
    if K.shape[0] != V.shape[0] or hq % K.shape[0] != 0:
        raise ValueError(f"{name}: n_heads mismatch")
    if K.shape[2] != d or V.shape[2] != d:
        raise ValueError(f"{name}: head_dim mismatch")
    if K.shape[1] != V.shape[1]:
        raise ValueError(f"{name}: K and V seq_len mismatch")
    return hq, K.shape[0], q_len, K.shape[1], d


def sdpa_causal(Q: GPUArray, K: GPUArray, V: GPUArray, scale: float = 0.0, *, out: GPUArray | None = None) -> GPUArray:
    """softmax(Q K^T * scale + causal mask) V; scale <= 0 -> 1/sqrt(head_dim); the mask lets query i see
    kv positions <= (kv_len - q_len) + i."""
    hq, hkv, q_len, kv_len, d = _check_qkv(Q, K, V, "sdpa_causal")
    o = check_out(out, (hq, q_len, d), Q.dtype, "sdpa_causal")
    call("pgk_sdpa_causal", Q._p, K._p, V._p, o._p, hq, hkv, q_len, kv_len, d, float(scale), q_len * d, d, kv_len * d, d,
         q_len * d, d, Q.dtype.code, None)
    return o


def sdpa_causal_strided(q: GPUArray, k: GPUArray, v: GPUArray, out: GPUArray, hq: int, hkv: int, q_len: int, kv_len: int,
                        d: int, q_strides, kv_strides, o_strides, scale: float = 0.0) -> None:
    """Same op on [S,H,D]-layout (or any head/row-strided) buffers: strides are (head, row) in elements."""
    call("pgk_sdpa_causal", q._p, k._p, v._p, out._p, hq, hkv, q_len, kv_len, d, float(scale), q_strides[0], q_strides[1],
         kv_strides[0], kv_strides[1], o_strides[0], o_strides[1], q.dtype.code, None)


def _workspace(hq: int, d: int, max_seq: int) -> GPUArray:
    key = (hq, d, max_seq)
    ws = _ws_cache.get(key)
    if ws is None:
        nbytes = _hip.load().pgk_sdpa_decode_workspace_bytes(hq, d, max_seq)
        ws = GPUArray(((nbytes + 3) // 4,), float32)
        _ws_cache[key] = ws
    return ws


def sdpa_causal_fixed_cache(Q: GPUArray, K: GPUArray, V: GPUArray, out: GPUArray, context_len: int, scale: float = 0.0) -> None:
    """Attention of Q [Hq,q_len,D] over the first context_len rows of the fixed caches K,V [Hc,max_seq,D]."""
    hq, hc, q_len, max_seq, d = _check_qkv(Q, K, V, "sdpa_causal_fixed_cache")
    if out.shape != (hq, q_len, d) or out.dtype != Q.dtype:
        raise ValueError("sdpa_causal_fixed_cache: output shape/dtype mismatch")
    if context_len <= 0 or context_len > max_seq:
        raise ValueError(f"sdpa_causal_fixed_cache: invalid context_len {context_len}")
    ws = _workspace(hq, d, max_seq) if q_len == 1 else None
    call("pgk_sdpa_fixed_cache", Q._p, K._p, V._p, out._p, hq, hc, q_len, max_seq, d, float(scale), context_len, None,
         ws._p if ws is not None else None, Q.dtype.code, None)


def sdpa_causal_fixed_cache_ptr(Q: GPUArray, K: GPUArray, V: GPUArray, out: GPUArray, context_len_buf: GPUArray,
                                max_kv_len: int, scale: float = 0.0) -> None:
    """As above with context_len read from a device int32 (graph replay)."""
    hq, hc, q_len, max_seq, d = _check_qkv(Q, K, V, "sdpa_causal_fixed_cache_ptr")
    if context_len_buf.dtype != int32:
        raise ValueError("sdpa_causal_fixed_cache_ptr: context_len_buf must be int32")
    if q_len != 1:
        raise ValueError("sdpa_causal_fixed_cache_ptr: q_len must be 1")
    ws = _workspace(hq, d, max_seq)
    call("pgk_sdpa_fixed_cache", Q._p, K._p, V._p, out._p, hq, hc, q_len, max_seq, d, float(scale), 0, context_len_buf._p,
         ws._p, Q.dtype.code, None)


def window_attention(q: GPUArray, k: GPUArray, v: GPUArray, scale: float, window: int, *, gate: GPUArray | None = None,
                     slopes: GPUArray | None = None, out: GPUArray | None = None) -> GPUArray:
    """q [q_len, Hq, dk], k [kv_len, Hkv, dk], v [kv_len, Hkv, dv] -> [q_len, Hq, dv]: query i is position kv_len - q_len + i and sees the
    `window` positions that end with its own.  gate [q_len, Hq] or [q_len, Hq, dv]: head outputs (or their elements) are multiplied by
    its sigmoid.  slopes float32 [Hq]: slope * distance is taken off the scaled score."""
    validate_float(q, "window_attention")
    if q.ndim != 3 or k.ndim != 3 or v.ndim != 3 or k.dtype != q.dtype or v.dtype != q.dtype:
        raise ValueError("window_attention expects q, k, v as [seq, heads, width] of one dtype")
    (q_len, hq, dk), (kv_len, hkv, dk2), (kv2, hkv2, dv) = q.shape, k.shape, v.shape
    if dk != dk2 or kv_len != kv2 or hkv != hkv2 or hq % hkv or kv_len < q_len:
        raise ValueError(f"window_attention: shapes {q.shape}, {k.shape}, {v.shape} do not match")
    if window < 1:
        raise ValueError(f"window_attention: window {window}")
    if gate is not None and (gate.shape not in ((q_len, hq), (q_len, hq, dv)) or gate.dtype != q.dtype):
        raise ValueError("window_attention: gate must be [q_len, Hq] or [q_len, Hq, dv] in q's dtype")
    if slopes is not None and (slopes.shape != (hq,) or slopes.dtype != float32):
        raise ValueError("window_attention: slopes must be float32 [Hq]")
    each = gate is not None and gate.ndim == 3
    o = check_out(out, (q_len, hq, dv), q.dtype, "window_attention")
    call("pgk_window_attention", q._p, k._p, v._p, o._p, hq, hkv, q_len, kv_len, dk, dv, float(scale), min(int(window), 2**30),
         gate._p if gate is not None else None, hq * dv if each else hq, int(each), slopes._p if slopes is not None else None, q.dtype.code, None)
    return o


def head_norm_rope(x: GPUArray, norm: GPUArray | None, freq: GPUArray | None, first: int, eps: float = 1e-5) -> GPUArray:
    """x [n, heads, dim], row i at position first + i: RMS norm over every head (norm float32 [dim] or None), then columns i and
    i + rot / 2 turned by position * freq[i] (freq float32 [rot / 2]); columns from rot on pass."""
    validate_float(x, "head_norm_rope")
    rot = 0 if freq is None else 2 * freq.size
    if x.ndim != 3 or rot > x.shape[2] or first < 0 or (norm is not None and (norm.shape != (x.shape[2],) or norm.dtype != float32)) or (freq is not None and freq.dtype != float32):
        raise ValueError(f"head_norm_rope: x {x.shape}, {rot} turned columns")
    o = GPUArray(x.shape, x.dtype)
    call("pgk_head_norm_rope", x._p, norm._p if norm is not None else None, freq._p if freq is not None else None, o._p, *x.shape, rot, first, float(eps), x.dtype.code, None)
    return o


def talk_attention(q: GPUArray, k: GPUArray, v: GPUArray, scale: float, window: int, *, chunked: bool = False, first: int = 0, talk: GPUArray | None = None,
                   sink: GPUArray | None = None, out: GPUArray | None = None) -> GPUArray:
    """q [q_len, Hq, dk], k [kv_len, Hkv, dk], v [kv_len, Hkv, dv] -> [q_len, Hq, dv]: row t of k is position first + t, the queries are the
    last q_len positions.  A query sees the `window` positions that end with its own, or (chunked) those of its own chunk of
    `window` positions, counted from position 0.  talk float32 [Hq, Hq] mixes the heads' scaled scores; exp(sink), float32 [Hq],
    stands in the softmax's denominator."""
    if q.ndim != 3 or k.ndim != 3 or v.ndim != 3 or q.dtype not in (float32, bfloat16) or k.dtype != q.dtype or v.dtype != q.dtype:
        raise ValueError("talk_attention expects q, k, v as [seq, heads, width], float32 or bfloat16")
    (q_len, hq, dk), (kv_len, hkv, dk2), (kv2, hkv2, dv) = q.shape, k.shape, v.shape
    if dk != dk2 or kv_len != kv2 or hkv != hkv2 or hq % hkv or kv_len < q_len or window < 1 or first < 0:
        raise ValueError(f"talk_attention: shapes {q.shape}, {k.shape}, {v.shape}, window {window}, first position {first}")
    for a, shape in ((talk, (hq, hq)), (sink, (hq,))):
        if a is not None and (a.shape != shape or a.dtype != float32):
            raise ValueError(f"talk_attention: talk and sink are float32 [Hq, Hq] and [Hq], got {a.shape}")
    o = check_out(out, (q_len, hq, dv), q.dtype, "talk_attention")
    call("pgk_talk_attention", q._p, k._p, v._p, talk._p if talk is not None else None, sink._p if sink is not None else None, o._p, hq, hkv, q_len, kv_len, int(first), dk, dv,
         float(scale), min(int(window), 2**30), int(chunked), q.dtype.code, None)
    return o


def head_gate(x: GPUArray, gate: GPUArray) -> GPUArray:
    """x [rows, heads, d] *= sigmoid(gate [rows, heads]) in place."""
    validate_float(x, "head_gate")
    if x.ndim != 3 or gate.shape != x.shape[:2] or gate.dtype != x.dtype:
        raise ValueError(f"head_gate: x {x.shape} and gate {gate.shape} do not match")
    call("pgk_head_gate", x._p, gate._p, x.shape[0], x.shape[1], x.shape[2], x.shape[1], x.dtype.code, None)
    return x


def sigmoid_mul(x: GPUArray, gate: GPUArray) -> GPUArray:
    """x *= sigmoid(gate), element by element, in place."""
    validate_float(x, "sigmoid_mul")
    if gate.shape != x.shape or gate.dtype != x.dtype:
        raise ValueError(f"sigmoid_mul: x {x.shape} and gate {gate.shape} do not match")
    call("pgk_sigmoid_mul", x._p, gate._p, x.size, x.dtype.code, None)
    return x
