"""Plain NumPy restatement of the Fetezen decoder, one function per mechanism (float64 by default, no caches, no batching).

    s streams x_1 .. x_s, each the embedding row at the start; a sublayer F (a mixer, then a feed-forward) with its numbers c, d, M:
        u = sum_a c_a x_a,   y = F(n(u)),   x_b <- sum_a M[a, b] x_a + d_b y   (all b from the old streams)
    n(u)          = each of `groups` equal parts of u over its own root mean square, times w
    attention:    q, k, v = W h + b per head, q and k over their root mean square times a weight, their first `dims` columns turned
                  (column i with column i + dims/2); raw_h(i, j) = scale q_h(i) . k(j);  score_h = sum_g T[h, g] raw_g
                  over the keys j <= i of i's chunk of positions; softmax with exp(sink_h) added to the denominator
                  (a layer may use an earlier one's k and v)
    dense:        W_d p(W_u h),   p(z) = a r(z) + b r(z^2) + c r(z^3) + e,   r(z) = z over its root mean square
    experts:      the token's row of a table names `top` of them, each W_d gelu(W_u h) / top;
                  plus a shared one times sigmoid(w . h)
    logits        = cap * tanh(head . n(sum of the streams) / cap)

Shares no code with pygpukit_amd: it is what the HIP kernels are compared with."""

from __future__ import annotations

import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def gelu(z: np.ndarray) -> np.ndarray:
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)).astype(z.dtype))


def rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def group_norm(x: np.ndarray, w: np.ndarray, groups: int, eps: float) -> np.ndarray:
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape) * w


def poly_norm(z: np.ndarray, act: np.ndarray, eps: float) -> np.ndarray:
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z * z, eps) + c * rms(z * z * z, eps) + e


def rotate_half(x: np.ndarray, positions: np.ndarray, base: float, dims: int) -> np.ndarray:
    """x [n, heads, d]: columns i and i + dims / 2 turned by position * base^(-2i / dims); columns from dims on stay."""
    half = dims // 2
    a = positions[:, None, None] * base ** (-2.0 * np.arange(half) / dims)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., dims:]], axis=-1)


def chunk_mask(n: int, size: int | None) -> np.ndarray:
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    m = j <= i
    return m if size is None else m & (i // size == j // size)


def sink_softmax(s: np.ndarray, sink: np.ndarray, mask: np.ndarray) -> np.ndarray:
    """s [heads, n, n], sink [heads]: the weights of the keys; the sink takes its share and has no value."""
    s = np.where(mask, s, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - top))


def keys_values(h: np.ndarray, w: dict, m: dict, eps: float) -> tuple[np.ndarray, np.ndarray]:
    n, G = h.shape[0], m["kv_heads"]
    k = rms((h @ w["k"].T + w["k.b"]).reshape(n, G, m["dim"]), eps) * w["k.norm"]
    return rotate_half(k, np.arange(n), m["rot"]["base"], m["rot"]["dims"]), (h @ w["v"].T + w["v.b"]).reshape(n, G, m["vdim"])


def talking_attention(q: np.ndarray, k: np.ndarray, v: np.ndarray, talk: np.ndarray, sink: np.ndarray, scale: float, mask: np.ndarray) -> np.ndarray:
    """q [n, H, d], k [n, G, d], v [n, G, vd] -> [n, H, vd]"""
    rep = q.shape[1] // k.shape[1]
    raw = np.matmul(q.transpose(1, 0, 2), np.repeat(k, rep, axis=1).transpose(1, 2, 0)) * scale
    s = np.tensordot(talk, raw, axes=1)
    return np.matmul(sink_softmax(s, sink, mask), np.repeat(v, rep, axis=1).transpose(1, 0, 2)).transpose(1, 0, 2)


def attention(h: np.ndarray, w: dict, m: dict, eps: float, kv: tuple[np.ndarray, np.ndarray]) -> np.ndarray:
    n, H = h.shape[0], m["heads"]
    q = rms((h @ w["q"].T + w["q.b"]).reshape(n, H, m["dim"]), eps) * w["q.norm"]
    q = rotate_half(q, np.arange(n), m["rot"]["base"], m["rot"]["dims"])
    y = talking_attention(q, *kv, w["talk"], w["sink"], m["scale"], chunk_mask(n, (m.get("mask") or {}).get("size")))
    return y.reshape(n, -1) @ w["o"].T + w["o.b"]


def dense(h: np.ndarray, w: dict, eps: float) -> np.ndarray:
    return poly_norm(h @ w["up"].T, w["act"], eps) @ w["down"].T


def table_experts(h: np.ndarray, tokens: np.ndarray, w: dict, top: int) -> np.ndarray:
    out = np.zeros((h.shape[0], h.shape[1]), h.dtype)
    chosen = np.asarray(w["table"])[tokens]
    for e in np.unique(chosen):
        rows = np.nonzero((chosen == e).any(axis=1))[0]
        out[rows] += gelu(h[rows] @ w[f"e{e}.up"].T) @ w[f"e{e}.down"].T / top
    return out


def shared_expert(h: np.ndarray, w: dict) -> np.ndarray:
    return sigmoid(h @ w["shared.sg"].T) * (gelu(h @ w["shared.up"].T) @ w["shared.down"].T)


def feed_forward(h: np.ndarray, tokens: np.ndarray, w: dict, mlp: dict, eps: float) -> np.ndarray:
    if mlp["kind"] == "dense":
        return dense(h, w, eps)
    y = table_experts(h, tokens, w, mlp["router"]["top"])
    return y + shared_expert(h, w) if mlp.get("shared") else y


def hyper_in(x: np.ndarray, w: dict, q: int) -> np.ndarray:
    """x [streams, n, width] -> what sublayer q reads."""
    return np.tensordot(w[f"hc{q}.in"], x, axes=1)


def hyper_out(x: np.ndarray, y: np.ndarray, w: dict, q: int) -> np.ndarray:
    return np.tensordot(w[f"hc{q}.mix"].T, x, axes=1) + w[f"hc{q}.out"][:, None, None] * y


def under(W: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}


def layers(tokens, cfg: dict, W: dict, dtype=np.float64):
    """Yields the sum of the streams after every layer."""
    W = {k: (np.asarray(v) if k.endswith(".table") else np.asarray(v, dtype)) for k, v in W.items()}
    t, groups, eps = np.asarray(tokens), cfg["norm"]["groups"], cfg["norm"]["eps"]
    x = np.repeat(W["embed"][t][None], cfg["streams"], axis=0)
    kept: list = []
    for i, l in enumerate(cfg["layers"]):
        w, m = under(W, f"l{i}."), l["mixer"]
        mix = under(w, "mix.")
        h = group_norm(hyper_in(x, w, 1), w["norm1"], groups, eps)
        kept.append(kept[m["kv_from"]] if m.get("kv_from") is not None else keys_values(h, mix, m, eps))
        x = hyper_out(x, attention(h, mix, m, eps, kept[i]), w, 1)
        if l["mlp"]:
            h = group_norm(hyper_in(x, w, 2), w["norm2"], groups, eps)
            x = hyper_out(x, feed_forward(h, t, under(w, "mlp."), l["mlp"], eps), w, 2)
        yield x.sum(axis=0)


def forward(tokens, cfg: dict, W: dict, dtype=np.float64) -> np.ndarray:
    """fp logits [n, vocab]"""
    for x in layers(tokens, cfg, W, dtype):
        pass
    h = group_norm(x, np.asarray(W["final.norm"], dtype), cfg["norm"]["groups"], cfg["norm"]["eps"])
    z = h @ np.asarray(W["head"], dtype).T
    cap = cfg.get("logit_softcap")
    return z if cap is None else cap * np.tanh(z / cap)
