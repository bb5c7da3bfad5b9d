"""Plain NumPy restatement of the Malasun decoder, one function per mechanism (float64 by default, no caches, no batching).

    x_0[p]      = E[token_p]
    per layer:    x <- x + g1 * mixer(x) / rms(mixer(x))          rms(y) = sqrt(mean(y^2) + eps), g1 a single number
                  x <- x + g2 * ff(x) / rms(ff(x))                (absent when the layer has no feed-forward)
    ff(x):        D act(U x),  act = xIELU with two numbers
    attention:    q | k | v = causal taps over time of (W x + b);  q and k divided by the rms of the whole row, times a weight;
                  s_a(i, j) = scale * q_a(i) . k(j) - 2^(-8 (a + 1) / H) (i - j)  for 0 <= i - j < window;
                  O (sigmoid(G x) * [softmax(s_a) v]);  a layer may take the keys and values of another one
    hgrn2:        q = silu(Q x),  v = V x,  f = l + (1 - l) sigmoid(F x + b);  S <- diag(f) S + (1 - f) v^T,  o = S^T q;
                  O [o_a / rms(o_a) * w]
    logits      = head . (g x / rms(x))

Shares no code with pygpukit_amd: it is what the HIP kernels are compared with."""

from __future__ import annotations

import numpy as np

from oracle.totolorn_ref import group, masked_softmax, rms_scale, sigmoid, window_mask


def scalar_norm(x: np.ndarray, g: np.ndarray, eps: float) -> np.ndarray:
    return rms_scale(x, eps) * np.reshape(g, ())


def softplus(z: float) -> float:
    return float(np.logaddexp(0.0, z))


def xielu(z: np.ndarray, p: float, q: float) -> np.ndarray:
    neg = np.minimum(z, 0.0)
    return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(neg) - neg)) + 0.5 * z


def short_conv(u: np.ndarray, w: np.ndarray) -> np.ndarray:
    """u [n, channels], w [channels, taps]: the last tap multiplies the row itself."""
    taps = w.shape[1]
    out = np.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j
        if back < u.shape[0]:
            out[back:] += w[:, j] * u[:u.shape[0] - back]
    return out


def distance_slopes(heads: int) -> np.ndarray:
    return 2.0 ** (-8.0 * np.arange(1, heads + 1) / heads)


def attend(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, window: int | None, slopes: np.ndarray) -> np.ndarray:
    """q [n, H, dim], k [n, G, dim], v [n, G, vdim] -> [n, H, vdim]."""
    n, H, _ = q.shape
    rep, vis = H // k.shape[1], window_mask(n, window)
    dist = np.arange(n)[:, None] - np.arange(n)[None, :]
    out = np.empty((n, H, v.shape[2]), v.dtype)
    for a in range(H):
        out[:, a] = masked_softmax(scale * (q[:, a] @ k[:, a // rep].T) - slopes[a] * dist, vis) @ v[:, a // rep]
    return out


def projected(h: np.ndarray, w: dict, name: str) -> np.ndarray:
    u = h @ w[name].T + w[name + ".b"]
    return short_conv(u, w[name + ".conv"]) if name + ".conv" in w else u


def keys_values(h: np.ndarray, w: dict, m: dict, eps: float) -> tuple[np.ndarray, np.ndarray]:
    n, G = h.shape[0], m["kv_heads"]
    k = rms_scale(projected(h, w, "k"), eps) * w["k.norm"]
    return k.reshape(n, G, m["dim"]), projected(h, w, "v").reshape(n, G, m["vdim"])


def attention(h: np.ndarray, w: dict, m: dict, eps: float, kv: tuple[np.ndarray, np.ndarray]) -> np.ndarray:
    n, H = h.shape[0], m["heads"]
    q = (rms_scale(projected(h, w, "q"), eps) * w["q.norm"]).reshape(n, H, m["dim"])
    window = m["mask"]["size"] if m.get("mask") else None
    y = attend(q, *kv, m["scale"], window, distance_slopes(H)).reshape(n, H * m["vdim"])
    return (y * sigmoid(h @ w["g"].T)) @ w["o"].T


def gated_recurrence(q: np.ndarray, f: np.ndarray, v: np.ndarray, state: np.ndarray | None = None) -> tuple[np.ndarray, np.ndarray]:
    """q, f [n, heads, dim], v [n, heads, vdim] -> o [n, heads, vdim] and the state [heads, dim, vdim] after the last row."""
    n, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), v.dtype) if state is None else state.copy()
    o = np.empty(v.shape, v.dtype)
    for t in range(n):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def forget_gate(z: np.ndarray, b: np.ndarray, lower: np.ndarray) -> np.ndarray:
    return lower + (1.0 - lower) * sigmoid(z + b)


def hgrn2(h: np.ndarray, w: dict, m: dict, eps: float) -> np.ndarray:
    n, H, d, vd = h.shape[0], m["heads"], m["dim"], m["vdim"]
    z = h @ w["q"].T
    f = forget_gate(h @ w["f"].T, w["f.b"], w["lower"])
    o, _ = gated_recurrence((z * sigmoid(z)).reshape(n, H, d), f.reshape(n, H, d), (h @ w["v"].T).reshape(n, H, vd))
    return (rms_scale(o, eps) * w["norm"]).reshape(n, H * vd) @ w["o"].T


def feed_forward(h: np.ndarray, w: dict) -> np.ndarray:
    return xielu(h @ w["up"].T, *w["act"]) @ w["down"].T


def layer(x: np.ndarray, i: int, cfg: dict, W: dict, kv: dict) -> np.ndarray:
    eps, spec = cfg["norm"]["eps"], cfg["layers"][i]
    w, m = group(W, f"l{i}.mix."), spec["mixer"]
    if spec["type"] == "hgrn2":
        y = hgrn2(x, w, m, eps)
    else:
        kv[i] = keys_values(x, w, m, eps) if m.get("kv_from") is None else kv[m["kv_from"]]
        y = attention(x, w, m, eps, kv[i])
    x = x + scalar_norm(y, W[f"l{i}.norm1"], eps)
    if spec["mlp"] is not None:
        x = x + scalar_norm(feed_forward(x, group(W, f"l{i}.mlp.")), W[f"l{i}.norm2"], eps)
    return x


def forward(tokens, cfg: dict, W: dict, dtype=np.float64, want_layers: bool = False):
    """logits [n, vocab] (and the residual stream after every layer)."""
    W = {k: v.astype(dtype) for k, v in W.items()}
    x, kv, states = W["embed"][np.asarray(tokens)], {}, []
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, W, kv)
        states.append(x)
    logits = scalar_norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T
    return (logits, states) if want_layers else logits


def greedy(prompt, n_new: int, cfg: dict, W: dict) -> list[int]:
    out = [int(t) for t in prompt]
    for _ in range(n_new):
        out.append(int(np.argmax(forward(out, cfg, W)[-1])))
    return out
