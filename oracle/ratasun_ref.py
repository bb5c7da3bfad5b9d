"""Plain NumPy restatement of the Ratasun decoder, one function per mechanism (float64 by default, no caches, no batching).

    x_0[p]      = E[token_p]
    layers run in order; layers start .. stop-1 run `times` times over, and before pass t of them  x <- L [x; x_0] + s_t
    per layer:    h = ln(x) * w,   x <- x + mixer(h) + moe(h)      (moe absent when the layer has none)
    latent:       c = rms(D_c h) * w_c,  r = rot(D_r h) shared by all heads,  q_a = [n_a | rot(p_a)];
                  score = scale * (n_a . U_a c + p_a . r) over all earlier positions and its own,  v_a = V_a c
    delta:        q, k, v = silu(taps over time), q and k of unit length per head (q also times dim^-1/2), b = sigmoid(B h),
                  g = exp(-exp(A) softplus(W_2 W_1 h + d)) per key channel;
                  S <- diag(g) S,  u = b (v - S^T k),  S <- S + k u^T,  o = S^T q;   O [rms(o_a) * w * sigmoid(G_2 G_1 h)]
    ssd:          x, B, C = silu(taps over time + bias),  t = softplus(t + d);
                  S <- exp(-exp(A) t) S + t B x^T,  y = S^T C + D x;   O [rms in parts(y * silu(z)) * w]
    moe:          s = sigmoid(R h); the best groups by their two largest s + c, in them the `top` largest s + c;
                  sum of the chosen experts' SwiGLU weighted by scale * s / sum s
    logits      = logit_scale * head . (ln(x) * w)

Shares no code with pygpukit_amd: it is what the HIP kernels are compared with."""

from __future__ import annotations

import numpy as np


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z: np.ndarray) -> np.ndarray:
    return z * sigmoid(z)


def softplus(z: np.ndarray) -> np.ndarray:
    return np.logaddexp(0.0, z)


def layer_norm(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def rms(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rotate(x: np.ndarray, positions: np.ndarray, base: float) -> np.ndarray:
    """x [n, ..., d]: neighbours (2i, 2i + 1) turned by position * base^(-2i / d)."""
    d = x.shape[-1]
    a = positions[:, None] * base ** (-2.0 * np.arange(d // 2) / d)
    c, s = np.cos(a), np.sin(a)
    while c.ndim < x.ndim:
        c, s = c[:, None], s[:, None]
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2], out[..., 1::2] = u * c - v * s, v * c + u * s
    return out


def causal_softmax(s: np.ndarray) -> np.ndarray:
    n = s.shape[0]
    s = np.where(np.arange(n)[:, None] >= np.arange(n)[None, :], s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_attention(h: np.ndarray, w: dict, m: dict, eps: float) -> np.ndarray:
    n, H, d, r, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    p, base = np.arange(n), m["rot"]["base"]
    q = (h @ w["q"].T).reshape(n, H, d + r)
    down = h @ w["dkv"].T
    c, kr = rms(down[:, :R], eps) * w["dkv.norm"], rotate(down[:, R:], p, base)
    k, v, qr = (c @ w["uk"].T).reshape(n, H, d), (c @ w["uv"].T).reshape(n, H, m["vdim"]), rotate(q[:, :, d:], p, base)
    out = np.empty((n, H, m["vdim"]), h.dtype)
    for a in range(H):
        out[:, a] = causal_softmax((q[:, a, :d] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]) @ v[:, a]
    return out.reshape(n, -1) @ w["o"].T


def short_conv(u: np.ndarray, w: np.ndarray, bias: np.ndarray | None = None) -> np.ndarray:
    """u [n, channels], w [channels, taps]: the last tap multiplies the row itself."""
    taps = w.shape[1]
    out = np.zeros_like(u) if bias is None else np.tile(bias, (u.shape[0], 1))
    for j in range(taps):
        back = taps - 1 - j
        out[back:] += w[:, j] * u[:u.shape[0] - back] if back < u.shape[0] else 0.0
    return out


def unit(x: np.ndarray) -> np.ndarray:
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(q: np.ndarray, k: np.ndarray, v: np.ndarray, g: np.ndarray, beta: np.ndarray, state: np.ndarray | None = None) -> tuple[np.ndarray, np.ndarray]:
    """q, k, g [n, heads, dim], v [n, heads, vdim], beta [n, heads] -> o [n, heads, vdim] and the state [heads, dim, vdim]."""
    n, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), v.dtype) if state is None else state.copy()
    o = np.empty(v.shape, v.dtype)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def channel_delta(h: np.ndarray, w: dict, m: dict, eps: float) -> np.ndarray:
    n, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[x].T, w[x + ".conv"])) for x in "qkv")
    q, k = (np.repeat(unit(x.reshape(n, G, d)), H // G, axis=1) for x in (q, k))
    z = (h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]
    g = np.exp(-np.exp(w["A_log"])[:, None] * softplus(z).reshape(n, H, d))
    o, _ = delta_rule(q * d ** -0.5, k, v.reshape(n, H, vd), g, sigmoid(h @ w["b"].T))
    o = rms(o, eps) * w["norm"] * sigmoid((h @ w["g1"].T) @ w["g2"].T).reshape(n, H, vd)
    return o.reshape(n, -1) @ w["o"].T


def state_space(x: np.ndarray, B: np.ndarray, C: np.ndarray, dt: np.ndarray, a: np.ndarray, D: np.ndarray,
                state: np.ndarray | None = None) -> tuple[np.ndarray, np.ndarray]:
    """x [n, heads, vdim], B, C [n, heads, N], dt [n, heads], a, D [heads] -> y [n, heads, vdim] and the state [heads, N, vdim]."""
    n, H, vd = x.shape
    S = np.zeros((H, B.shape[2], vd), x.dtype) if state is None else state.copy()
    y = np.empty_like(x)
    for t in range(n):
        S = np.exp(-a * dt[t])[:, None, None] * S + (dt[t][:, None] * B[t])[:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hnv,hn->hv", S, C[t]) + D[:, None] * x[t]
    return y, S


def parts_norm(x: np.ndarray, parts: int, eps: float) -> np.ndarray:
    return rms(x.reshape(x.shape[0], parts, -1), eps).reshape(x.shape)


def mamba2(h: np.ndarray, w: dict, m: dict, eps: float) -> np.ndarray:
    n, H, vd, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * vd
    z, u, dt = np.split(h @ w["in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    x, B, C = np.split(silu(short_conv(u, w["conv"], w["conv.b"])), [inner, inner + G * N], axis=1)
    B, C = (np.repeat(y.reshape(n, G, N), H // G, axis=1) for y in (B, C))
    y, _ = state_space(x.reshape(n, H, vd), B, C, softplus(dt + w["dt_bias"]), np.exp(w["A_log"]), w["D"])
    return (parts_norm(y.reshape(n, inner) * silu(z), m["norm_groups"], eps) * w["norm"]) @ w["o"].T


def choose(s: np.ndarray, correction: np.ndarray, r: dict) -> tuple[np.ndarray, np.ndarray]:
    """scores [n, experts] -> the chosen experts [n, top] and their weights."""
    n, E = s.shape
    c = s + correction
    if r.get("groups"):
        cnt, keep = r["groups"]["count"], r["groups"]["keep"]
        best = np.sort(c.reshape(n, cnt, E // cnt), axis=2)[:, :, -2:].sum(axis=2)
        rank = np.argsort(-best, axis=1, kind="stable")
        out = np.ones((n, cnt), bool)
        np.put_along_axis(out, rank[:, :keep], False, axis=1)
        c = np.where(np.repeat(out, E // cnt, axis=1), -np.inf, c)
    e = np.argsort(-c, axis=1, kind="stable")[:, :r["top"]]
    p = np.take_along_axis(s, e, axis=1)
    return e, p / (p.sum(axis=1, keepdims=True) + 1e-20) * r["scale"]


def moe(h: np.ndarray, w: dict, m: dict) -> np.ndarray:
    e, p = choose(sigmoid(h @ w["router"].T), w["correction"], m["router"])
    y = np.zeros((h.shape[0], w["e0.down"].shape[0]), h.dtype)
    for i in range(m["router"]["experts"]):
        t, j = np.nonzero(e == i)
        x = h[t]
        y[t] += p[t, j][:, None] * ((silu(x @ w[f"e{i}.gate"].T) * (x @ w[f"e{i}.up"].T)) @ w[f"e{i}.down"].T)
    return y


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta, "mamba2": mamba2}


def group(W: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}


def layer(x: np.ndarray, i: int, cfg: dict, W: dict) -> np.ndarray:
    spec, eps = cfg["layers"][i], cfg["norm"]["eps"]
    h = layer_norm(x, W[f"l{i}.norm1"], eps)
    y = MIXERS[spec["type"]](h, group(W, f"l{i}.mix."), spec["mixer"], eps)
    return x + (y if spec["mlp"] is None else y + moe(h, group(W, f"l{i}.mlp."), spec["mlp"]))


def schedule(cfg: dict) -> list[tuple[int, int | None]]:
    """The runs in order: (layer, number of the pass that starts with it or None)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def forward(tokens, cfg: dict, W: dict, dtype=np.float64, want_layers: bool = False):
    """logits [n, vocab] (and the residual stream after every run of a layer)."""
    W = {k: v.astype(dtype) for k, v in W.items()}
    x0 = W["embed"][np.asarray(tokens)]
    x, states = x0, []
    for i, t in schedule(cfg):
        if t is not None:
            x = np.concatenate([x, x0], axis=1) @ W["loop.in"].T + W["loop.step"][t]
        x = layer(x, i, cfg, W)
        states.append(x)
    logits = layer_norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T * cfg["logit_scale"]
    return (logits, states) if want_layers else logits


def greedy(prompt, n_new: int, cfg: dict, W: dict) -> list[int]:
    out = [int(t) for t in prompt]
    for _ in range(n_new):
        out.append(int(np.argmax(forward(out, cfg, W)[-1])))
    return out
