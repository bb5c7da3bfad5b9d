"""Plain NumPy restatement of the Totolorn decoder, one function per mechanism (float64 by default, no caches, no batching).

    x_0[p]      = E[token_p] + P[p]
    per layer:    x <- x + m * rho(mixer(rho(x; n1)); n1b)        rho(x; w) = x / sqrt(mean(x^2) + eps) * (1 + w)
                  x <- x + m * rho(swiglu(rho(x; n2)); n2b)       (absent when the layer has no feed-forward)
    mixer(h):     c = rms(D h) * w_c,   q = Q h,   k_a = U_a c,   v_a = V_a c     (head a)
                  s_a(i, j) = scale * q_a(i) . k_a(j)  for 0 <= i - j < window;   y_a = sigmoid((G h)_a) * softmax(s_a) v_a;   O y
    logits      = head . rho(x; final)

Shares no code with pygpukit_amd: it is what the HIP kernels are compared with."""

from __future__ import annotations

import numpy as np


def rms_scale(x: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_around_zero(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    return rms_scale(x, eps) * (1.0 + w)


def sigmoid(z: np.ndarray) -> np.ndarray:
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def swiglu(h: np.ndarray, gate: np.ndarray, up: np.ndarray, down: np.ndarray) -> np.ndarray:
    z = h @ gate.T
    return (z * sigmoid(z) * (h @ up.T)) @ down.T


def latents(h: np.ndarray, dkv: np.ndarray, dkv_norm: np.ndarray, eps: float) -> np.ndarray:
    return rms_scale(h @ dkv.T, eps) * dkv_norm


def window_mask(n: int, window: int | None) -> np.ndarray:
    d = np.arange(n)[:, None] - np.arange(n)[None, :]
    return (d >= 0) & ((d < window) if window is not None else True)


def masked_softmax(s: np.ndarray, visible: np.ndarray) -> np.ndarray:
    s = np.where(visible, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def attend(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, window: int | None) -> np.ndarray:
    """q, k [n, heads, dim], v [n, heads, vdim] -> [n, heads, vdim]."""
    vis = window_mask(q.shape[0], window)
    out = np.empty(v.shape, v.dtype)
    for a in range(q.shape[1]):
        out[:, a] = masked_softmax(scale * (q[:, a] @ k[:, a].T), vis) @ v[:, a]
    return out


def latent_attention(h: np.ndarray, w: dict, m: dict, eps: float) -> np.ndarray:
    n, H = h.shape[0], m["heads"]
    c = latents(h, w["dkv"], w["dkv.norm"], eps)
    q = (h @ w["q"].T).reshape(n, H, m["dim"])
    k = (c @ w["uk"].T).reshape(n, H, m["dim"])
    v = (c @ w["uv"].T).reshape(n, H, m["vdim"])
    window = m["mask"]["size"] if m.get("mask") else None
    y = attend(q, k, v, m["scale"], window) * sigmoid(h @ w["g"].T)[:, :, None]
    return y.reshape(n, H * m["vdim"]) @ w["o"].T


def embed(tokens, W: dict, start: int = 0) -> np.ndarray:
    t = np.asarray(tokens)
    return W["embed"][t] + W["pos"][start:start + len(t)]


def group(W: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}


def layer(x: np.ndarray, i: int, cfg: dict, W: dict) -> np.ndarray:
    eps, mult, spec = cfg["norm"]["eps"], cfg["residual_mult"], cfg["layers"][i]
    y = latent_attention(norm_around_zero(x, W[f"l{i}.norm1"], eps), group(W, f"l{i}.mix."), spec["mixer"], eps)
    x = x + mult * norm_around_zero(y, W[f"l{i}.norm1b"], eps)
    if spec["mlp"] is not None:
        f = group(W, f"l{i}.mlp.")
        y = swiglu(norm_around_zero(x, W[f"l{i}.norm2"], eps), f["gate"], f["up"], f["down"])
        x = x + mult * norm_around_zero(y, W[f"l{i}.norm2b"], eps)
    return x


def forward(tokens, cfg: dict, W: dict, dtype=np.float64, want_layers: bool = False):
    """logits [n, vocab] (and the residual stream after every layer)."""
    W = {k: v.astype(dtype) for k, v in W.items()}
    x = embed(tokens, W)
    states = []
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, W)
        states.append(x)
    logits = norm_around_zero(x, W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T
    return (logits, states) if want_layers else logits


def greedy(prompt, n_new: int, cfg: dict, W: dict) -> list[int]:
    out = [int(t) for t in prompt]
    for _ in range(n_new):
        out.append(int(np.argmax(forward(out, cfg, W)[-1])))
    return out
