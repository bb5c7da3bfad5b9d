"""Ratasun (layer-list decoder of parallel layers: rotated latent attention, a gated delta rule, a state-space mixer, mixtures of experts,
a stretch of layers that runs several times) against the plain NumPy restatement in oracle/ratasun_ref.py.

Weights are random with sharp attention scores and decays between fast and almost none, so that a lost key, a stale cache row or a lost state
moves the logits by far more than the tolerances; test_weights_tell_mechanisms_apart asserts that on the CPU.  A token's experts are decided
by three columns of the residual stream that the layers leave alone (eight classes of tokens), with router seeds for which no choice is
close: bfloat16 rounding must not change it.  The operator's own tests route by whole random rows."""

from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests.layer_list import bf16, dev, host, logit_err, rounded, save, tokens
from oracle import ratasun_ref as R

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
gpu = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 5e-2}       # rms over the vocabulary of the logit difference / rms of the logits
ROUGH = 0.25                                    # bfloat16, for single rows: a head's read-out near zero is blown up by its norm, rounding with it
CODE = 3                                        # columns that decide the experts


def near(got, want, dtype):
    """fp32: every row is within the tolerance; bfloat16: all rows but one, or one in fifty, are, and those are within ROUGH."""
    d = np.asarray(got, np.float64) - want
    err = np.sqrt(np.mean(d * d, axis=-1)) / np.sqrt(np.mean(want * want))
    if dtype == "float32":
        return bool(np.all(err < TOL[dtype]))
    return bool(np.all(err < ROUGH)) and int(np.sum(err > TOL[dtype])) <= max(1, err.size // 50)


def latent(heads, dim, rot, vdim, rank, scale, base=10000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale, "rot": {"base": base, "dims": rot}}}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def mamba(heads, groups, state, vdim, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}}


def moe(experts, top, ff, groups, keep, scale=1.0):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}}


def config(width, vocab, layers, loop=None, eps=1e-5, logit_scale=1.0, ranks=(20, 12)):
    c = {"architecture": "Ratasun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": [dict(m, mlp=e) for m, e in layers]}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c, ranks


_C = {
    # every layer different, no width a multiple of 16, feed-forwards absent beside each kind of mixer, a loop in the middle
    "mixed": config(90, 211, [(latent(6, 24, 10, 40, 50, 0.2), moe(10, 3, 50, 5, 2, 1.7)), (delta(6, 2, 24, 40, 4), moe(9, 2, 33, 3, 2, 0.8)), (mamba(6, 2, 24, 20, 3, 3), None),
                              (latent(3, 18, 6, 22, 33, 0.3, 500.0), None), (delta(3, 3, 10, 6, 2), None), (mamba(4, 4, 10, 18, 4, 1), moe(8, 4, 40, 2, 1, 2.5)),
                              (latent(4, 30, 4, 10, 130, 0.2), moe(6, 2, 70, 6, 4))], (1, 4, 2), 1e-6, 0.5),
    # one head, one tap, one expert, one pair of rotated columns; everything loops, a recurrence first and last
    "odd": config(70, 97, [(mamba(1, 1, 6, 10, 1, 1), moe(1, 1, 20, 1, 1, 1.3)), (latent(1, 7, 2, 9, 11, 0.5, 100.0), moe(2, 1, 30, 1, 1)), (delta(1, 1, 6, 10, 1), moe(4, 4, 10, 2, 2, 3.0))],
                  (0, 3, 3), 1e-3, 2.0, (1, 3)),
    # head widths past each width class of the kernels, more taps than the registers hold
    "wide": config(192, 130, [(latent(2, 144, 32, 72, 300, 0.1), moe(16, 3, 64, 4, 2)), (delta(2, 1, 144, 272, 6), None), (mamba(2, 1, 256, 64, 7, 2), moe(5, 2, 128, 1, 1)),
                              (latent(1, 136, 64, 300, 900, 0.1), None), (mamba(3, 3, 48, 144, 5, 1), None), (delta(1, 1, 200, 64, 3), None)], (4, 6, 2), ranks=(70, 130)),
    # widths the engine takes without padding, no loop
    "tiles": config(128, 256, [(latent(16, 48, 16, 64, 192, 0.15), moe(16, 4, 64, 4, 2, 1.5)), (delta(4, 2, 64, 64, 4), moe(16, 2, 128, 4, 1)), (mamba(4, 1, 64, 64, 4, 4), moe(8, 2, 64, 4, 3)),
                               (latent(20, 96, 32, 128, 448, 0.1), None), (delta(2, 2, 128, 128, 4), None), (mamba(2, 2, 128, 128, 4, 2), None), (delta(3, 1, 32, 48, 4), None)], ranks=(64, 64)),
    # long rows, wide experts
    "long": config(1100, 120, [(latent(2, 30, 20, 30, 64, 0.2), moe(6, 2, 1400, 2, 1)), (mamba(3, 1, 32, 48, 4, 3), moe(4, 2, 300, 2, 2)), (delta(3, 3, 32, 48, 3), None)], (1, 3, 2)),
    # many experts; near one-hot attention over hundreds of keys
    "deep": config(64, 90, [(latent(8, 16, 16, 64, 40, 0.2), moe(96, 6, 32, 8, 3, 2.0)), (delta(2, 1, 16, 48, 4), None), (latent(33, 16, 8, 48, 64, 0.2), None), (mamba(2, 1, 16, 48, 4, 1), None)],
                   (2, 4, 2)),
}
CONFIGS, RANKS = {k: c for k, (c, _) in _C.items()}, {k: r for k, (_, r) in _C.items()}
SHARP = {"deep": 6.0}
# seeds of the routers, layer by layer (test_no_choice_is_close)
ROUTERS = {"mixed": {0: 8, 1: 12, 5: 0, 6: 53}, "odd": {0: 0, 1: 2, 2: 0}, "wide": {0: 20, 2: 0}, "tiles": {0: 10, 1: 1, 2: 19}, "long": {0: 0, 1: 4}, "deep": {0: 56}}


def weights(name, seed=0, routers=None):
    cfg, (rank_a, rank_g), sharp = CONFIGS[name], RANKS[name], SHARP.get(name, 2.5)
    routers = ROUTERS.get(name, {}) if routers is None else routers
    rng = np.random.default_rng(seed)

    def draw(*shape, std):
        return rng.standard_normal(shape) * std

    def into(rows, cols):                                      # a sublayer's output matrix: the code columns stay as they are
        w = draw(rows, cols, std=0.6 / np.sqrt(cols))
        w[:CODE] = 0.0
        return w

    H, W = cfg["width"], {}
    W["embed"] = draw(cfg["vocab"], H, std=1.0)
    W["embed"] = R.layer_norm(W["embed"], 1.0, 0.0)
    W["embed"][:, :CODE] = 2.0 * np.sign(draw(cfg["vocab"], CODE, std=1.0))
    if cfg.get("loop"):
        W["loop.in"], W["loop.step"] = into(H, 2 * H) / 0.6, draw(cfg["loop"]["times"], H, std=0.3)
        W["loop.in"][range(CODE), range(CODE)], W["loop.step"][:, :CODE] = 1.0, 0.0
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        n, v = m["heads"], m["vdim"]
        lin = lambda rows: draw(rows, H, std=1 / np.sqrt(H))  # noqa: E731
        W[p + "norm1"] = 1.0 + draw(H, std=0.2)
        if l["type"] == "latent_attention":
            d, r, K = m["dim"], m["rot_dim"], m["kv_rank"]
            W[p + "mix.q"] = lin(n * (d + r)) * sharp / (m["scale"] * np.sqrt(d + r))                  # scores of standard deviation `sharp`
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = lin(K + r), 1.0 + draw(K, std=0.3)
            W[p + "mix.uk"], W[p + "mix.uv"] = draw(n * d, K, std=1 / np.sqrt(K)), draw(n * v, K, std=1 / np.sqrt(K))
        elif l["type"] == "channel_delta":
            d, g = m["dim"], m["kv_heads"]
            for x, rows in (("q", g * d), ("k", g * d), ("v", n * v)):
                W[p + f"mix.{x}"], W[p + f"mix.{x}.conv"] = lin(rows), draw(rows, m["conv"], std=0.8)
            W[p + "mix.b"], W[p + "mix.A_log"], W[p + "mix.dt_bias"] = lin(n), rng.uniform(-1, 1, n), rng.uniform(-6, 1, n * d)
            W[p + "mix.a1"], W[p + "mix.a2"] = lin(rank_a), draw(n * d, rank_a, std=1 / np.sqrt(rank_a))
            W[p + "mix.g1"], W[p + "mix.g2"] = lin(rank_g), draw(n * v, rank_g, std=1 / np.sqrt(rank_g))
            W[p + "mix.norm"] = 1.0 + draw(v, std=0.3)
        else:
            N, g = m["state"], m["groups"]
            ch = n * v + 2 * g * N
            W[p + "mix.in"], W[p + "mix.conv"], W[p + "mix.conv.b"] = lin(n * v + ch + n), draw(ch, m["conv"], std=0.8), draw(ch, std=0.3)
            W[p + "mix.A_log"], W[p + "mix.dt_bias"], W[p + "mix.D"] = rng.uniform(-3, 1, n), rng.uniform(-3, 1, n), draw(n, std=1.0)
            W[p + "mix.norm"] = 1.0 + draw(n * v, std=0.3)
        W[p + "mix.o"] = into(H, n * v)
        if l["mlp"]:
            f, E = l["mlp"]["expert"]["ff"], l["mlp"]["router"]["experts"]
            for e in range(E):
                W[p + f"mlp.e{e}.gate"], W[p + f"mlp.e{e}.up"], W[p + f"mlp.e{e}.down"] = lin(f), lin(f), into(H, f)
            own = np.random.default_rng(1000 * i + routers.get(i, 0))
            W[p + "mlp.router"] = own.standard_normal((E, H)) * 0.01 / np.sqrt(H)
            W[p + "mlp.router"][:, :CODE] = own.standard_normal((E, CODE)) * 0.5
            W[p + "mlp.correction"] = own.uniform(-0.8, 0.8, E)
    W["final.norm"], W["head"] = 1.0 + draw(H, std=0.2), draw(cfg["vocab"], H, std=1 / np.sqrt(H))
    return {k: bf16(x) for k, x in W.items()}


def choice_margins(cfg, W, t):
    """Per layer with experts: the smallest distance of a choice (of groups, of experts) from another one, over the tokens and passes."""
    out: dict[int, float] = {}
    W = {k: v.astype(np.float64) for k, v in W.items()}
    x0 = x = W["embed"][np.asarray(t)]
    for i, begin in R.schedule(cfg):
        if begin is not None:
            x = np.concatenate([x, x0], axis=1) @ W["loop.in"].T + W["loop.step"][begin]
        l = cfg["layers"][i]
        if l["mlp"]:
            r, p = l["mlp"]["router"], f"l{i}.mlp."
            c = R.sigmoid(R.layer_norm(x, W[f"l{i}.norm1"], cfg["norm"]["eps"]) @ W[p + "router"].T) + W[p + "correction"]
            n, E, cnt, keep = len(t), r["experts"], r["groups"]["count"], r["groups"]["keep"]
            best = np.sort(c.reshape(n, cnt, -1), axis=2)[:, :, -2:].sum(axis=2)
            gaps = [np.inf]
            rank = np.argsort(-best, axis=1)
            g = np.take_along_axis(best, rank, axis=1)
            if keep < cnt:
                gaps.append(np.min(g[:, keep - 1] - g[:, keep]))
            free = np.zeros((n, cnt), bool)
            np.put_along_axis(free, rank[:, :keep], True, axis=1)
            c = -np.sort(-np.where(np.repeat(free, E // cnt, axis=1), c, -np.inf), axis=1)
            if r["top"] < E:
                gaps.append(np.min(c[:, r["top"] - 1] - c[:, r["top"]]))
            out[i] = min(out.get(i, np.inf), *gaps)
        x = R.layer(x, i, cfg, W)
    return out


# ------------------------------------------------------------------------------------------------ CPU: configuration, oracle
def test_config_is_read_layer_by_layer():
    from pygpukit_amd.llm import RATASUN_SPEC, detect_model_spec, layer_list_config

    c = layer_list_config(CONFIGS["mixed"])
    assert (c.hidden_size, c.vocab_size, c.num_layers, c.norm_eps, c.logit_scale, c.norm_type) == (90, 211, 7, 1e-6, 0.5, "layernorm")
    a, b, d, e = c.layers[:4]
    assert (a.mixer, a.num_heads, a.head_dim, a.rot_dim, a.v_head_dim, a.kv_rank, a.scale, a.rot_base, a.window, a.intermediate_size) == \
        ("latent_attention", 6, 24, 10, 40, 50, 0.2, 10000.0, None, 50)
    assert (a.experts.count, a.experts.top, a.experts.groups, a.experts.keep, a.experts.scale) == (10, 3, 5, 2, 1.7)
    assert (b.mixer, b.num_heads, b.num_kv_heads, b.head_dim, b.v_head_dim, b.conv_taps) == ("channel_delta", 6, 2, 24, 40, 4)
    assert (d.mixer, d.num_heads, d.num_kv_heads, d.head_dim, d.v_head_dim, d.conv_taps, d.norm_groups, d.experts) == ("mamba2", 6, 2, 24, 20, 3, 3, None)
    assert e.rot_base == 500.0 and e.intermediate_size is None
    assert [r for r, _ in c.loop.runs(7)] == [0, 1, 2, 3, 1, 2, 3, 4, 5, 6] and [t for _, t in c.loop.runs(7)] == [None, 0, None, None, 1, None, None, None, None, None]
    assert detect_model_spec(["embed"], CONFIGS["mixed"]) is RATASUN_SPEC
    assert layer_list_config(CONFIGS["tiles"]).loop is None

    def broken(layer, part, **kw):
        x = json.loads(json.dumps(CONFIGS["mixed"]))
        target = x["layers"][layer]
        for key in part:
            target = target[key]
        target.update(kw)
        return x

    for layer, part, kw in ((0, ("mixer",), {"rot_dim": 9}), (0, ("mixer", "rot"), {"dims": 8}), (1, ("mixer",), {"kv_heads": 4}), (2, ("mixer",), {"norm_groups": 7}),
                            (2, ("mixer",), {"groups": 4}), (0, ("mlp", "router"), {"top": 5}), (0, ("mlp", "router", "groups"), {"count": 3}), (1, (), {"type": "gru"})):
        with pytest.raises(ValueError, match=f"layer {layer}"):
            layer_list_config(broken(layer, part, **kw))
    with pytest.raises(ValueError, match="cannot run layers"):
        layer_list_config({**CONFIGS["mixed"], "loop": {"start": 3, "stop": 3, "times": 2}})


def test_oracle_mechanisms_on_hand_made_numbers():
    np.testing.assert_allclose(R.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 5.0]), 0.0), [[-2.0, 5.0]])
    np.testing.assert_allclose(R.rotate(np.array([[1.0, 0.0, 0.0, 1.0]]), np.array([2]), 100.0), [[np.cos(2), np.sin(2), -np.sin(0.2), np.cos(0.2)]])
    u = np.array([[1.0], [10.0], [100.0]])
    np.testing.assert_allclose(R.short_conv(u, np.array([[3.0, 2.0]]), np.array([5.0]))[:, 0], [7.0, 28.0, 235.0])
    # one channel: S = 4 after the write; the decay comes first, the read-out sees the write
    k, one = np.ones((2, 1, 1)), np.ones((2, 1))
    o, S = R.delta_rule(2 * k, k, np.array([4.0, 10.0]).reshape(2, 1, 1), np.full((2, 1, 1), 0.5), np.array([[1.0], [0.25]]))
    np.testing.assert_allclose((o[0, 0, 0], o[1, 0, 0], S[0, 0, 0]), (8.0, 2 * (2 + 0.25 * 8), 4.0))
    y, S = R.state_space(np.array([4.0, 10.0]).reshape(2, 1, 1), k, 3 * k, one * np.log(2.0), np.array([1.0]), np.array([0.5]))
    np.testing.assert_allclose(y[:, 0, 0], [12 * np.log(2) + 2, 3 * (2 + 10) * np.log(2) + 5])
    np.testing.assert_allclose(R.parts_norm(np.array([[3.0, 4.0, 0.0, 2.0]]), 2, 0.0), [[3 / 12.5**0.5, 4 / 12.5**0.5, 0.0, 2**0.5]])
    s, corr = np.array([[0.9, 0.1, 0.5, 0.6]]), np.array([-0.8, 0.0, -0.1, -0.3])
    e, p = R.choose(s, corr, {"top": 2, "scale": 2.0})
    assert list(e[0]) == [2, 3]
    np.testing.assert_allclose(p[0], [2 * 0.5 / 1.1, 2 * 0.6 / 1.1])
    assert list(R.choose(s, corr - 1.0, {"top": 2, "scale": 1.0, "groups": {"count": 2, "keep": 1}})[0][0]) == [2, 3]       # closed groups lose to negative choices too
    assert list(R.choose(s, np.array([0.5, 0.0, 0.2, -0.3]), {"top": 2, "scale": 1.0, "groups": {"count": 2, "keep": 1}})[0][0]) == [0, 1]


@pytest.mark.parametrize("name", list(CONFIGS))
def test_no_choice_is_close(name):
    m = choice_margins(CONFIGS[name], weights(name), tokens(CONFIGS[name], 200, 3))
    assert min(m.values()) > 0.012, m


def test_weights_tell_mechanisms_apart():
    """A missing tap, bias, decay, gate or norm, another rotation, another choice of experts, another order of steps in the loop: each moves
    the logits by hundreds of times the fp32 tolerance."""
    name = "mixed"
    cfg, t = CONFIGS[name], tokens(CONFIGS[name], 100, 3)
    W = weights(name)
    want = R.forward(t, cfg, W)

    def moved(c, w):
        return logit_err(R.forward(t, c, w), want) > 300 * TOL["float32"]

    closed = []
    for i, l in enumerate(cfg["layers"]):
        keys = {"latent_attention": ("dkv.norm", "uk", "uv"), "channel_delta": ("q.conv", "k.conv", "v.conv", "b", "A_log", "a2", "dt_bias", "g2", "norm"),
                "mamba2": ("conv", "conv.b", "A_log", "dt_bias", "D", "norm")}[l["type"]]
        for key in (f"l{i}.mix.{k}" for k in keys):
            if W[key].size > 1:
                assert moved(cfg, {**W, key: np.roll(W[key], 1, axis=-1)}), key
                assert moved(cfg, {**W, key: np.zeros_like(W[key])}), key
        parts = [("mixer", "scale", 0.9), ("rot", "base", 0.8)] if l["type"] == "latent_attention" else []
        if l["mlp"]:
            assert moved(cfg, {**W, f"l{i}.mlp.correction": np.zeros_like(W[f"l{i}.mlp.correction"])}) and moved(cfg, {**W, f"l{i}.norm1": np.ones_like(W[f"l{i}.norm1"])})
            parts += [("router", "scale", 0.9), ("router", "keep", 2)]
        for part, key, f in parts:
            other = json.loads(json.dumps(cfg))
            m = other["layers"][i]
            target = m["mixer"] if part == "mixer" else m["mixer"]["rot"] if part == "rot" else m["mlp"]["router"] if key == "scale" else m["mlp"]["router"]["groups"]
            target[key] = target["count"] if key == "keep" else target[key] * f
            if key == "keep":                                  # (where the closed groups hold no large choice, it does not show)
                closed.append(moved(other, W))
            else:
                assert moved(other, W), (i, part, key)
    assert any(closed)
    assert moved(cfg, {**W, "loop.step": W["loop.step"][::-1]}) and moved(cfg, {**W, "loop.in": np.roll(W["loop.in"], cfg["width"], axis=1)})
    assert moved({**cfg, "loop": dict(cfg["loop"], times=1)}, W)


def test_loop_gives_every_pass_its_own_cache():
    """The product's order of runs is the restatement's."""
    from pygpukit_amd.llm import LoopConfig

    for name, cfg in CONFIGS.items():
        if cfg.get("loop"):
            assert LoopConfig(**cfg["loop"]).runs(len(cfg["layers"])) == R.schedule(cfg), name


# ------------------------------------------------------------------------------------------------ GPU: operators
OP_TOL = {"float32": 3e-6, "bfloat16": 1.5e-2}
both = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def worst(got, want):
    return float(np.max(np.abs(got - want)) / np.max(np.abs(want)))


@gpu
@both
def test_norm_taps_and_rotation(dtype):
    from pygpukit_amd.ops.basic import conv_silu, latent_rows, layernorm_f32, rotate_pairs

    rng = np.random.default_rng(1)
    x, w = (rng.standard_normal((9, 77)) * 3 + 5).astype(np.float32), (1 + 0.3 * rng.standard_normal(77)).astype(np.float32)
    assert worst(host(layernorm_f32(dev(x, "float32"), dev(w, "float32"), 1e-3, dtype=dev(x, dtype).dtype)), R.layer_norm(x.astype(np.float64), w, 1e-3)) < OP_TOL[dtype]
    for taps, ch in ((1, 8), (2, 12), (3, 4), (4, 1028), (5, 20), (9, 8)):
        u, c, b = rounded(rng.standard_normal((40, ch)), dtype), rounded(rng.standard_normal((ch, taps)), dtype), rng.standard_normal(ch).astype(np.float32)
        for bias in (None, b):
            want = R.silu(R.short_conv(u.astype(np.float64), c.astype(np.float64), None if bias is None else bias.astype(np.float64)))
            db = None if bias is None else dev(bias, "float32")
            assert worst(host(conv_silu(dev(u, dtype), dev(c.T, dtype), bias=db)), want) < OP_TOL[dtype]
            if taps > 1:
                for cut in (taps - 1, 22):
                    assert worst(host(conv_silu(dev(u[cut:], dtype), dev(c.T, dtype), dev(u[cut - taps + 1:cut], dtype), bias=db)), want[cut:]) < OP_TOL[dtype]
    for rank, rot, first in ((50, 10, 0), (128, 64, 7), (1, 2, 900), (513, 30, 40)):
        x, c = rounded(rng.standard_normal((6, rank + rot)), dtype), (1 + 0.3 * rng.standard_normal(rank)).astype(np.float32)
        freq = (300.0 ** (-2.0 * np.arange(rot // 2) / rot)).astype(np.float32)
        p = first + np.arange(6)
        turned = R.rotate(x[:, rank:].astype(np.float64), p, 300.0)
        want = np.concatenate([R.rms(x[:, :rank].astype(np.float64), 1e-4) * c, turned], axis=1)
        tol = max(OP_TOL[dtype], 3e-7 * first)                                      # an fp32 angle of `first` radians
        assert worst(host(latent_rows(dev(x, dtype), dev(c, "float32"), dev(freq, "float32"), first, eps=1e-4)), want) < tol
        q = rounded(rng.standard_normal((6, 3, rank + rot)), dtype)
        want = q.astype(np.float64)
        want[:, :, rank:] = R.rotate(want[:, :, rank:], p, 300.0)
        assert worst(host(rotate_pairs(dev(q, dtype), dev(freq, "float32"), first)), want) < tol


def delta_case(rng, n, heads, kv, dim, vdim, dtype, extreme=False):
    q, k, v, z, b, g = (rounded(rng.standard_normal((n, w)) * s, dtype) for w, s in ((kv * dim, 1.0), (kv * dim, 1.0), (heads * vdim, 1.0), (heads * dim, 30.0 if extreme else 1.0),
                                                                                    (heads, 20.0 if extreme else 1.5), (heads * vdim, 2.0)))
    rate, bias, norm = np.exp(rng.uniform(-1, 1, heads)), rng.uniform(-6, 1, heads * dim), 1 + 0.3 * rng.standard_normal(vdim)
    return (q, k, v, z, b, g), tuple(x.astype(np.float32) for x in (rate, bias, norm))


def delta_oracle(rows, consts, heads, dim, vdim, eps=1e-4):
    q, k, v, z, b, g = (x.astype(np.float64) for x in rows)
    rate, bias, norm = (x.astype(np.float64) for x in consts)
    n, kv = q.shape[0], q.shape[1] // dim
    q, k = (np.repeat(R.unit(x.reshape(n, kv, dim)), heads // kv, axis=1) for x in (q, k))
    f = np.exp(-rate[:, None] * R.softplus(z + bias).reshape(n, heads, dim))
    o, S = R.delta_rule(q * dim**-0.5, k, v.reshape(n, heads, vdim), f, R.sigmoid(b))
    return (R.rms(o, eps) * norm * R.sigmoid(g).reshape(n, heads, vdim)).reshape(n, -1), S


@gpu
@both
@pytest.mark.parametrize("heads,kv,dim,vdim", [(3, 3, 64, 80), (4, 2, 32, 48), (2, 1, 128, 128), (3, 1, 24, 40), (1, 1, 144, 272), (2, 1, 16, 16), (1, 1, 4, 4), (1, 1, 64, 512)])
def test_delta_rule(heads, kv, dim, vdim, dtype):
    """Both forms, lengths around their blocks and chunks; portions continue the state."""
    from pygpukit_amd.ops.basic import delta_rule

    rng = np.random.default_rng(dim + vdim)
    rows, consts = delta_case(rng, 330, heads, kv, dim, vdim, dtype)
    want, _ = delta_oracle(rows, consts, heads, dim, vdim)
    rate, bias, norm = (dev(x, "float32") for x in consts)
    tol = OP_TOL[dtype] if dtype == "bfloat16" else 2e-5
    for cuts in ([330], [1, 2, 15, 16, 17, 64, 65, 150], [63, 32, 31, 204]):
        state, at = dev(rng.standard_normal((heads, dim, vdim)), "float32"), 0      # fresh: what is in it does not matter
        for c in cuts:
            got = host(delta_rule(*(dev(x[at:at + c], dtype) for x in rows[:3]), dev(rows[3][at:at + c], "float32"), *(dev(x[at:at + c], dtype) for x in rows[4:]), state, decay=rate,
                                  step_bias=bias, norm=norm, eps=1e-4, fresh=at == 0))
            assert worst(got, want[at:at + c]) < tol, (cuts, at)
            at += c
            assert worst(host(state), delta_oracle([x[:at] for x in rows], consts, heads, dim, vdim)[1]) < 1e-5, (cuts, at)


@gpu
@both
def test_decays_and_strengths_at_their_limits(dtype):
    """Decays down to e^-100 a row beside none at all, strengths of 0 and 1, in every block of a chunk."""
    from pygpukit_amd.ops.basic import delta_rule

    rng = np.random.default_rng(8)
    rows, consts = delta_case(rng, 200, 2, 1, 32, 48, dtype, extreme=True)
    want, S = delta_oracle(rows, consts, 2, 32, 48)
    state = dev(np.zeros((2, 32, 48)), "float32")
    rate, bias, norm = (dev(x, "float32") for x in consts)
    got = host(delta_rule(*(dev(x, dtype) for x in rows[:3]), dev(rows[3], "float32"), *(dev(x, dtype) for x in rows[4:]), state, decay=rate, step_bias=bias, norm=norm, eps=1e-4))
    assert np.isfinite(got).all() and worst(got, want) < (OP_TOL[dtype] if dtype == "bfloat16" else 5e-5) and worst(host(state), S) < 2e-5


@gpu
def test_a_write_far_back_is_still_there():
    """One written row, decays of almost 1 and other keys after it: hundreds of rows later its key still finds it."""
    from pygpukit_amd.ops.basic import delta_rule

    n, d = 700, 32
    q, k, v = np.zeros((n, d), np.float32), np.zeros((n, d), np.float32), np.zeros((n, d), np.float32)
    k[:, 1:] = np.random.default_rng(2).standard_normal((n, d - 1))
    k[3], v[3], q[:, 0] = 0.0, 50.0, 1.0
    k[3, 0] = 1.0
    rows = (q, k, v, np.full((n, d), -8.0, np.float32), np.full((n, 1), 1.0, np.float32), np.zeros((n, d), np.float32))
    consts = tuple(np.asarray(x, np.float32) for x in (np.ones(1), np.zeros(d), np.ones(d)))
    want, S = delta_oracle(rows, consts, 1, d, d)
    state = dev(np.zeros((1, d, d)), "float32")
    got = host(delta_rule(*(dev(x, "float32") for x in rows), state, decay=dev(consts[0], "float32"), step_bias=dev(consts[1], "float32"), norm=dev(consts[2], "float32"), eps=1e-4))
    assert want[-1].min() > 0.4 and np.max(np.abs(got[4:] - want[4:])) < 1e-4 and worst(host(state), S) < 1e-4


@gpu
@both
@pytest.mark.parametrize("heads,groups,dim,vdim,parts", [(2, 1, 64, 64, 1), (6, 2, 24, 20, 3), (4, 4, 128, 128, 2), (1, 1, 256, 64, 1), (3, 3, 48, 144, 1), (1, 1, 6, 10, 1), (6, 2, 32, 80, 2),
                                                         (2, 2, 16, 512, 4)])
def test_state_space(heads, groups, dim, vdim, parts, dtype):
    from pygpukit_amd.ops.basic import state_space

    rng = np.random.default_rng(dim + vdim)
    n, v, g = 330, heads * vdim, groups * dim
    xbc, z, t = (rounded(rng.standard_normal((n, w)), dtype) for w in (v + 2 * g, v, heads))
    rate, bias, skip, norm = (x.astype(np.float32) for x in (np.exp(rng.uniform(-3, 1.5, heads)), rng.uniform(-3, 1, heads), rng.standard_normal(heads), 1 + 0.3 * rng.standard_normal(v)))

    def oracle(m):
        X, B, C = np.split(xbc[:m].astype(np.float64), [v, v + g], axis=1)
        B, C = (np.repeat(a.reshape(m, groups, dim), heads // groups, axis=1) for a in (B, C))
        y, S = R.state_space(X.reshape(m, heads, vdim), B, C, R.softplus(t[:m].astype(np.float64) + bias), rate.astype(np.float64), skip.astype(np.float64))
        return R.parts_norm(y.reshape(m, v) * R.silu(z[:m].astype(np.float64)), parts, 1e-4) * norm, S

    want, _ = oracle(n)
    kw = dict(groups=groups, decay=dev(rate, "float32"), step_bias=dev(bias, "float32"), skip=dev(skip, "float32"), norm=dev(norm, "float32"), norm_groups=parts, eps=1e-4)
    tol = OP_TOL[dtype] if dtype == "bfloat16" else 2e-5
    for cuts in ([330], [1, 2, 15, 16, 17, 64, 65, 150], [63, 32, 31, 204]):
        state, at = dev(rng.standard_normal((heads, dim, vdim)), "float32"), 0
        for c in cuts:
            got = host(state_space(*(dev(x[at:at + c], dtype) for x in (xbc, z, t)), state, fresh=at == 0, **kw))
            assert worst(got, want[at:at + c]) < tol, (cuts, at)
            at += c
            assert worst(host(state), oracle(at)[1]) < 1e-5, (cuts, at)


@gpu
@both
@pytest.mark.parametrize("n", [1, 3, 40, 130, 700])
@pytest.mark.parametrize("E,top,groups,keep,ff,H", [(15, 4, 5, 3, 80, 320), (8, 2, 0, 0, 50, 90), (1, 1, 0, 0, 64, 64), (5, 5, 5, 5, 30, 200), (200, 8, 10, 4, 64, 192), (16, 1, 8, 2, 320, 576)])
def test_experts(n, E, top, groups, keep, ff, H, dtype):
    """Routing by whole random rows, negative choices among them; one row, few rows per expert, and tiles of them."""
    from pygpukit_amd.ops.basic import mixture_of_experts

    rng = np.random.default_rng(n + E)
    x, router = rounded(rng.standard_normal((n, H)), dtype), rounded(rng.standard_normal((E, H)) * 1.5 / np.sqrt(H), dtype)
    gu, down = rounded(rng.standard_normal((E, 2 * ff, H)) / np.sqrt(H), dtype), rounded(rng.standard_normal((E, H, ff)) / np.sqrt(ff), dtype)
    corr = rng.uniform(-1, 0.5, E).astype(np.float32)
    w = {"router": router, "correction": corr}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = gu[e, :ff], gu[e, ff:], down[e]
    r = {"experts": E, "top": top, "scale": 1.7}
    if groups:
        r["groups"] = {"count": groups, "keep": keep}
    want = R.moe(x.astype(np.float64), {k: v.astype(np.float64) for k, v in w.items()}, {"router": r})
    got = host(mixture_of_experts(dev(x, dtype), dev(router, dtype), dev(corr, "float32"), dev(gu, dtype), dev(down, dtype), top=top, groups=groups, keep=keep, scale=1.7))
    assert got.shape == want.shape and worst(got, want) < OP_TOL[dtype]


# ------------------------------------------------------------------------------------------------ GPU: model and engine
_models: dict = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """(config, weights, model) by name and dtype, loaded from a checkpoint on disk by the product loader."""
    from pygpukit_amd.llm import load_model_from_safetensors

    def get(name, dtype):
        if (name, dtype) not in _models:
            W = weights(name)
            folder = save(tmp_path_factory.mktemp(name), CONFIGS[name], W)
            _models[name, dtype] = (CONFIGS[name], W, load_model_from_safetensors(folder, dtype=dtype), folder)
        return _models[name, dtype][:3]

    yield get
    _models.clear()


_ref: dict = {}


def reference(name, n, seed=5):
    if (name, n, seed) not in _ref:
        t = tokens(CONFIGS[name], n, seed)
        _ref[name, n, seed] = (t, R.forward(t, CONFIGS[name], weights(name)))
    return _ref[name, n, seed]


every = pytest.mark.parametrize("name", list(CONFIGS))


@gpu
@both
@every
def test_eager_model(models, name, dtype):
    cfg, W, model = models(name, dtype)
    t, want = reference(name, 90)
    hidden, past = model(t[:80], use_cache=True)
    got = [host(model.get_logits(hidden))]
    for i in range(80, 84):
        before = [tuple(host(a).copy() for a in p) for p in past] if i == 80 else None
        hidden, new = model([t[i]], past_key_values=past, use_cache=True)
        if before is not None:                                 # a step leaves the state it started from alone
            for p, saved in zip(past, before):
                for a, b in zip(p, saved):
                    np.testing.assert_array_equal(host(a), b)
        past = new
        got.append(host(model.get_logits(hidden)))
    hidden, _ = model(t[84:], past_key_values=past, use_cache=True)
    got.append(host(model.get_logits(hidden)))
    assert near(np.concatenate(got), want, dtype)


@gpu
@both
def test_fixed_cache_strategies(models, dtype):
    from pygpukit_amd.llm import DecodeBatch, DecodeBuffers, DecodeM1

    cfg, W, model = models("tiles", dtype)
    t, want = reference("tiles", 90)
    model.init_fixed_cache(100)
    got = [host(model.prefill_fixed_cache(t[:50]))]
    m1, mb = DecodeM1(), DecodeBatch(4)
    m1.bind(model)
    mb.bind(model)
    buf = DecodeBuffers.allocate(model.config, dtype=dtype, vocab_size=cfg["vocab"])
    saved = None
    for i in range(50, 60):
        got.append(host(m1.step(t[i], i, i + 1, buf)).copy())
        if i == 54:
            saved = model.snapshot_kv_cache()
    got.append(host(mb.step_batch(t[60:64], 60, 64)))
    assert near(np.concatenate(got), want[:64], dtype)
    model.restore_kv_cache(saved)
    assert near(host(mb.step_batch(t[55:60], 55, 60)), want[55:60], dtype)
    assert near(host(mb.step_batch(t[:5], 0, 5)), want[:5], dtype)       # position 0 starts again
    with pytest.raises(NotImplementedError, match="one pass"):
        models("mixed", dtype)[2].init_fixed_cache(100)


@gpu
@both
@every
def test_engine_prompt_every_row(models, name, dtype):
    cfg, W, model = models(name, dtype)
    n = {"tiles": 400, "deep": 700}.get(name, 150)
    t, want = reference(name, n)
    e = model.build_engine(max_seq_len=n, max_batch=2)
    got = e.prefill_batch([t], [1], want=[list(range(n))])
    assert got.shape == want.shape and near(got, want, dtype)
    for k in (1, 2, 3, 4, 17):                                 # the first tokens of a sequence as whole prompts
        assert near(e.prefill(t[:k], seq=0)[None], want[k - 1:k], dtype)


@gpu
@both
@every
@pytest.mark.parametrize("batch", [1, 3, 9])
def test_engine_decode_is_the_prompt(models, name, dtype, batch):
    """Token by token from the very first one, in batches of sequences that run at different positions."""
    cfg, W, model = models(name, dtype)
    n = 110
    t, want = reference(name, 150)
    e = model.build_engine(max_seq_len=128, max_batch=batch)
    lag = [5 * b for b in range(batch)]                        # sequence b starts with a prompt of lag[b] tokens
    for b in range(batch):
        if lag[b]:
            e.prefill(t[:lag[b]], seq=b, want_last_logits=False)
    got, exp = [], []
    for i in range(n - max(lag)):
        e.set_state([t[p + i] for p in lag], [p + i for p in lag])
        e.decode_step(batch)
        got.append(e.logits(batch).to_numpy())
        exp.append(want[[p + i for p in lag]])
    assert near(np.concatenate(got), np.concatenate(exp), dtype)


@gpu
@both
@every
@pytest.mark.parametrize("sizes", [[2], [3, 64, 1], [63, 2, 65], [1, 2, 33, 7, 50]])
def test_engine_portions(models, name, dtype, sizes):
    cfg, W, model = models(name, dtype)
    n = 120 if sizes == [2] else 150
    t, want = reference(name, 150)
    e = model.build_engine(max_seq_len=160, max_batch=1)
    got, at, k = [], 0, 0
    while at < n:
        m = min(sizes[k % len(sizes)], n - at)
        got.append(e.prefill_batch([t[at:at + m]], [0], [at], want=[list(range(m))]))
        at, k = at + m, k + 1
    assert near(np.concatenate(got), want[:n], dtype)


@gpu
@both
@every
def test_unequal_batch_and_slots_used_again(models, name, dtype):
    """Requests of different lengths together equal each alone; finished ones give their slots, with what is in them, to new ones."""
    from pygpukit_amd.llm import BatchScheduler

    cfg, W, model = models(name, dtype)
    lens = [1, 40, 7, 90]
    ref = [reference(name, n + 12, seed=20 + i) for i, n in enumerate(lens)]
    s = BatchScheduler(model.build_engine(max_seq_len=128, max_batch=4))
    for again in range(2):
        order = [3, 1, 0, 2] if again else [0, 1, 2, 3]
        out = s.step([((again, i), ref[i][0][:lens[i]], [lens[i] - 1, 0]) for i in order])
        for i, o in zip(order, out):
            assert near(o, ref[i][1][[lens[i] - 1, 0]], dtype)
        live = list(order)
        for k in range(12):
            out = s.step([((again, i), [ref[i][0][lens[i] + k]], [0]) for i in live])
            for i, o in zip(live, out):
                assert near(o, ref[i][1][[lens[i] + k]], dtype)
            if k == 4:                                         # shorter ones end earlier
                for i in (1, 0):
                    s.release((again, i))
                    live.remove(i)
        for i in live:
            s.release((again, i))
    assert s.live == ()


@gpu
@both
@pytest.mark.parametrize("batch", [1, 2, 17, 40])
def test_far_keys_in_batches(models, dtype, batch):
    """Near one-hot attention at positions up to 700, in batch sizes that give one split and several."""
    cfg, W, model = models("deep", dtype)
    n = 700
    t, want = reference("deep", n)
    e = model.build_engine(max_seq_len=720, max_batch=batch)
    at = [(590 + 13 * b) % 690 + 1 if b < 8 else 1 + (37 * b) % 680 for b in range(batch)]
    e.prefill_batch([t[:p] for p in at], want=[[]] * batch)
    got, exp = [], []
    for i in range(6):
        e.set_state([t[p + i] for p in at], [p + i for p in at])
        e.decode_step(batch)
        got.append(e.logits(batch).to_numpy())
        exp.append(want[[p + i for p in at]])
    assert near(np.concatenate(got), np.concatenate(exp), dtype)


@gpu
@pytest.mark.parametrize("packed,big_tiles", [("0", "0"), ("1", "0"), ("1", "1")])
@pytest.mark.parametrize("name", ["long", "tiles"])
def test_projection_routes_agree(models, name, packed, big_tiles, monkeypatch):
    """Fragment-major copies on and off, 128- and 256-row tiles: prompts of 2..300 rows and batches take other kernels, the logits stay
    the same."""
    monkeypatch.setenv("PGK_PACKED_PREFILL", packed)
    monkeypatch.setenv("PGK_GEMM256", big_tiles)
    cfg, W, model = models(name, "bfloat16")
    t, want = reference(name, 400)
    e = model.build_engine(max_seq_len=310, max_batch=12)
    for n in (2, 20, 100, 128, 129, 300):
        assert near(e.prefill_batch([t[:n]], want=[[0, n // 2, n - 1]]), want[[0, n // 2, n - 1]], "bfloat16")
    at = [3 * b + 1 for b in range(12)]
    e.prefill_batch([t[:p] for p in at], want=[[]] * 12)
    e.set_state([t[p] for p in at], at)
    e.decode_step(12)
    assert near(e.logits(12).to_numpy(), want[at], "bfloat16")


@gpu
@both
@pytest.mark.parametrize("name", ["tiles", "mixed"])
def test_long_decoding(models, name, dtype):
    """Hundreds of decoded tokens; the same logits from the captured graph."""
    cfg, W, model = models(name, dtype)
    t, want = reference(name, 400)
    e = model.build_engine(max_seq_len=450, max_batch=2)
    e.prefill(t[:3], seq=0, want_last_logits=False)
    e.prefill(t[:100], seq=1, want_last_logits=False)
    e.capture(2)
    got, exp = [], []
    for i in range(290):
        e.set_state([t[3 + i], t[100 + i]], [3 + i, 100 + i])
        if i % 3:
            e.replay(1)
        else:
            e.decode_step(2)
        if i % 7 == 0 or i > 280 or 58 <= i <= 66 or 121 <= i <= 128:
            got.append(e.logits(2).to_numpy())
            exp.append(want[[3 + i, 100 + i]])
    assert near(np.concatenate(got), np.concatenate(exp), dtype)
    if name == "tiles":
        assert e.recurrent_state(1).shape == (2, 4, 64, 64) and e.latent_cache(0).shape[0] == 2
        with pytest.raises(ValueError):
            e.recurrent_state(0)
    else:                                                      # runs 2 and 5 are two passes of one layer, with a state each
        assert not np.array_equal(e.recurrent_state(2).to_numpy(), e.recurrent_state(5).to_numpy())


def check_greedy(got, prompt, cfg, W, dtype):
    """Every generated token is the oracle's choice given the tokens before it, or within rounding of it."""
    want = R.forward(got[:-1], cfg, W)
    scale = np.sqrt(np.mean(want * want))
    for i in range(len(prompt), len(got)):
        row = want[i - 1]
        assert row.max() - row[got[i]] <= 3 * TOL[dtype] * scale


@gpu
@both
@pytest.mark.parametrize("name", ["mixed", "tiles", "odd"])
def test_greedy_generation(models, name, dtype):
    from pygpukit_amd.llm import BatchScheduler, DecodeBatch, DecodeM1Graph

    cfg, W, model = models(name, dtype)
    prompts = [tokens(cfg, n, 40 + n) for n in (1, 17, 5, 60, 33)]
    n_new = 24
    e = model.build_engine(max_seq_len=100, max_batch=2)
    alone = [e.generate_greedy(p, n_new) for p in prompts]
    for p, g in zip(prompts, alone):
        assert g[:len(p)] == p and len(g) == len(p) + n_new
        check_greedy(g, p, cfg, W, dtype)
    assert e.generate_greedy(prompts[1], n_new, use_graph=False) == alone[1]
    batch = BatchScheduler(model.build_engine(max_seq_len=100, max_batch=3)).generate(prompts, n_new)     # five prompts, three slots
    for p, g in zip(prompts, batch):
        check_greedy(g, p, cfg, W, dtype)
    eager = model.generate(prompts[2], max_new_tokens=8, temperature=0.0, top_k=0, top_p=1.0)
    check_greedy(eager, prompts[2], cfg, W, dtype)
    if dtype == "float32":                                     # sharp enough to be identical
        assert batch == alone and eager == alone[2][:len(eager)]
    m1 = DecodeM1Graph()
    m1.bind(model)
    m1.init_graph(100)
    first = int(np.argmax(m1.prefill(prompts[3])))
    assert prompts[3] + [first] + m1.run_greedy(first, len(prompts[3]), n_new - 1) == alone[3]
    db = DecodeBatch(3)
    db.bind(model)
    db.init_graph(100)
    f = db.prefill(prompts[:3])
    toks = db.run_greedy(f, [len(p) for p in prompts[:3]], n_new - 1)
    for b in range(3):
        check_greedy(prompts[b] + [int(f[b])] + [int(x) for x in toks[:, b]], prompts[b], cfg, W, dtype)


@gpu
@pytest.mark.parametrize("name", ["tiles", "mixed"])
def test_graph_replays_equal_eager_steps(models, name):
    """Several replays with eager work and synchronisation between them: each equals the eager step from the same state."""
    cfg, W, model = models(name, "bfloat16")
    t = tokens(cfg, 80, 77)
    for batch in (1, 5):
        a, b = (model.build_engine(max_seq_len=128, max_batch=batch) for _ in range(2))
        for e in (a, b):
            for s in range(batch):
                e.prefill(t[:60 + s], seq=s, want_last_logits=False)
        a.capture(batch)
        for i in range(8):
            tok, pos = [t[(60 + s + i) % 80] for s in range(batch)], [60 + s + i for s in range(batch)]
            a.set_state(tok, pos)
            b.set_state(tok, pos)
            a.replay(1)
            a.synchronize()
            b.decode_step(batch)
            np.testing.assert_array_equal(a.logits(batch).to_numpy(), b.logits(batch).to_numpy())


@gpu
def test_sampling_inside_the_step(models):
    cfg, W, model = models("mixed", "bfloat16")
    e = model.build_engine(max_seq_len=80, max_batch=1)
    p = tokens(cfg, 9, 3)
    a, b = (e.generate(p, 20, temperature=0.9, top_k=20, top_p=0.95, seed=4) for _ in range(2))
    c = e.generate(p, 20, temperature=0.9, top_k=20, top_p=0.95, seed=5)
    assert a == b and a != c and len(a) == 29 and all(0 <= x < cfg["vocab"] for x in a)
    assert e.generate(p, 6, temperature=0) == e.generate_greedy(p, 6)


@gpu
def test_positions_that_cannot_go_on_are_refused(models):
    cfg, W, model = models("mixed", "float32")
    e = model.build_engine(max_seq_len=100, max_batch=1)
    t, want = reference("mixed", 90)
    e.prefill(t[:60], want_last_logits=False)
    with pytest.raises(RuntimeError, match="holds 60 positions"):
        e.set_state([t[61]], [61])
    with pytest.raises(RuntimeError, match="recurrent state cannot go back"):
        e.prefill(t[59:60], start_pos=59)
    e.set_state([t[60]], [60])                                 # going on is fine, and so is starting again
    e.decode_step()
    assert near(e.logits(1).to_numpy(), want[60:61], "float32")
    assert near(e.prefill(t[:20])[None], want[19:20], "float32")
    for bad in (lambda: e.prefill([cfg["vocab"]]), lambda: e.prefill(t[:1], seq=1), lambda: e.prefill_batch([t + [0] * 20], [0], [0]), lambda: e.prefill_batch([t[:2], t[:2]], [0, 0])):
        with pytest.raises(RuntimeError):
            bad()


@gpu
def test_loader_checks_shapes(tmp_path):
    from pygpukit_amd.llm import load_model_from_safetensors, load_ratasun_from_safetensors

    cfg, W = CONFIGS["mixed"], weights("mixed")
    folder = save(tmp_path, cfg, W)
    m = load_ratasun_from_safetensors(os.path.join(folder, "model.safetensors"), dtype="float32")
    assert m.config.loop.times == 2 and m.blocks[0].mlp.num_experts == 10 and m.blocks[2].mlp is None and m.blocks[1].attn.head_dim == 24
    for layer, key, value, tensor in ((1, "conv", 5, "l1.mix.q.conv"), (2, "vdim", 21, "l2.mix.in"), (0, "kv_rank", 51, "l0.mix.dkv"), (3, "dim", 20, "l3.mix.q")):
        other = json.loads(json.dumps(cfg))
        other["layers"][layer]["mixer"][key] = value
        save(tmp_path, other, W)
        with pytest.raises(ValueError, match=tensor.replace(".", r"\.")):
            load_model_from_safetensors(folder)
    for missing in ("l0.mlp.e9.down", "l1.mlp.correction", "loop.step", "l1.mix.a1"):
        save(tmp_path, cfg, {k: v for k, v in W.items() if k != missing})
        with pytest.raises(ValueError, match=missing.replace(".", r"\.")):
            load_model_from_safetensors(folder)


@gpu
def test_trace_runner_and_command_line(models, tmp_path, capsys):
    cfg, W, model = models("mixed", "float32")
    folder = _models["mixed", "float32"][3]
    t, want = reference("mixed", 90)
    t2, want2 = reference("mixed", 30, seed=6)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:70], "want": [0, 69]}, {"id": "y", "tokens": t2[:28], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": [t[70]], "want": [0]}, {"id": "y", "tokens": [t2[28]], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": [t[71]], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "z", "tokens": t2[:5], "want": [4]}], "end": ["z"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.split("\n")[:4] == ["done 0", "done 1", "done 2", "done 3"]
    got = [np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"]) for i in (0, 1, 3)]
    assert near(got[0], want[[0, 69]], "float32") and near(got[1], np.stack([want[70], want2[28]]), "float32")
    assert near(got[2], want2[4:5], "float32") and not (tmp_path / "2.f32").exists()
    from pygpukit_amd.llm.__main__ import main

    assert main(["generate", "--model", folder, "--dtype", "float32", "--tokens", "3,4,5", "--tokens", "9", "--max-new-tokens", "6"]) == 0
    lines = [[int(x) for x in l.split(",")] for l in capsys.readouterr().out.strip().split("\n")]
    assert lines[0][:3] == [3, 4, 5] and len(lines[0]) == 9 and lines[1] == R.greedy([9], 6, cfg, W)
