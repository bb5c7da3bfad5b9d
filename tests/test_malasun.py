"""Malasun (layer-list decoder without norms ahead of its sublayers: window attention with taps over time, norms over whole projections,
distance bias, elementwise gate and keys shared between layers; gated linear recurrence; xIELU) against the plain NumPy restatement in
oracle/malasun_ref.py.

Weights are random with scores made sharp (large norm weights of q and k) and gates between almost closed and almost open, so that one
key too many or too few in a window, a stale cache row or a lost state moves the logits by far more than the tolerances;
test_weights_tell_mechanisms_apart asserts that on the CPU."""

from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests.layer_list import FakeEngine, bf16, dev, host, logit_err, rounded, save, tokens
from oracle import malasun_ref as R

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
gpu = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 5e-2}       # rms over the vocabulary of the logit difference / rms of the logits


def attn(heads, kv_heads, dim, vdim, window, scale, conv=4, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window}, "conv": conv}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def hgrn2(heads, dim, vdim):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def config(width, vocab, layers, eps=1e-5):
    return {"architecture": "Malasun", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "layers": [dict(m, mlp=None if ff is None else {"kind": "dense", "ff": ff}) for m, ff in layers]}


CONFIGS = {
    # every layer different, no width a multiple of 16; a taker with a larger window than its source's and one with a smaller; a window of
    # one; layers of both kinds with and without feed-forward
    "mixed": config(90, 211, [(attn(6, 2, 24, 40, 7, 0.4), 150), (hgrn2(2, 24, 40), 90), (attn(6, 2, 24, 40, 33, 0.3, kv_from=0), None), (hgrn2(3, 40, 20), None),
                              (attn(4, 1, 20, 12, 1, 0.5, conv=2), None), (attn(4, 1, 20, 12, 1, 0.4, conv=3, kv_from=4), 70),
                              (attn(6, 2, 24, 40, 5, 0.3, conv=2, kv_from=0), 33)], 1e-6),
    # one head, one tap, windows beyond every sequence, a recurrence first and last
    "odd": config(70, 97, [(hgrn2(1, 10, 6), 33), (attn(1, 1, 18, 22, 500, 0.5, conv=1), None), (attn(3, 3, 18, 10, 12, 0.8, conv=6), 50), (hgrn2(5, 18, 34), 20)], 1e-3),
    # head widths past each width class of the decode kernels; states that take chunks of 32 rows and several column tiles per wave
    "wide": config(192, 130, [(attn(4, 2, 144, 72, 20, 0.15), 128), (hgrn2(1, 144, 272), None), (attn(2, 1, 136, 300, 70, 0.12, conv=3), None), (hgrn2(2, 256, 64), 100),
                              (attn(2, 1, 136, 300, 9, 0.2, kv_from=2), 64)]),
    # widths the engine takes without padding, 16 and 20 heads over one or two key heads, windows around the 64-key tiles
    "tiles": config(128, 256, [(attn(16, 2, 64, 64, 65, 0.3), 256), (hgrn2(4, 64, 128), None), (attn(20, 1, 128, 128, 64, 0.2, conv=3), 192), (hgrn2(2, 128, 128), 128),
                               (attn(20, 1, 128, 128, 127, 0.1, kv_from=2), None), (attn(4, 4, 64, 48, 63, 0.3), 64)]),
    # long rows: every preload depth of the one-row projection, split-K slabs
    "long": config(1100, 120, [(attn(2, 1, 30, 30, 50, 0.3), 4200), (hgrn2(3, 32, 48), 2100)]),
    # windows of several hundred: several key tiles per split
    "deep": config(64, 90, [(attn(8, 2, 32, 64, 600, 0.3), 64), (hgrn2(2, 16, 48), None), (attn(33, 3, 16, 48, 1000, 0.4), None), (attn(8, 2, 32, 64, 300, 0.3, kv_from=0), 48)]),
}


def weights(cfg, seed=0, sharp=2.5):
    rng = np.random.default_rng(seed)

    def draw(*shape, std):
        return rng.standard_normal(shape) * std

    H, W = cfg["width"], {}
    W["embed"] = draw(cfg["vocab"], H, std=1.0)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        n, d, v = m["heads"], m["dim"], m["vdim"]
        lin = lambda rows: draw(rows, H, std=1 / np.sqrt(H))  # noqa: E731
        W[p + "norm1"] = np.float64(rng.uniform(0.6, 1.4))
        if l["type"] == "hgrn2":
            W[p + "mix.q"], W[p + "mix.f"], W[p + "mix.v"] = lin(n * d), lin(n * d), lin(n * v)
            W[p + "mix.f.b"], W[p + "mix.lower"] = rng.uniform(-3, 9, n * d), rng.uniform(0, 0.9, n * d) * (rng.random(n * d) < 0.7)
            W[p + "mix.norm"] = draw(v, std=0.3) + 1.0
        else:
            s = (sharp / (m["scale"] * np.sqrt(d))) ** 0.5                       # scores of standard deviation `sharp`
            g = m["kv_heads"]
            for name, rows in (("q", n * d),) + ((("k", g * d), ("v", g * v)) if m.get("kv_from") is None else ()):
                W[p + f"mix.{name}"], W[p + f"mix.{name}.b"] = lin(rows), draw(rows, std=0.3)
                W[p + f"mix.{name}.conv"] = draw(rows, m["conv"], std=0.6)
                if name != "v":
                    W[p + f"mix.{name}.norm"] = s * (1.0 + draw(rows, std=0.3))
            W[p + "mix.g"] = lin(n * v)
        W[p + "mix.o"] = draw(H, n * v, std=1 / np.sqrt(n * v))
        if l["mlp"]:
            f = l["mlp"]["ff"]
            W[p + "norm2"] = np.float64(rng.uniform(0.6, 1.4))
            W[p + "mlp.up"], W[p + "mlp.down"], W[p + "mlp.act"] = lin(f), draw(H, f, std=1 / np.sqrt(f)), rng.uniform(-1, 1, 2)
    W["final.norm"], W["head"] = np.float64(rng.uniform(0.8, 1.5)), draw(cfg["vocab"], H, std=1 / np.sqrt(H))
    return {k: bf16(x) for k, x in W.items()}


# ------------------------------------------------------------------------------------------------ CPU: configuration, oracle
def test_config_is_read_layer_by_layer():
    from pygpukit_amd.llm import MALASUN_SPEC, detect_model_spec, layer_list_config
    from pygpukit_amd.llm.config import distance_slopes

    c = layer_list_config(CONFIGS["mixed"])
    assert (c.hidden_size, c.vocab_size, c.num_layers, c.norm_eps, c.residual_mult, c.activation) == (90, 211, 7, 1e-6, 1.0, "xielu")
    a, b, d = c.layers[:3]
    assert (a.mixer, a.num_heads, a.num_kv_heads, a.head_dim, a.v_head_dim, a.window, a.scale, a.conv_taps, a.kv_from, a.intermediate_size) == \
        ("attention", 6, 2, 24, 40, 7, 0.4, 4, None, 150)
    assert (b.mixer, b.num_heads, b.head_dim, b.v_head_dim, b.intermediate_size) == ("hgrn2", 2, 24, 40, 90)
    assert d.kv_from == 0 and d.window == 33 and d.intermediate_size is None
    assert detect_model_spec(["embed"], CONFIGS["mixed"]) is MALASUN_SPEC
    np.testing.assert_allclose(distance_slopes(6), R.distance_slopes(6))
    for layer, bad in ((1, {"type": "recurrent"}), (0, {"mlp": {"kind": "sparse", "ff": 4}})):
        broken = json.loads(json.dumps(CONFIGS["mixed"]))
        broken["layers"][layer].update(bad)
        with pytest.raises(ValueError, match=f"layer {layer}"):
            layer_list_config(broken)
    for layer, bad in ((0, {"kv_heads": 4}), (2, {"kv_from": 1}), (2, {"kv_from": 3}), (6, {"kv_from": 2}), (2, {"dim": 23})):
        broken = json.loads(json.dumps(CONFIGS["mixed"]))
        broken["layers"][layer]["mixer"].update(bad)
        with pytest.raises(ValueError, match=f"layer {layer}"):
            layer_list_config(broken)


def test_oracle_mechanisms_on_hand_made_numbers():
    x = np.array([[3.0, 4.0]])
    np.testing.assert_allclose(R.scalar_norm(x, np.float64(2.0), 0.0), 2 * x / np.sqrt(12.5))
    u = np.array([[1.0], [10.0], [100.0]])
    np.testing.assert_allclose(R.short_conv(u, np.array([[3.0, 2.0]]))[:, 0], [2.0, 23.0, 230.0])
    np.testing.assert_allclose(R.short_conv(u[:1], np.array([[5.0, 4.0, 3.0, 2.0]]))[:, 0], [2.0])
    np.testing.assert_allclose(R.distance_slopes(4), [0.25, 0.0625, 2.0**-6, 2.0**-8])
    v = np.arange(5.0)[:, None, None]
    got = R.attend(np.zeros((5, 1, 2)), np.zeros((5, 1, 2)), v, 1.0, 3, np.array([np.log(2.0)]))[4, 0, 0]
    np.testing.assert_allclose(got, (4 + 3 / 2 + 2 / 4) / 1.75)                                    # weights 1, 1/2, 1/4 by distance
    z = np.array([-700.0, -1.0, 0.0, 2.0])
    p, q = np.log1p(np.exp(0.3)), np.log1p(np.exp(-0.2))
    np.testing.assert_allclose(R.xielu(z, 0.3, -0.2), [(0.5 + q) * 699 - 350, (0.5 + q) * np.exp(-1) - 0.5, 0.0, 4 * p + 1])
    o, S = R.gated_recurrence(np.ones((3, 1, 1)), np.full((3, 1, 1), 0.75), np.array([8.0, 0.0, 4.0]).reshape(3, 1, 1))
    np.testing.assert_allclose(o[:, 0, 0], [2.0, 1.5, 2.125])
    o2, S2 = R.gated_recurrence(np.ones((1, 1, 1)), np.full((1, 1, 1), 0.5), np.zeros((1, 1, 1)), S)
    np.testing.assert_allclose((o2[0, 0, 0], S2[0, 0, 0]), (1.0625, 1.0625))
    np.testing.assert_allclose(R.forget_gate(np.array([-90.0, 90.0, 1.0]), np.array([0.0, 0.0, -1.0]), np.array([0.25, 0.25, 0.5])), [0.25, 1.0, 0.75])


@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_weights_tell_mechanisms_apart(name):
    """A window one key off, another source of keys, a missing bias, tap, gate, lower bound or norm: each moves the logits by hundreds of
    times the fp32 tolerance."""
    cfg, t = CONFIGS[name], tokens(CONFIGS[name], 140, 3)
    W = weights(cfg)
    want = R.forward(t, cfg, W)

    def moved(c, w):
        return logit_err(R.forward(t, c, w), want) > 300 * TOL["float32"]

    for i, l in enumerate(cfg["layers"]):
        w = dict(W)
        p = f"l{i}.mix."
        if l["type"] == "hgrn2":
            for key in ("f.b", "lower"):
                assert moved(cfg, {**w, p + key: np.zeros_like(W[p + key])}), (i, key)
            assert moved(cfg, {**w, p + "norm": np.ones_like(W[p + "norm"])}), i
            continue
        for delta in (-1, 1):
            other = json.loads(json.dumps(cfg))
            other["layers"][i]["mixer"]["mask"]["size"] += delta
            if other["layers"][i]["mixer"]["mask"]["size"] >= 1:
                assert moved(other, W), (i, delta)
        for key in ("q.b", "q.norm", "q.conv", "g"):
            if l["mixer"]["mask"]["size"] > 1 or key == "g":
                assert moved(cfg, {**w, p + key: np.zeros_like(W[p + key]) if key in ("q.b", "g") else np.roll(W[p + key], 1, axis=-1)}), (i, key)


def test_scheduler_drives_one_batch_at_a_time():
    """All sequences start in one ragged prompt call, then go on together by one token; shorter ones end earlier."""
    from pygpukit_amd.llm.scheduler import BatchScheduler

    e = FakeEngine(max_batch=4)
    s = BatchScheduler(e)
    s.step([("a", [1, 2, 3], []), ("b", [4], [0]), ("c", [5, 6], [1])])
    assert e.calls == [("prefill", [0, 1, 2], [0, 0, 0], [3, 1, 2])]
    s.step([("a", [7], [0]), ("b", [8], [0]), ("c", [9], [0])])
    s.release("b")
    s.step([("a", [7], [0]), ("c", [9], [0])])                             # the free slot in the middle takes a dummy row at position 0
    assert e.calls[1:] == [("decode", 3), ("decode", 3)] and e.state[1] == (1, 0, 0)


# ------------------------------------------------------------------------------------------------ GPU: operators
OP_TOL = {"float32": 3e-6, "bfloat16": 1.5e-2}
both = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def worst(got, want):
    return float(np.max(np.abs(got - want)) / np.max(np.abs(want)))


@gpu
@both
def test_activation_gate_and_taps(dtype):
    from pygpukit_amd.ops.basic import short_conv, sigmoid_mul, xielu

    rng = np.random.default_rng(1)
    z = rounded(np.concatenate([rng.standard_normal(1000) * 4, rng.standard_normal(1000) * 1e-3, [0.0, -60.0, 30.0]]), dtype)
    p, q = 0.37, -1.2
    got = host(xielu(dev(z, dtype), R.softplus(p), 0.5 + R.softplus(q)))
    want = R.xielu(z.astype(np.float64), p, q)
    assert np.max(np.abs(got - want) / np.maximum(np.maximum(np.abs(want), np.abs(z)), 1e-3)) < OP_TOL[dtype]      # (it crosses zero at some z < 0)
    x, g = rounded(rng.standard_normal((7, 33)), dtype), rounded(rng.standard_normal((7, 33)) * 4, dtype)
    assert worst(host(sigmoid_mul(dev(x, dtype), dev(g, dtype))), x * R.sigmoid(g.astype(np.float64))) < OP_TOL[dtype]
    for taps in (1, 2, 4, 7):
        u, w = rounded(rng.standard_normal((20, 11)), dtype), rounded(rng.standard_normal((11, taps)), dtype)
        want = R.short_conv(u.astype(np.float64), w.astype(np.float64))
        assert worst(host(short_conv(dev(u, dtype), dev(w, dtype))), want) < OP_TOL[dtype]
        if taps > 1:
            for cut in (taps - 1, 13):
                got = host(short_conv(dev(u[cut:], dtype), dev(w, dtype), dev(u[cut - taps + 1:cut], dtype)))
                assert worst(got, want[cut:]) < OP_TOL[dtype]


@gpu
@both
@pytest.mark.parametrize("heads,kv_heads,dk,dv", [(2, 1, 64, 64), (6, 2, 128, 128), (5, 5, 20, 36), (4, 2, 200, 64)])
@pytest.mark.parametrize("q_len,kv_len,window", [(1, 1, 1), (5, 5, 2), (130, 130, 1), (200, 333, 64), (70, 300, 65), (129, 257, 63), (300, 300, 1000), (2, 400, 129), (90, 120, 500),
                                                 (700, 1100, 900)])
def test_window_attention_with_distance_bias(heads, kv_heads, dk, dv, q_len, kv_len, window, dtype):
    from pygpukit_amd.ops.basic import window_attention

    rng = np.random.default_rng(q_len + kv_len + window + heads)
    q, k, v, g = (rounded(rng.standard_normal(s), dtype) for s in ((q_len, heads, dk), (kv_len, kv_heads, dk), (kv_len, kv_heads, dv), (q_len, heads, dv)))
    scale, slopes = 1.5 / np.sqrt(dk), R.distance_slopes(heads)
    full = np.zeros((kv_len, heads, dk))
    full[kv_len - q_len:] = q
    want = R.attend(full, k.astype(np.float64), v.astype(np.float64), scale, window, slopes)[kv_len - q_len:]
    args = (dev(q, dtype), dev(k, dtype), dev(v, dtype), scale, window)
    sl = dev(slopes, "float32")
    assert worst(host(window_attention(*args, slopes=sl)), want) < OP_TOL[dtype]
    want = want * R.sigmoid(g.astype(np.float64))
    assert worst(host(window_attention(*args, slopes=sl, gate=dev(g, dtype))), want) < OP_TOL[dtype]


@gpu
@both
@pytest.mark.parametrize("d", [48, 64, 128])
def test_window_edges_and_distances_with_one_loud_key(d, dtype):
    """Key j is aligned with every query and its value is the only one that is not zero; the slope is so steep that its weight against
    the query's own key tells every distance apart."""
    from pygpukit_amd.ops.basic import window_attention

    n, slope = 333, 0.02
    for window in (1, 2, 63, 64, 65, 129, 200):
        for j in (0, 63, 64, 100):
            q, k, v = np.zeros((n, 1, d), np.float32), np.zeros((n, 1, d), np.float32), np.zeros((n, 1, d), np.float32)
            q[:, 0, 0], k[j, 0, 0], v[j, 0, :] = 8.0, 0.5, 1.0
            got = host(window_attention(dev(q, dtype), dev(k, dtype), dev(v, dtype), 1.0, window, slopes=dev(np.full(1, slope), "float32")))[:, 0, :]
            want = R.attend(q.astype(np.float64), k.astype(np.float64), v.astype(np.float64), 1.0, window, np.full(1, slope))[:, 0, :]
            assert np.max(np.abs(got - want)) < (1e-5 if dtype == "float32" else 1e-2)
            assert not got[:j].any() and not got[j + window:].any()


def recurrence_case(rng, n, heads, dim, vdim, dtype, extreme=False):
    q, f, v = (rounded(rng.standard_normal((n, heads * w)) * s, dtype) for w, s in ((dim, 1.5), (dim, 40.0 if extreme else 2.0), (vdim, 1.0)))
    b = (rng.uniform(-3, 9, heads * dim) if not extreme else np.zeros(heads * dim)).astype(np.float32)
    low = (rng.uniform(0, 0.9, heads * dim) * (rng.random(heads * dim) < 0.5)).astype(np.float32)
    norm = (1.0 + 0.3 * rng.standard_normal(vdim)).astype(np.float32)
    return q, f, v, b, low, norm


def recurrence_oracle(q, f, v, b, low, norm, heads, state=None, eps=1e-4):
    n = q.shape[0]
    q, f, v = (x.astype(np.float64) for x in (q, f, v))
    o, S = R.gated_recurrence((q * R.sigmoid(q)).reshape(n, heads, -1), R.forget_gate(f, b.astype(np.float64), low.astype(np.float64)).reshape(n, heads, -1),
                              v.reshape(n, heads, -1), state)
    if norm is not None:
        o = R.rms_scale(o, eps) * norm
    return o.reshape(n, -1), S


@gpu
@both
@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 128), (3, 24, 40), (1, 256, 64), (2, 16, 16), (1, 144, 272), (3, 48, 512), (2, 10, 6), (1, 128, 128)])
def test_gated_recurrence(heads, dim, vdim, dtype):
    """Every form (chunks of 64 and 32 rows, token by token), lengths around its blocks; portions continue the state."""
    from pygpukit_amd.ops.basic import gated_recurrence

    rng = np.random.default_rng(dim + vdim)
    case = recurrence_case(rng, 330, heads, dim, vdim, dtype)
    q, f, v, b, low, norm = case
    want, _ = recurrence_oracle(*case, heads)
    tol = OP_TOL[dtype] if dtype == "bfloat16" else 5e-6
    for cuts in ([330], [1, 2, 15, 16, 17, 64, 65, 150], [63, 32, 31, 204]):
        state = dev(rng.standard_normal((heads, dim, vdim)), "float32")         # fresh: what is in it does not matter
        at = 0
        for c in cuts:
            got = host(gated_recurrence(dev(q[at:at + c], dtype), dev(f[at:at + c], dtype), dev(v[at:at + c], dtype), dev(low, "float32"), state, f_bias=dev(b, "float32"),
                                        norm=dev(norm, "float32"), eps=1e-4, fresh=at == 0))
            assert worst(got, want[at:at + c]) < tol, (cuts, at)
            at += c
            _, S = recurrence_oracle(q[:at], f[:at], v[:at], b, low, norm, heads)
            assert worst(host(state), S) < 5e-6, (cuts, at)
    plain = host(gated_recurrence(dev(q, dtype), dev(f, dtype), dev(v, dtype), dev(low, "float32"), dev(np.zeros((heads, dim, vdim)), "float32")))
    assert worst(plain, recurrence_oracle(q, f, v, 0 * b, low, None, heads)[0]) < tol


@gpu
@both
def test_gates_that_close_and_open_completely(dtype):
    """Gate arguments of tens in both directions: decays down to e^-100 per row beside decays of 1, in every block of a chunk."""
    from pygpukit_amd.ops.basic import gated_recurrence

    rng = np.random.default_rng(8)
    case = recurrence_case(rng, 200, 2, 32, 48, dtype, extreme=True)
    q, f, v, b, low, norm = case
    want, S = recurrence_oracle(*case, 2)
    state = dev(np.zeros((2, 32, 48)), "float32")
    got = host(gated_recurrence(dev(q, dtype), dev(f, dtype), dev(v, dtype), dev(low, "float32"), state, norm=dev(norm, "float32"), eps=1e-4))
    assert np.isfinite(got).all() and worst(got, want) < (OP_TOL[dtype] if dtype == "bfloat16" else 2e-5) and worst(host(state), S) < 1e-5


@gpu
def test_a_write_far_back_is_still_there():
    """One written row, gates of almost 1 after it: hundreds of rows later the state holds it at its decayed size."""
    from pygpukit_amd.ops.basic import gated_recurrence

    n, z = 700, 7.0
    q, f, v = np.full((n, 16), 2.0, np.float32), np.full((n, 16), z, np.float32), np.zeros((n, 16), np.float32)
    v[3], f[3] = 1000.0, 0.0
    want, S = recurrence_oracle(q, f, v, np.zeros(16, np.float32), np.zeros(16, np.float32), None, 1)
    state = dev(np.zeros((1, 16, 16)), "float32")
    got = host(gated_recurrence(dev(q, "float32"), dev(f, "float32"), dev(v, "float32"), dev(np.zeros(16), "float32"), state))
    assert want[-1].min() > 1.0 and np.max(np.abs(got[4:] / want[4:] - 1)) < 1e-4 and worst(host(state), S) < 1e-4      # 700 times the rounding of one gate


# ------------------------------------------------------------------------------------------------ GPU: model and engine
_models: dict = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """(config, weights, model) by name and dtype, loaded from a checkpoint on disk by the product loader."""
    from pygpukit_amd.llm import load_model_from_safetensors

    def get(name, dtype):
        if (name, dtype) not in _models:
            cfg = CONFIGS[name]
            W = weights(cfg)
            folder = save(tmp_path_factory.mktemp(name), cfg, W)
            _models[name, dtype] = (cfg, W, load_model_from_safetensors(folder, dtype=dtype), folder)
        return _models[name, dtype][:3]

    yield get
    _models.clear()


_ref: dict = {}


def reference(name, n, seed=5):
    if (name, n, seed) not in _ref:
        t = tokens(CONFIGS[name], n, seed)
        _ref[name, n, seed] = (t, R.forward(t, CONFIGS[name], weights(CONFIGS[name])))
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
    assert logit_err(np.concatenate(got), want) < TOL[dtype]


@gpu
@both
def test_fixed_cache_strategies(models, dtype):
    from pygpukit_amd.llm import DecodeBatch, DecodeBuffers, DecodeM1

    cfg, W, model = models("mixed", dtype)
    t, want = reference("mixed", 90)
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
    assert logit_err(np.concatenate(got), want[:64]) < TOL[dtype]
    model.restore_kv_cache(saved)
    assert logit_err(host(mb.step_batch(t[55:60], 55, 60)), want[55:60]) < TOL[dtype]
    assert logit_err(host(mb.step_batch(t[:5], 0, 5)), want[:5]) < TOL[dtype]       # position 0 starts again


@gpu
@both
@every
def test_engine_prompt_every_row(models, name, dtype):
    cfg, W, model = models(name, dtype)
    n = {"tiles": 400, "deep": 700}.get(name, 150)
    t, want = reference(name, n)
    e = model.build_engine(max_seq_len=n, max_batch=2)
    got = e.prefill_batch([t], [1], want=[list(range(n))])
    assert got.shape == want.shape and logit_err(got, want) < TOL[dtype]
    for k in (1, 2, 3, 4, 17):                                 # the first tokens of a sequence as whole prompts
        assert logit_err(e.prefill(t[:k], seq=0)[None], want[k - 1:k]) < TOL[dtype]


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
    err = 0.0
    for i in range(n - max(lag)):
        e.set_state([t[p + i] for p in lag], [p + i for p in lag])
        e.decode_step(batch)
        err = max(err, logit_err(e.logits(batch).to_numpy(), want[[p + i for p in lag]]))
    assert err < TOL[dtype]


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
    assert logit_err(np.concatenate(got), want[:n]) < TOL[dtype]


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
            assert logit_err(o, ref[i][1][[lens[i] - 1, 0]]) < TOL[dtype]
        live = list(order)
        for k in range(12):
            out = s.step([((again, i), [ref[i][0][lens[i] + k]], [0]) for i in live])
            for i, o in zip(live, out):
                assert logit_err(o, ref[i][1][[lens[i] + k]]) < TOL[dtype]
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
def test_deep_windows_in_batches(models, dtype, batch):
    """Sequences around and beyond a 600-key window, in batch sizes that give one split and several."""
    cfg, W, model = models("deep", dtype)
    n = 700
    t, want = reference("deep", n)
    e = model.build_engine(max_seq_len=720, max_batch=batch)
    at = [(590 + 13 * b) % 690 + 1 if b < 8 else 1 + (37 * b) % 680 for b in range(batch)]
    e.prefill_batch([t[:p] for p in at], want=[[]] * batch)
    err = 0.0
    for i in range(6):
        e.set_state([t[p + i] for p in at], [p + i for p in at])
        e.decode_step(batch)
        err = max(err, logit_err(e.logits(batch).to_numpy(), want[[p + i for p in at]]))
    assert err < TOL[dtype]


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
        assert logit_err(e.prefill_batch([t[:n]], want=[[0, n // 2, n - 1]]), want[[0, n // 2, n - 1]]) < TOL["bfloat16"]
    at = [3 * b + 1 for b in range(12)]
    e.prefill_batch([t[:p] for p in at], want=[[]] * 12)
    e.set_state([t[p] for p in at], at)
    e.decode_step(12)
    assert logit_err(e.logits(12).to_numpy(), want[at]) < TOL["bfloat16"]


@gpu
@both
def test_long_decoding_past_every_window(models, dtype):
    """Far more decoded tokens than any ring has rows; the same logits from the captured graph."""
    cfg, W, model = models("tiles", dtype)
    t, want = reference("tiles", 400)
    e = model.build_engine(max_seq_len=450, max_batch=2)
    e.prefill(t[:3], seq=0, want_last_logits=False)
    e.prefill(t[:100], seq=1, want_last_logits=False)
    e.capture(2)
    err = 0.0
    for i in range(300):
        e.set_state([t[3 + i], t[100 + i]], [3 + i, 100 + i])
        if i % 3:
            e.replay(1)
        else:
            e.decode_step(2)
        if i % 7 == 0 or i > 290 or 58 <= i <= 66 or 121 <= i <= 128:
            err = max(err, logit_err(e.logits(2).to_numpy(), want[[3 + i, 100 + i]]))
    assert err < TOL[dtype]
    assert e.recurrent_state(1).shape == (2, 4, 64, 128)
    with pytest.raises(ValueError):
        e.recurrent_state(0)


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
def test_graph_replays_equal_eager_steps(models):
    """Several replays with eager work and synchronisation between them: each equals the eager step from the same state."""
    cfg, W, model = models("tiles", "bfloat16")
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
    for pos in (50, 59):
        with pytest.raises(RuntimeError, match="no longer in its ring" if pos == 50 else "recurrent state cannot go back"):
            e.prefill(t[pos:60], start_pos=pos)
    e.set_state([t[60]], [60])                                 # going on is fine, and so is starting again
    e.decode_step()
    assert logit_err(e.logits(1).to_numpy(), want[60:61]) < TOL["float32"]
    assert logit_err(e.prefill(t[:20])[None], want[19:20]) < TOL["float32"]
    for bad in (lambda: e.prefill([cfg["vocab"]]), lambda: e.prefill(t[:1], seq=1), lambda: e.prefill_batch([t[:101 - 0] + [0] * 20], [0], [0]),
                lambda: e.prefill_batch([t[:2], t[:2]], [0, 0])):
        with pytest.raises(RuntimeError):
            bad()


@gpu
def test_loader_checks_shapes(tmp_path):
    from pygpukit_amd.llm import load_malasun_from_safetensors, load_model_from_safetensors

    cfg, W = CONFIGS["mixed"], weights(CONFIGS["mixed"])
    folder = save(tmp_path, cfg, W)
    m = load_malasun_from_safetensors(os.path.join(folder, "model.safetensors"), dtype="float32")
    assert m.config.layers[5].conv_taps == 3 and m.blocks[2].attn.source is m.blocks[0].attn and m.blocks[1].attn.head_dim == 24
    for layer, key, value, name in ((0, "conv", 5, "l0.mix.q.conv"), (1, "vdim", 41, "l1.mix.v"), (2, "dim", 24, "l2.mix.q.norm")):
        other = json.loads(json.dumps(cfg))
        other["layers"][layer]["mixer"][key] = value
        save(tmp_path, other, {**W, "l2.mix.q.norm": W["l2.mix.q.norm"][:-1]} if layer == 2 else W)
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            load_model_from_safetensors(folder)
    save(tmp_path, cfg, {k: v for k, v in W.items() if k != "l3.mix.lower"})
    with pytest.raises(ValueError, match="l3.mix.lower"):
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
    assert logit_err(got[0], want[[0, 69]]) < TOL["float32"] and logit_err(got[1], np.stack([want[70], want2[28]])) < TOL["float32"]
    assert logit_err(got[2], want2[4:5]) < TOL["float32"] and not (tmp_path / "2.f32").exists()
    from pygpukit_amd.llm.__main__ import main

    assert main(["generate", "--model", folder, "--dtype", "float32", "--tokens", "3,4,5", "--tokens", "9", "--max-new-tokens", "6"]) == 0
    lines = [[int(x) for x in l.split(",")] for l in capsys.readouterr().out.strip().split("\n")]
    assert lines[0][:3] == [3, 4, 5] and len(lines[0]) == 9 and lines[1] == R.greedy([9], 6, cfg, W)
