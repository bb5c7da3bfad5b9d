"""Fetezen (layer-list decoder with hyper-connected residual streams, attention whose heads mix their scores, with sinks and in chunks of
positions, polynomial-norm feed-forwards and experts that a table of tokens chooses) against the plain NumPy restatement in
oracle/fetezen_ref.py.

Weights are random with sharp attention scores, so that a lost key, a stale cache row or a sink that is left out moves the logits by far
more than the tolerances; test_weights_tell_mechanisms_apart asserts that on the CPU."""

from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests.layer_list import FakeEngine, bf16, dev, host, logit_err, rounded, save, tokens
from oracle import fetezen_ref as R

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
gpu = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 5e-2}       # rms over the vocabulary of the logit difference / rms of the logits
ROUGH = 0.25                                    # bfloat16, for single rows: a sharp choice between two keys turns rounding into a step


def near(got, want, dtype, positions=0):
    """fp32: every row is within the tolerance (an fp32 angle at position p is p / 2^24 off, and sharp scores pass it on); bfloat16: all rows but one, or one in fifty, are, and those are within ROUGH."""
    d = np.asarray(got, np.float64) - want
    err = np.sqrt(np.mean(d * d, axis=-1)) / np.sqrt(np.mean(want * want))
    if dtype == "float32":
        return bool(np.all(err < TOL[dtype] + positions * 4e-8))
    return bool(np.all(err < ROUGH)) and int(np.sum(err > TOL[dtype])) <= max(1, err.size // 50)


def attn(heads, kv_heads, dim, vdim, rot, chunk, scale=0.2, base=10000.0, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": rot}, "mask": None if chunk is None else {"size": chunk}}
    return {"type": "attention", "mixer": m if kv_from is None else dict(m, kv_from=kv_from)}


def poly(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    e = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    return e if shared is None else dict(e, shared={"ff": shared})


def config(width, vocab, layers, streams, groups, eps=1e-5, cap=None):
    c = {"architecture": "Fetezen", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps, "groups": groups}, "layers": [dict(m, mlp=e) for m, e in layers]}
    return c if cap is None else dict(c, logit_softcap=cap)


CONFIGS = {
    # every layer different, no width a multiple of 16, takers with larger and smaller chunks than their source's, a layer without a mask
    "mixed": config(90, 211, [(attn(6, 2, 24, 40, 10, 33), poly(50)), (attn(6, 2, 24, 40, 10, 70, 0.3, kv_from=0), moe(10, 3, 50, 33)), (attn(6, 2, 24, 40, 10, 7, kv_from=0), None),
                              (attn(5, 5, 18, 22, 18, 16, 0.5, 500.0), moe(9, 2, 33)), (attn(4, 1, 30, 10, 4, None), poly(70)), (attn(4, 1, 30, 10, 4, 21, kv_from=4), moe(6, 6, 70, 130)),
                              (attn(3, 3, 14, 30, 2, 64, 0.1, 50.0), None)], 3, 5, 1e-4, 2.5),
    # one stream, one head, a chunk of one position, one expert; norm groups of an odd size
    "odd": config(70, 97, [(attn(1, 1, 7, 9, 2, 1, 1.0), moe(1, 1, 20, 10)), (attn(1, 1, 9, 7, 6, 5, 0.5, 100.0), poly(30)), (attn(3, 1, 10, 6, 0, 12), moe(4, 4, 10))], 1, 14, 1e-3, 0.7),
    # head widths past each width class of the kernels
    "wide": config(192, 130, [(attn(2, 1, 144, 72, 100, 60, 0.1), moe(16, 3, 64, 200)), (attn(2, 2, 200, 272, 200, 45), None), (attn(6, 3, 128, 100, 64, 80, 0.1), poly(500)),
                              (attn(1, 1, 520, 30, 32, 90), moe(5, 2, 128, 64))], 2, 1),
    # widths the engine takes without padding, every width of the matrix kernels
    "tiles": config(128, 256, [(attn(16, 4, 64, 64, 64, 64, 0.15), moe(16, 4, 64, 128)), (attn(8, 8, 128, 128, 128, 128, 0.1), poly(256)), (attn(20, 4, 96, 128, 64, 100, 0.1), moe(16, 2, 128, 64)),
                               (attn(32, 8, 64, 64, 32, 150, 0.15), poly(128)), (attn(32, 8, 64, 64, 32, 40, kv_from=3), moe(8, 1, 64)), (attn(12, 2, 128, 64, 16, 90), None)], 4, 8, cap=3.0),
    # long rows, wide feed-forwards
    "long": config(1100, 120, [(attn(2, 2, 30, 20, 30, 50), moe(6, 2, 1400, 300)), (attn(3, 1, 32, 48, 20, 70), poly(5000)), (attn(3, 1, 32, 48, 20, 30, kv_from=1), moe(4, 2, 300, 1400))], 2, 4),
    # many heads and streams; near one-hot attention over hundreds of keys
    "deep": config(64, 90, [(attn(8, 4, 64, 64, 32, 300), moe(96, 6, 32, 40)), (attn(33, 3, 16, 48, 8, 350), None), (attn(24, 8, 64, 64, 64, 256), poly(90)), (attn(24, 8, 64, 64, 64, 500, kv_from=2), None)],
                   6, 2, cap=2.0),
    # numbers of key heads and widths for every shape of the decode kernel, and past them
    "heads": config(96, 110, [(attn(12, 12, 64, 64, 64, 48), None), (attn(16, 16, 128, 100, 32, 70), poly(64)), (attn(5, 5, 144, 180, 100, 40), None), (attn(8, 8, 200, 256, 200, 90), None),
                              (attn(18, 18, 40, 64, 20, 30), None), (attn(24, 1, 64, 64, 64, 64), None), (attn(40, 4, 64, 64, 8, 77), moe(5, 2, 64)), (attn(9, 3, 192, 150, 64, 100), None)], 2, 3),
    # one layer of near one-hot attention: what lies outside a chunk moves nothing
    "edge37": config(64, 40, [(attn(8, 2, 64, 64, 32, 37), None)], 2, 2),
    "edge64": config(64, 40, [(attn(6, 6, 48, 40, 32, 64), None)], 2, 2),
}
SHARP = {"deep": 6.0, "edge37": 6.0, "edge64": 6.0}


def weights(name, seed=0):
    cfg, sharp = CONFIGS[name], SHARP.get(name, 2.5)
    rng = np.random.default_rng(seed)

    def draw(*shape, std):
        return rng.standard_normal(shape) * std

    H, S, V, W = cfg["width"], cfg["streams"], cfg["vocab"], {}
    into = lambda rows, cols: draw(rows, cols, std=0.6 / np.sqrt(cols))  # noqa: E731
    lin = lambda rows: draw(rows, H, std=1 / np.sqrt(H))  # noqa: E731
    W["embed"] = draw(V, H, std=1.0)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        n, g, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for q in (1, 2) if l["mlp"] else (1,):
            W[p + f"norm{q}"] = 1.0 + draw(H, std=0.2)
            W[p + f"hc{q}.in"], W[p + f"hc{q}.out"] = 1 / S + draw(S, std=0.3), 1.0 + draw(S, std=0.3)
            W[p + f"hc{q}.mix"] = 0.7 * np.eye(S) + draw(S, S, std=0.3 / np.sqrt(S))
        W[p + "mix.q"], W[p + "mix.q.b"] = lin(n * d), draw(n * d, std=0.5)
        W[p + "mix.q.norm"] = (1.0 + draw(d, std=0.2)) * sharp / (m["scale"] * np.sqrt(d))             # scores of standard deviation `sharp`
        if m.get("kv_from") is None:
            for x, rows in (("k", g * d), ("v", g * v)):
                W[p + f"mix.{x}"], W[p + f"mix.{x}.b"] = lin(rows), draw(rows, std=0.5)
            W[p + "mix.k.norm"] = 1.0 + draw(d, std=0.2)
        W[p + "mix.talk"], W[p + "mix.sink"] = np.eye(n) + draw(n, n, std=0.5 / np.sqrt(n)), rng.uniform(0.0, 2.0 * sharp, n)
        W[p + "mix.o"], W[p + "mix.o.b"] = into(H, n * v), draw(H, std=0.2)
        if not l["mlp"]:
            continue
        if l["mlp"]["kind"] == "dense":
            f = l["mlp"]["ff"]
            W[p + "mlp.up"], W[p + "mlp.down"], W[p + "mlp.act"] = lin(f), into(H, f), rng.uniform(0.3, 0.9, 4)
            continue
        f, r = l["mlp"]["expert"]["ff"], l["mlp"]["router"]
        for e in range(r["experts"]):
            W[p + f"mlp.e{e}.up"], W[p + f"mlp.e{e}.down"] = 2 * lin(f), 2 * into(H, f)
        W[p + "mlp.table"] = np.stack([rng.permutation(r["experts"])[:r["top"]] for _ in range(V)]).astype(np.int32)
        if l["mlp"].get("shared"):
            f = l["mlp"]["shared"]["ff"]
            W[p + "mlp.shared.up"], W[p + "mlp.shared.down"], W[p + "mlp.shared.sg"] = 2 * lin(f), 2 * into(H, f), 2 * lin(1)
    W["final.norm"], W["head"] = 1.0 + draw(H, std=0.2), draw(V, H, std=1 / np.sqrt(H))
    return {k: x if k.endswith(".table") else bf16(x) for k, x in W.items()}


# ------------------------------------------------------------------------------------------------ CPU: configuration, oracle
def test_config_is_read_layer_by_layer():
    from pygpukit_amd.llm import FETEZEN_SPEC, detect_model_spec, layer_list_config

    c = layer_list_config(CONFIGS["mixed"])
    assert (c.hidden_size, c.vocab_size, c.num_layers, c.norm_eps, c.norm_groups, c.streams, c.logit_softcap, c.norm_type) == (90, 211, 7, 1e-4, 5, 3, 2.5, "rmsnorm")
    a, b, d, e, f = c.layers[:5]
    assert (a.mixer, a.num_heads, a.num_kv_heads, a.head_dim, a.v_head_dim, a.rot_dim, a.rot_base, a.scale, a.window, a.chunked, a.kv_from, a.intermediate_size, a.experts) == \
        ("attention", 6, 2, 24, 40, 10, 10000.0, 0.2, 33, True, None, 50, None)
    assert (b.kv_from, b.window, b.scale, b.intermediate_size, b.experts.count, b.experts.top, b.experts.table, b.experts.shared_size) == (0, 70, 0.3, 50, 10, 3, True, 33)
    assert d.intermediate_size is None and (e.rot_base, e.experts.shared_size) == (500.0, None) and (f.window, f.chunked) == (None, False)
    assert detect_model_spec(["embed"], CONFIGS["mixed"]) is FETEZEN_SPEC
    odd = layer_list_config(CONFIGS["odd"])
    assert (odd.streams, odd.norm_groups, odd.logit_softcap, odd.layers[2].rot_dim) == (1, 14, 0.7, 0) and layer_list_config(CONFIGS["wide"]).logit_softcap is None

    def broken(layer, part, **kw):
        x = json.loads(json.dumps(CONFIGS["mixed"]))
        target = x["layers"][layer]
        for key in part:
            target = target[key]
        target.update(kw)
        return x

    for layer, part, kw in ((0, ("mixer", "rot"), {"dims": 9}), (0, ("mixer", "rot"), {"dims": 26}), (0, ("mixer", "mask"), {"size": 0}), (1, ("mixer",), {"kv_heads": 3}), (2, ("mixer",), {"kv_from": 1}),
                            (1, ("mixer",), {"dim": 22}), (1, ("mixer",), {"kv_from": 3}), (1, ("mlp", "router"), {"top": 11}), (3, ("mixer",), {"kv_heads": 4}), (1, (), {"type": "gru"})):
        with pytest.raises(ValueError, match=f"layer {layer}"):
            layer_list_config(broken(layer, part, **kw))
    for kw in ({"streams": 0}, {"norm": {"eps": 1e-5, "groups": 4}}, {"logit_softcap": 0.0}):
        with pytest.raises(ValueError, match="norm groups"):
            layer_list_config({**CONFIGS["mixed"], **kw})
    with pytest.raises(ValueError, match="norm groups"):                        # the relatives have none of it
        layer_list_config({"architecture": "Malasun", "width": 8, "vocab": 4, "streams": 2, "norm": {"eps": 1e-5}, "layers": [{"type": "hgrn2", "mixer": {"heads": 1, "dim": 4, "vdim": 4}, "mlp": None}]})


def test_oracle_mechanisms_on_hand_made_numbers():
    np.testing.assert_allclose(R.group_norm(np.array([[3.0, 4.0, 0.0, 2.0]]), np.array([1.0, 1.0, 1.0, 5.0]), 2, 0.0), [[3 / 12.5**0.5, 4 / 12.5**0.5, 0.0, 5 * 2**0.5]])
    np.testing.assert_allclose(R.rotate_half(np.array([[[1.0, 0.0, 0.0, 1.0, 7.0]]]), np.array([2]), 100.0, 4), [[[np.cos(2), -np.sin(0.2), np.sin(2), np.cos(0.2), 7.0]]])
    np.testing.assert_array_equal(R.chunk_mask(5, 3)[3:].astype(int), [[0, 0, 0, 1, 0], [0, 0, 0, 1, 1]])
    np.testing.assert_allclose(R.sink_softmax(np.log([[[1.0, 3.0]]]), np.log([4.0]), np.array([[True, True]])), [[[1 / 8, 3 / 8]]])
    z = np.array([[1.0, -2.0, 3.0]])
    r = lambda x: x / np.sqrt(np.mean(x * x))  # noqa: E731
    np.testing.assert_allclose(R.poly_norm(z, np.array([2.0, 3.0, 5.0, 7.0]), 0.0), 2 * r(z) + 3 * r(z**2) + 5 * r(z**3) + 7)
    np.testing.assert_allclose(R.gelu(np.array([1.0, -1.0])), [0.8413447460685429, -0.15865525393145707])
    x = np.array([[[1.0]], [[10.0]]])                            # two streams, one row, one column
    w = {"hc1.in": np.array([2.0, 3.0]), "hc1.out": np.array([1.0, -1.0]), "hc1.mix": np.array([[1.0, 4.0], [0.5, 0.0]])}
    np.testing.assert_allclose(R.hyper_in(x, w, 1), [[32.0]])
    np.testing.assert_allclose(R.hyper_out(x, np.array([[100.0]]), w, 1), [[[1 + 5 + 100.0]], [[4.0 - 100.0]]])
    q = np.array([[[1.0], [2.0]]])                               # one query, two heads of width 1 over one key head
    y = R.talking_attention(q, np.array([[[3.0]]]), np.array([[[1.0]]]), np.array([[1.0, 1.0], [0.0, 1.0]]), np.zeros(2), 1.0, np.array([[True]]))
    np.testing.assert_allclose(y[0, :, 0], [1 / (1 + np.exp(-9.0)), 1 / (1 + np.exp(-6.0))])
    one = {"table": np.array([[1, 0], [1, 2]]), **{f"e{e}.up": np.eye(1) * (e + 1) for e in range(3)}, **{f"e{e}.down": np.eye(1) for e in range(3)}}
    np.testing.assert_allclose(R.table_experts(np.array([[1.0], [1.0]]), np.array([1, 0]), one, 2)[:, 0], [(R.gelu(np.array(2.0)) + R.gelu(np.array(3.0))) / 2, (R.gelu(np.array(2.0)) + R.gelu(np.array(1.0))) / 2])


def test_weights_tell_mechanisms_apart():
    """A missing bias, norm, sink or mix, another rotation, chunk, expert or stream: each moves the logits by hundreds of times the fp32
    tolerance."""
    name = "mixed"
    cfg, t, W = CONFIGS[name], tokens(CONFIGS[name], 100, 3), weights(name)
    want = R.forward(t, cfg, W)

    def moved(c, w):
        return logit_err(R.forward(t, c, w), want) > 300 * TOL["float32"]

    for i, l in enumerate(cfg["layers"]):
        own = l["mixer"].get("kv_from") is None
        for key in ("q.b", "q.norm", "talk", "sink", "o.b") + (("k.b", "v.b", "k.norm") if own else ()):
            key = f"l{i}.mix.{key}"
            assert moved(cfg, {**W, key: np.roll(W[key], 1, axis=-1)}) and moved(cfg, {**W, key: np.zeros_like(W[key])}), key
        assert moved(cfg, {**W, f"l{i}.mix.talk": W[f"l{i}.mix.talk"].T})
        for q in (1, 2) if l["mlp"] else (1,):
            for key in ("out", "mix") if (i, q) == (0, 1) else ("in", "out", "mix"):        # (ahead of the first sublayer all streams are equal)
                other = W[f"l{i}.hc{q}.{key}"].copy()
                other.flat[0] += 0.3
                assert moved(cfg, {**W, f"l{i}.hc{q}.{key}": other}), (i, q, key)
            assert moved(cfg, {**W, f"l{i}.hc{q}.mix": W[f"l{i}.hc{q}.mix"].T})
        parts = [("scale", 0.9), ("mask", 1), ("mask", -1)] + ([("base", 0.8), ("dims", -2)] if own and l["mixer"]["rot"]["dims"] > 2 else [])
        for key, by in parts:
            other = json.loads(json.dumps(cfg))
            m = other["layers"][i]["mixer"]
            if key == "mask":
                if m["mask"] is None:
                    continue
                m["mask"]["size"] += by
            else:
                target = m if key == "scale" else m["rot"]
                target[key] = target[key] + by if key == "dims" else target[key] * by
            assert moved(other, W), (i, key)
        if l["mlp"] and l["mlp"]["kind"] == "dense":
            for k in range(4):
                a = W[f"l{i}.mlp.act"].copy()
                a[k] = 0.0
                assert moved(cfg, {**W, f"l{i}.mlp.act": a})
        elif l["mlp"]:
            if l["mlp"]["router"]["top"] < l["mlp"]["router"]["experts"]:
                assert moved(cfg, {**W, f"l{i}.mlp.table": np.roll(W[f"l{i}.mlp.table"], 1, axis=0)})
            if l["mlp"].get("shared"):
                assert moved(cfg, {**W, f"l{i}.mlp.shared.sg": -W[f"l{i}.mlp.shared.sg"]})
    for groups in (1, 10):
        assert moved({**cfg, "norm": {**cfg["norm"], "groups": groups}}, W)
    assert moved({**cfg, "logit_softcap": 2.6}, W) and moved({k: v for k, v in cfg.items() if k != "logit_softcap"}, W)


def test_scheduler_feeds_unequal_requests_and_gives_slots_back():
    from pygpukit_amd.llm import BatchScheduler

    e = FakeEngine()
    s = BatchScheduler(e)
    a, b = s.step([("a", [5, 6, 7], [0, 2]), ("b", [8], [0])])
    assert a.tolist() == [[0, 0, 5], [0, 2, 7]] and b.tolist() == [[1, 0, 8]]
    a, b = s.step([("a", [1], [0]), ("b", [2], [0])])
    assert a.tolist() == [[0, 3, 1]] and b.tolist() == [[1, 1, 2]] and e.calls[-1] == ("decode", 2)
    s.release("a")
    assert s.step([("b", [3], [0])])[0].tolist() == [[1, 2, 3]]
    assert s.step([("c", [4, 4], [1])])[0].tolist() == [[0, 1, 4]]            # the freed slot, from position 0


# ------------------------------------------------------------------------------------------------ GPU: operators
OP_TOL = {"float32": 3e-6, "bfloat16": 1.5e-2}
both = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


def worst(got, want):
    return float(np.max(np.abs(got - want)) / np.max(np.abs(want)))


@gpu
@both
def test_streams_norms_and_activations(dtype):
    from pygpukit_amd.ops.basic import gelu_erf, group_norm_f32, hyper_read, hyper_write, poly_norm, soft_cap

    rng = np.random.default_rng(1)
    f32 = lambda *s: rng.standard_normal(s).astype(np.float32)  # noqa: E731
    for S, W in ((1, 5), (2, 77), (5, 300), (8, 64)):
        x, y, c, d, M = f32(9, S, W), rounded(f32(9, W), dtype), f32(S), f32(S), f32(S, S)
        w = {"hc1.in": c, "hc1.out": d, "hc1.mix": M}
        dx = dev(x, "float32")
        assert worst(host(hyper_read(dx, dev(c, "float32"))), R.hyper_in(x.transpose(1, 0, 2).astype(np.float64), w, 1)) < OP_TOL["float32"]
        assert worst(host(hyper_read(dx)), x.sum(axis=1)) < OP_TOL["float32"]
        want = R.hyper_out(x.transpose(1, 0, 2).astype(np.float64), y.astype(np.float64), w, 1).transpose(1, 0, 2)
        assert worst(host(hyper_write(dx, dev(y, dtype), dev(d, "float32"), dev(M, "float32"))), want) < OP_TOL["float32"]
    for W, groups in ((60, 1), (60, 4), (77, 11), (300, 300), (5000, 2)):
        x, w = f32(7, W) * np.linspace(0.01, 3, W, dtype=np.float32), f32(W)
        assert worst(host(group_norm_f32(dev(x, "float32"), dev(w, "float32"), groups, 1e-3, dtype=dev(x[:1], dtype).dtype)), R.group_norm(x.astype(np.float64), w, groups, 1e-3)) < OP_TOL[dtype]
    act = rng.uniform(-1, 1, 4).astype(np.float32)
    for W in (1, 6, 77, 512, 5000, 20000):
        z = rounded(f32(5, W) * 3, dtype)
        assert worst(host(poly_norm(dev(z, dtype), dev(act, "float32"), 1e-3)), R.poly_norm(z.astype(np.float64), act, 1e-3)) < OP_TOL[dtype]
    z = rounded(np.linspace(-9, 9, 1111).reshape(1, -1), dtype)
    assert worst(host(gelu_erf(dev(z, dtype))), R.gelu(z.astype(np.float64))) < OP_TOL[dtype]
    assert worst(host(soft_cap(dev(z, dtype), 2.5)), 2.5 * np.tanh(z.astype(np.float64) / 2.5)) < OP_TOL[dtype]


@gpu
@both
def test_norm_and_rotation_of_heads(dtype):
    from pygpukit_amd.ops.basic import head_norm_rope

    rng = np.random.default_rng(2)
    for heads, dim, rot, first in ((1, 2, 2, 0), (3, 24, 10, 7), (4, 128, 128, 900), (2, 65, 0, 3), (5, 300, 64, 40)):
        x, w = rounded(rng.standard_normal((6, heads, dim)) * 2, dtype), (1 + 0.3 * rng.standard_normal(dim)).astype(np.float32)
        freq = dev((300.0 ** (-2.0 * np.arange(rot // 2) / rot)).astype(np.float32), "float32") if rot else None
        p = first + np.arange(6)
        for norm in (w, None):
            h = x.astype(np.float64) if norm is None else R.rms(x.astype(np.float64), 1e-4) * w
            want = R.rotate_half(h, p, 300.0, rot) if rot else h
            got = host(head_norm_rope(dev(x, dtype), None if norm is None else dev(w, "float32"), freq, first, 1e-4))
            assert worst(got, want) < max(OP_TOL[dtype], 3e-7 * first)               # an fp32 angle of `first` radians


def talk_case(rng, n, H, G, dk, dv, dtype):
    q, k, v = (rounded(rng.standard_normal(s), dtype) for s in ((n, H, dk), (n, G, dk), (n, G, dv)))
    return q, k, v, (np.eye(H) + 0.4 * rng.standard_normal((H, H))).astype(np.float32), rng.uniform(-1, 4, H).astype(np.float32)


@gpu
@both
@pytest.mark.parametrize("H,G,dk,dv", [(1, 1, 7, 9), (4, 2, 24, 40), (6, 6, 64, 64), (8, 2, 128, 128), (33, 3, 30, 18), (2, 1, 520, 30)])
def test_talk_attention(H, G, dk, dv, dtype):
    """Chunks, windows and neither; with and without mix and sink; queries that start inside a chunk."""
    from pygpukit_amd.ops.basic import talk_attention

    rng = np.random.default_rng(3)
    n = 150
    q, k, v, talk, sink = talk_case(rng, n, H, G, dk, dv, dtype)
    scale = 1.5 / np.sqrt(dk)
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    for size, chunked in ((1, True), (37, True), (64, True), (500, True), (1, False), (40, False), (500, False)):
        mask = R.chunk_mask(n, size) if chunked else (j <= i) & (i - j < size)
        for t, s in ((talk, sink), (None, sink), (talk, None)):
            want = R.talking_attention(*(x.astype(np.float64) for x in (q, k, v)), np.eye(H) if t is None else t.astype(np.float64), np.full(H, -np.inf) if s is None else s.astype(np.float64), scale, mask)
            for start in (0, 100):                             # the queries from there on, with the keys they can see
                lo = 0 if start == 0 else start - start % size if chunked else max(0, start - size + 1)
                got = talk_attention(dev(q[start:], dtype), dev(k[lo:], dtype), dev(v[lo:], dtype), scale, size, chunked=chunked, first=lo, talk=None if t is None else dev(t, "float32"),
                                     sink=None if s is None else dev(s, "float32"))
                assert worst(host(got), want[start:]) < OP_TOL[dtype], (size, chunked, start)


@gpu
@both
def test_table_experts(dtype):
    from pygpukit_amd.core.factory import from_numpy
    from pygpukit_amd.ops.basic import table_experts

    rng = np.random.default_rng(4)
    for n, W, ff, E, top in ((1, 10, 20, 1, 1), (5, 64, 64, 7, 3), (60, 70, 33, 5, 5), (300, 128, 192, 4, 2), (700, 64, 128, 40, 1), (2000, 128, 256, 3, 1)):
        table = np.stack([rng.permutation(E)[:top] for _ in range(50)]).astype(np.int32)
        x, t = rounded(rng.standard_normal((n, W)), dtype), rng.integers(0, 50, n).astype(np.int32)
        w = {f"e{e}.{k}": rounded(rng.standard_normal(s) / np.sqrt(s[1]) * 1.5, dtype) for e in range(E) for k, s in (("up", (ff, W)), ("down", (W, ff)))}
        up, down = (np.stack([w[f"e{e}.{k}"] for e in range(E)]) for k in ("up", "down"))
        want = R.table_experts(x.astype(np.float64), t, {"table": table, **{k: a.astype(np.float64) for k, a in w.items()}}, top)
        got = host(table_experts(dev(x, dtype), from_numpy(t), from_numpy(table), dev(up, dtype), dev(down, dtype)))
        assert worst(got, want) < OP_TOL[dtype], (n, W, ff, E, top)


# ------------------------------------------------------------------------------------------------ GPU: whole models
_models: dict = {}
_refs: dict = {}
every = pytest.mark.parametrize("name", [c for c in CONFIGS if not c.startswith("edge")])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name, dtype):
        if (name, dtype) not in _models:
            from pygpukit_amd.llm import load_model_from_safetensors

            cfg, W = CONFIGS[name], weights(name)
            folder = save(tmp_path_factory.mktemp(name), cfg, W)
            _models[name, dtype] = cfg, W, load_model_from_safetensors(folder, dtype=dtype), folder
        return _models[name, dtype][:3]
    yield get
    _models.clear()
    _refs.clear()


def reference(name, n, seed=5):
    """n tokens and the restatement's logits of every row."""
    if (name, n, seed) not in _refs:
        t = tokens(CONFIGS[name], n, seed)
        _refs[name, n, seed] = t, R.forward(t, CONFIGS[name], weights(name))
    return _refs[name, n, seed]


@gpu
@both
@every
def test_streams_after_every_layer(models, name, dtype):
    """The first k layers of the model as a model of their own: the output norm and head tell where the streams first differ."""
    from pygpukit_amd.llm.engine import StackEngine

    cfg, W, model = models(name, dtype)
    t = tokens(cfg, 40, 8)
    full = model.build_engine(max_seq_len=64, max_batch=1)
    head, fnorm = model._stack_head
    for k in range(1, len(cfg["layers"])):
        e = StackEngine({x: v for x, v in full.config.items() if x != "num_layers"}, model.embed_tokens, None, head, fnorm, full.layers[:k], max_seq_len=64, max_batch=1)
        assert near(e.prefill_batch([t], want=[list(range(40))]), R.forward(t, dict(cfg, layers=cfg["layers"][:k]), W), dtype), k


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


@gpu
@both
@every
def test_engine_prompt_every_row(models, name, dtype):
    cfg, W, model = models(name, dtype)
    n = {"tiles": 400, "deep": 1100}.get(name, 150)
    t, want = reference(name, n)
    e = model.build_engine(max_seq_len=n, max_batch=2)
    got = e.prefill_batch([t], [1], want=[list(range(n))])
    assert got.shape == want.shape and near(got, want, dtype, n)
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
@pytest.mark.parametrize("name", ["edge37", "edge64"])
def test_keys_at_chunk_edges(models, name, dtype):
    """A token whose key stands out, put on a chunk's first position, moves the logits of the chunk's rows; put one before it, it moves none.
    In prompts and in decoding over a ring that holds both sides of the edge."""
    cfg, W, model = models(name, dtype)
    C = cfg["layers"][0]["mixer"]["mask"]["size"]
    t = tokens(cfg, 3 * C, 4)
    base = R.forward(t, cfg, W)
    rms = lambda a: np.sqrt(np.mean(np.square(a)))  # noqa: E731
    e = model.build_engine(max_seq_len=3 * C, max_batch=1)

    def both_ways(s, p):
        """Row p of a prompt that goes on behind it, of one that ends there, and decoded."""
        rows = [e.prefill_batch([s], want=[[p]])[0], e.prefill(s[:p + 1])]
        e.prefill(s[:p], want_last_logits=False)
        e.set_state([s[p]], [p])
        e.decode_step(1)
        return np.stack([*rows, e.logits(1).to_numpy()[0]])

    for first in (C, 2 * C):
        for p in (first + 1, first + C // 2, first + C - 1):
            swap = lambda j, z: t[:j] + [z] + t[j + 1:]  # noqa: E731
            z = max(range(cfg["vocab"]), key=lambda z: rms(R.forward(swap(first, z)[:p + 1], cfg, W)[p] - base[p]))
            inside, outside = swap(first, z), swap(first - 1, z)
            want = R.forward(inside, cfg, W)[p]
            assert rms(want - base[p]) > 0.3 * rms(base)
            assert rms(R.forward(outside, cfg, W)[p] - base[p]) == 0.0
            assert near(both_ways(inside, p), np.stack([want] * 3), dtype, p), p
            assert near(both_ways(outside, p), np.stack([base[p]] * 3), dtype, p), p


@gpu
@both
@pytest.mark.parametrize("batch", [1, 2, 17, 40])
def test_far_keys_in_batches(models, dtype, batch):
    """Near one-hot attention at positions up to 700, chunks of 256 to 500, in batch sizes that give one split and several."""
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
    assert near(np.concatenate(got), np.concatenate(exp), dtype, n)


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


def greedy(t, n, cfg, W):
    t = list(t)
    for _ in range(n):
        t.append(int(np.argmax(R.forward(t, cfg, W)[-1])))
    return t


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
    with pytest.raises(RuntimeError, match="no longer in its ring"):
        e.prefill(t[20:21], start_pos=20)
    got = e.prefill_batch([t[59:60]], [0], [59], want=[[0]])      # all of its chunks are still there
    assert near(got, want[59:60], "float32")
    e.set_state([t[60]], [60])                                 # going on is fine, and so is starting again
    e.decode_step()
    assert near(e.logits(1).to_numpy(), want[60:61], "float32")
    assert near(e.prefill(t[:20])[None], want[19:20], "float32")
    for bad in (lambda: e.prefill([cfg["vocab"]]), lambda: e.prefill(t[:1], seq=1), lambda: e.prefill_batch([t + [0] * 20], [0], [0]), lambda: e.prefill_batch([t[:2], t[:2]], [0, 0])):
        with pytest.raises(RuntimeError):
            bad()


@gpu
def test_loader_checks_shapes(tmp_path):
    from pygpukit_amd.llm import load_fetezen_from_safetensors, load_model_from_safetensors

    cfg, W = CONFIGS["mixed"], weights("mixed")
    folder = save(tmp_path, cfg, W)
    m = load_fetezen_from_safetensors(os.path.join(folder, "model.safetensors"), dtype="float32")
    assert m.config.streams == 3 and m.blocks[1].mlp.num_experts == 10 and m.blocks[2].mlp is None and m.blocks[1].attn.source is m.blocks[0].attn and m.blocks[3].mlp.shared_up is None
    for layer, key, value, tensor in ((3, "vdim", 21, "l3.mix.v"), (1, "heads", 4, "l1.mix.q"), (6, "dim", 16, "l6.mix.q")):
        other = json.loads(json.dumps(cfg))
        other["layers"][layer]["mixer"][key] = value
        save(tmp_path, other, W)
        with pytest.raises(ValueError, match=tensor.replace(".", r"\.")):
            load_model_from_safetensors(folder)
    for missing in ("l1.mlp.e9.down", "l1.mlp.table", "l0.mlp.act", "l0.mix.sink", "l2.mix.talk", "l4.mix.o.b", "l3.hc2.mix", "l1.mlp.shared.sg"):
        save(tmp_path, cfg, {k: v for k, v in W.items() if k != missing})
        with pytest.raises(ValueError, match=missing.replace(".", r"\.")):
            load_model_from_safetensors(folder)
    table = W["l1.mlp.table"].copy()
    table[200, 1] = 10
    save(tmp_path, cfg, {**W, "l1.mlp.table": table})
    with pytest.raises(ValueError, match="names experts outside"):
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
    assert lines[0][:3] == [3, 4, 5] and len(lines[0]) == 9 and lines[1] == greedy([9], 6, cfg, W)
