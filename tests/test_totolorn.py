"""Totolorn (layer-list decoder: fp32 residual stream, norms around zero before and after each sublayer, sliding-window latent attention
with a head gate, SwiGLU or no feed-forward) against the plain NumPy restatement in oracle/totolorn_ref.py.

Weights are random with scores made sharp (a large query / key scale), so that one key too many or too few in a window, a stale cache
row or a lost position moves the logits by far more than the tolerances; test_weights_tell_windows_apart asserts that on the CPU."""

from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

from tests.layer_list import FakeEngine, dev, host, logit_err, rounded, save, tokens
from oracle import cpu_ref as O
from oracle import totolorn_ref as R

ROOT = os.path.abspath(os.path.join(os.path.dirname(__file__), ".."))
gpu = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 4e-2}       # rms over the vocabulary of the logit difference / rms of the logits


def mixer(heads, dim, vdim, rank, window, scale):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "mask": {"size": window}}}


def config(width, vocab, layers, positions, eps=1e-5, mult=0.7):
    return {"architecture": "Totolorn", "width": width, "vocab": vocab, "max_positions": positions, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": [dict(m, mlp=None if ff is None else {"kind": "dense", "ff": ff}) for m, ff in layers]}


CONFIGS = {
    # every layer different; no width a multiple of 64; a window of one, a layer without feed-forward
    "mixed": config(96, 211, [(mixer(3, 24, 40, 72, 7, 0.4), 160), (mixer(5, 40, 16, 40, 1, 0.3), None), (mixer(2, 96, 80, 136, 33, 0.2), 90)], 300, 1e-6, 0.55),
    # widths that are multiples of nothing, one head, no window reached, residual factor 1
    "odd": config(70, 97, [(mixer(1, 18, 22, 10, 500, 0.5), 33), (mixer(7, 6, 10, 20, 12, 0.8), 50)], 200, 1e-3, 1.0),
    # head width above 128 (no MFMA prompt kernel) and a latent above 512
    "wide": config(192, 130, [(mixer(3, 144, 72, 520, 20, 0.15), 128), (mixer(2, 136, 160, 64, 70, 0.12), None)], 160, 1e-5, 0.8),
    # widths the engine takes without padding, 16 and 20 heads, windows around the 64-key tiles of the prompt kernel
    # long rows (every preload depth of the one-row projection, split-K slabs) and latents past each width class of the decode kernels
    "long": config(1100, 120, [(mixer(2, 30, 30, 30, 50, 0.3), 4200), (mixer(2, 20, 64, 1000, 9, 0.4), 2100)], 320, 1e-5, 0.9),
    "widest": config(4200, 50, [(mixer(3, 64, 64, 2000, 30, 0.2), 70)], 170),
    "middle": config(2100, 50, [(mixer(2, 64, 64, 300, 30, 0.2), None)], 170),
    # many heads and a window of several hundred: several key tiles per split
    "deep": config(64, 90, [(mixer(17, 32, 128, 256, 600, 0.3), 64), (mixer(33, 16, 48, 70, 1000, 0.4), None)], 720),
    "tiles": config(128, 256, [(mixer(16, 64, 64, 128, 65, 0.3), 256), (mixer(20, 128, 128, 192, 64, 0.2), 192), (mixer(4, 64, 48, 64, 127, 0.3), 64)], 700),
}


def weights(cfg, seed=0, sharp=2.5):
    rng = np.random.default_rng(seed)

    def draw(*shape, std):
        return O.bf16_bits_to_f32(O.f32_to_bf16_bits((rng.standard_normal(shape) * std).astype(np.float32))).reshape(shape)

    H, W = cfg["width"], {}
    W["embed"], W["pos"] = draw(cfg["vocab"], H, std=1.0), draw(cfg["max_positions"], H, std=0.5)
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        n, d, v, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        sub = ["norm1", "norm1b"] + (["norm2", "norm2b"] if l["mlp"] else [])
        for s in sub:
            W[p + s] = draw(H, std=0.2)
        s = (sharp / (m["scale"] * np.sqrt(d))) ** 0.5           # scores of standard deviation `sharp`
        W[p + "mix.q"], W[p + "mix.uk"] = draw(n * d, H, std=s / np.sqrt(H)), draw(n * d, r, std=s / np.sqrt(r))
        W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = draw(r, H, std=1 / np.sqrt(H)), draw(r, std=0.2) + np.float32(1.0)
        W[p + "mix.uv"], W[p + "mix.g"], W[p + "mix.o"] = draw(n * v, r, std=1 / np.sqrt(r)), draw(n, H, std=1 / np.sqrt(H)), draw(H, n * v, std=1 / np.sqrt(n * v))
        if l["mlp"]:
            f = l["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = draw(f, H, std=1 / np.sqrt(H)), draw(f, H, std=1 / np.sqrt(H)), draw(H, f, std=1 / np.sqrt(f))
    W["final.norm"], W["head"] = draw(H, std=0.2), draw(cfg["vocab"], H, std=1 / np.sqrt(H))
    return {k: O.bf16_bits_to_f32(O.f32_to_bf16_bits(v)).reshape(v.shape) for k, v in W.items()}


# ------------------------------------------------------------------------------------------------ CPU: configuration, oracle, scheduler
def test_config_is_read_layer_by_layer():
    from pygpukit_amd.llm import TOTOLORN_SPEC, detect_model_spec, layer_list_config

    c = layer_list_config(CONFIGS["mixed"])
    assert (c.hidden_size, c.vocab_size, c.num_layers, c.max_position_embeddings) == (96, 211, 3, 300)
    assert c.norm_eps == 1e-6 and c.residual_mult == 0.55 and not c.use_rope
    a, b, d = c.layers
    assert (a.num_heads, a.head_dim, a.v_head_dim, a.kv_rank, a.window, a.scale, a.intermediate_size) == (3, 24, 40, 72, 7, 0.4, 160)
    assert b.intermediate_size is None and b.window == 1 and d.num_heads == 2 and d.intermediate_size == 90
    assert detect_model_spec(["embed"], CONFIGS["mixed"]) is TOTOLORN_SPEC
    with pytest.raises(ValueError, match="unknown architecture"):
        detect_model_spec(["embed"], {"architecture": "Nothing"})
    for bad in ({"type": "recurrent"}, {"mlp": {"kind": "sparse", "ff": 4}}):
        broken = json.loads(json.dumps(CONFIGS["odd"]))
        broken["layers"][1].update(bad)
        with pytest.raises(ValueError, match="layer 1"):
            layer_list_config(broken)


def test_oracle_mechanisms_on_hand_made_numbers():
    x = np.array([[3.0, 4.0]])
    np.testing.assert_allclose(R.norm_around_zero(x, np.array([0.0, 1.0]), 0.0), x / np.sqrt(12.5) * [1.0, 2.0])
    np.testing.assert_array_equal(R.window_mask(4, 2), [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]])
    v = np.arange(5.0)[:, None, None]
    assert R.attend(np.zeros((5, 1, 2)), np.zeros((5, 1, 2)), v, 1.0, 3)[4, 0, 0] == 3.0           # mean of the last three values
    np.testing.assert_allclose(R.sigmoid(np.array([-700.0, 0.0, 700.0])), [0.0, 0.5, 1.0], atol=1e-12)


@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_weights_tell_windows_apart(name):
    """One key more or less in one layer's window moves the logits by hundreds of times the fp32 tolerance, in most layers by several
    times the bf16 one too (the kernels' own window edges are pinned in bf16 by test_window_edges_with_one_loud_key)."""
    cfg = CONFIGS[name]
    W, t = weights(cfg), tokens(cfg, 140, 3)
    want = R.forward(t, cfg, W)
    for layer in range(len(cfg["layers"])):
        for delta in (-1, 1):
            other = json.loads(json.dumps(cfg))
            other["layers"][layer]["mixer"]["mask"]["size"] += delta
            if other["layers"][layer]["mixer"]["mask"]["size"] < 1:
                continue
            assert logit_err(R.forward(t, other, W), want) > 500 * TOL["float32"]


def test_scheduler_slots_batches_and_order():
    from pygpukit_amd.llm.scheduler import BatchScheduler

    e = FakeEngine()
    s = BatchScheduler(e)
    out = s.step([("a", [5, 6, 7], [0, 2]), ("b", [8], [0])])
    np.testing.assert_array_equal(out[0], [[0, 0, 5], [0, 2, 7]])
    np.testing.assert_array_equal(out[1], [[1, 0, 8]])
    out = s.step([("b", [9], [0]), ("a", [4], [0])])                       # one token each: a decode step, in the caller's order
    assert e.calls[-1] == ("decode", 2)
    np.testing.assert_array_equal(out[0], [[1, 1, 9]])
    np.testing.assert_array_equal(out[1], [[0, 3, 4]])
    s.step([("b", [1], [])])                                               # 'a' lives but is not in the step: no decode over its slot
    assert e.calls[-1] == ("prefill", [1], [2], [1])
    s.step([("a", [1, 2], [1]), ("b", [3], [])])                           # portions
    assert e.calls[-1] == ("prefill", [0, 1], [4, 3], [2, 1]) and s.length("a") == 6
    s.release("a")
    assert s.live == ("b",)
    out = s.step([("b", [7], [0])])                                        # slot 0 idle: a dummy row at position 0
    assert e.calls[-1] == ("decode", 2) and e.state[0] == (0, 0, 0)
    np.testing.assert_array_equal(out[0], [[1, 4, 7]])
    s.step([("c", [1], []), ("d", [2], [])])
    with pytest.raises(RuntimeError, match="free"):
        s.step([("e", [1], [])])
    with pytest.raises(ValueError, match="exceed"):
        s.step([("c", [1] * 20, [])])
    with pytest.raises(ValueError, match="once"):
        s.step([("c", [1], []), ("c", [1], [])])
    assert set(s.live) == {"b", "c", "d"}


# ------------------------------------------------------------------------------------------------ GPU: operators
OP_TOL = {"float32": 2e-6, "float16": 2e-3, "bfloat16": 1.2e-2}


@gpu
@pytest.mark.parametrize("dtype", ["float32", "float16", "bfloat16"])
@pytest.mark.parametrize("rows,cols", [(1, 1), (3, 70), (5, 1024), (2, 5003)])
def test_stream_norms(rows, cols, dtype):
    from pygpukit_amd.core.dtypes import DataType
    from pygpukit_amd.ops.basic import rmsnorm_add_f32, rmsnorm_f32

    rng = np.random.default_rng(rows * cols)
    x, y, w = rng.standard_normal((rows, cols)), rounded(rng.standard_normal((rows, cols)) * 3, dtype), rng.standard_normal(cols)
    x, w = x.astype(np.float32), w.astype(np.float32)
    got = host(rmsnorm_f32(dev(x, "float32"), dev(w, "float32"), 1e-3, dtype=DataType.from_string(dtype)))
    want = R.norm_around_zero(x.astype(np.float64), w - 1.0, 1e-3)
    assert np.max(np.abs(got - want)) <= OP_TOL[dtype] * np.max(np.abs(want))
    s = dev(x, "float32")
    got = host(rmsnorm_add_f32(s, dev(y, dtype), dev(w, "float32"), 1e-3, 0.3))
    want = x + 0.3 * R.norm_around_zero(y.astype(np.float64), w.astype(np.float64) - 1.0, 1e-3)
    assert np.max(np.abs(got - want)) <= 2e-6 * np.max(np.abs(want))


@gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_head_gate_and_pad(dtype):
    from pygpukit_amd.ops.basic import head_gate, pad_2d

    rng = np.random.default_rng(1)
    x, g = rounded(rng.standard_normal((7, 3, 10)), dtype), rounded(rng.standard_normal((7, 3)) * 4, dtype)
    got = host(head_gate(dev(x, dtype), dev(g, dtype)))
    assert np.max(np.abs(got - x * R.sigmoid(g.astype(np.float64))[:, :, None])) < OP_TOL[dtype] * 4
    a = dev(x.reshape(7, 30), dtype)
    p = host(pad_2d(a, 9, 32))
    np.testing.assert_array_equal(p[:7, :30], x.reshape(7, 30))
    assert not p[7:].any() and not p[:, 30:].any() and pad_2d(a, 7, 30) is a
    with pytest.raises(ValueError):
        pad_2d(a, 6, 30)


@gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dk,dv", [(2, 64, 64), (3, 128, 128), (2, 20, 36), (1, 200, 64)])
@pytest.mark.parametrize("q_len,kv_len,window", [(1, 1, 1), (5, 5, 2), (130, 130, 1), (200, 333, 64), (70, 300, 65), (129, 257, 63), (300, 300, 1000), (2, 400, 129),
                                                 (100, 128, 500), (128, 128, 128), (30, 90, 90)])
def test_window_attention(heads, dk, dv, q_len, kv_len, window, dtype):
    from pygpukit_amd.ops.basic import window_attention

    rng = np.random.default_rng(q_len + kv_len + window)
    q, k, v, g = (rounded(rng.standard_normal(s), dtype) for s in ((q_len, heads, dk), (kv_len, heads, dk), (kv_len, heads, dv), (q_len, heads)))
    scale = 1.5 / np.sqrt(dk)
    full = np.zeros((kv_len, heads, dk))
    full[kv_len - q_len:] = q
    want = R.attend(full, k.astype(np.float64), v.astype(np.float64), scale, window)[kv_len - q_len:]
    tol = 3e-6 if dtype == "float32" else 1.5e-2
    got = host(window_attention(dev(q, dtype), dev(k, dtype), dev(v, dtype), scale, window))
    assert np.max(np.abs(got - want)) < tol * np.max(np.abs(want))
    got = host(window_attention(dev(q, dtype), dev(k, dtype), dev(v, dtype), scale, window, gate=dev(g, dtype)))
    want = want * R.sigmoid(g.astype(np.float64))[:, :, None]
    assert np.max(np.abs(got - want)) < tol * np.max(np.abs(want))


@gpu
@pytest.mark.parametrize("dtype,d", [("float32", 48), ("bfloat16", 64), ("bfloat16", 128), ("bfloat16", 48)])
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 128, 129, 200])
def test_window_edges_with_one_loud_key(dtype, d, window):
    """Key j is aligned with every query and its value is the only one that is not zero: query i sees it exactly while i - j < window."""
    from pygpukit_amd.ops.basic import window_attention

    n = 333
    for j in (0, 63, 64, 100):
        q, k, v = np.zeros((n, 1, d), np.float32), np.zeros((n, 1, d), np.float32), np.zeros((n, 1, d), np.float32)
        q[:, 0, 0], k[j, 0, 0], v[j, 0, :] = 8.0, 8.0, 1.0
        got = host(window_attention(dev(q, dtype), dev(k, dtype), dev(v, dtype), 0.5, window))[:, 0, :]
        seen = np.zeros(n)
        seen[j:j + window] = 1.0
        assert np.max(np.abs(got - seen[:, None])) < 1e-2


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
        cfg = CONFIGS[name]
        t = tokens(cfg, n, seed)
        _ref[name, n, seed] = (t, R.forward(t, cfg, weights(cfg)))
    return _ref[name, n, seed]


both = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
every = pytest.mark.parametrize("name", list(CONFIGS))


@gpu
@both
@every
def test_eager_model(models, name, dtype):
    cfg, W, model = models(name, dtype)
    t, want = reference(name, 90)
    hidden, past = model(t[:80], use_cache=True)
    assert past[0][0].shape == (80, cfg["layers"][0]["mixer"]["kv_rank"])
    got = [host(model.get_logits(hidden))]
    for i in range(80, 84):                                    # one token at a time over the growing latents
        hidden, past = model([t[i]], past_key_values=past, use_cache=True)
        got.append(host(model.get_logits(hidden)))
    hidden, _ = model(t[84:], past_key_values=past, use_cache=True)
    got.append(host(model.get_logits(hidden)))
    assert logit_err(np.concatenate(got), want) < TOL[dtype]


@gpu
@both
def test_fixed_cache_strategies(models, dtype):
    """DecodeM1 and the verify-style DecodeBatch on the model's own fixed latent caches."""
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


@gpu
@both
@every
def test_engine_prompt_every_row(models, name, dtype):
    cfg, W, model = models(name, dtype)
    n = {"tiles": 400}.get(name, 150)
    t, want = reference(name, n)
    e = model.build_engine(max_seq_len=cfg["max_positions"], max_batch=2)
    got = e.prefill_batch([t], [1], want=[list(range(n))])
    assert got.shape == want.shape and logit_err(got, want) < TOL[dtype]
    for k in (1, 2, 3):                                        # the first tokens of a sequence as whole prompts
        assert logit_err(e.prefill(t[:k], seq=0)[None], want[k - 1:k]) < TOL[dtype]


@gpu
@both
@every
@pytest.mark.parametrize("batch", [1, 3, 9])
def test_engine_decode_is_the_prompt(models, name, dtype, batch):
    """Token by token from the very first one, in batches of sequences that run at different positions."""
    cfg, W, model = models(name, dtype)
    n = 110
    t, want = reference(name, n)
    e = model.build_engine(max_seq_len=128, max_batch=batch)
    lag = [5 * b for b in range(batch)]                        # sequence b starts with a prompt of lag[b] tokens
    for b in range(batch):
        if lag[b]:
            e.prefill(t[:lag[b]], seq=b, want_last_logits=False)
    worst = 0.0
    for i in range(n - max(lag)):
        e.set_state([t[p + i] for p in lag], [p + i for p in lag])
        e.decode_step(batch)
        worst = max(worst, logit_err(e.logits(batch).to_numpy(), want[[p + i for p in lag]]))
    assert worst < TOL[dtype]


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
    """Requests of different lengths together equal each alone; finished ones give their slots to new ones."""
    from pygpukit_amd.llm import BatchScheduler

    cfg, W, model = models(name, dtype)
    lens = [1, 40, 7, 90]
    ref = [reference(name, n + 12, seed=20 + i) for i, n in enumerate(lens)]
    s = BatchScheduler(model.build_engine(max_seq_len=128, max_batch=4))
    for again in range(2):                                    # the second time every slot holds another request's leftovers
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
    """Sequences around and beyond a 600-key window, in batch sizes that give a split one key tile and several."""
    cfg, W, model = models("deep", dtype)
    n = 700
    t, want = reference("deep", n)
    e = model.build_engine(max_seq_len=720, max_batch=batch)
    at = [(590 + 13 * b) % 690 + 1 if b < 8 else 1 + (37 * b) % 680 for b in range(batch)]
    e.prefill_batch([t[:p] for p in at], want=[[]] * batch)
    worst = 0.0
    for i in range(6):
        e.set_state([t[p + i] for p in at], [p + i for p in at])
        e.decode_step(batch)
        worst = max(worst, logit_err(e.logits(batch).to_numpy(), want[[p + i for p in at]]))
    assert worst < TOL[dtype]


@gpu
@pytest.mark.parametrize("packed", ["0", "1"])
@pytest.mark.parametrize("name", ["long", "tiles"])
def test_projection_routes_agree(models, name, packed, monkeypatch):
    """Fragment-major copies on and off: prompts of 2..300 rows and batches take other kernels, the logits stay the same."""
    monkeypatch.setenv("PGK_PACKED_PREFILL", packed)
    cfg, W, model = models(name, "bfloat16")
    t, want = reference(name, 300)
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
    worst = 0.0
    for i in range(300):
        e.set_state([t[3 + i], t[100 + i]], [3 + i, 100 + i])
        if i % 3:
            e.replay(1)
        else:
            e.decode_step(2)
        if i % 7 == 0 or i > 290 or 60 <= i <= 66 or 123 <= i <= 128:
            worst = max(worst, logit_err(e.logits(2).to_numpy(), want[[3 + i, 100 + i]]))
    assert worst < TOL[dtype]
    assert e.latent_cache(1).shape == (2, 64, 192) and e.latent_cache(0).shape == (2, 65, 128)


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
def test_positions_that_left_the_ring_are_refused(models):
    cfg, W, model = models("mixed", "float32")
    e = model.build_engine(max_seq_len=100, max_batch=1)
    t, want = reference("mixed", 90)
    e.prefill(t[:60], want_last_logits=False)
    with pytest.raises(RuntimeError, match="holds 60 positions"):
        e.set_state([t[61]], [61])
    with pytest.raises(RuntimeError, match="no longer in its ring"):
        e.prefill(t[50:60], start_pos=50)
    e.set_state([t[60]], [60])                                 # going on is fine, and so is starting again
    e.decode_step()
    assert logit_err(e.logits(1).to_numpy(), want[60:61]) < TOL["float32"]
    assert logit_err(e.prefill(t[:20])[None], want[19:20]) < TOL["float32"]
    for bad in (lambda: e.prefill([cfg["vocab"]]), lambda: e.prefill(t[:1], seq=1), lambda: e.prefill_batch([t[:101 - 0]], [0], [1]),
                lambda: e.prefill_batch([t[:2], t[:2]], [0, 0])):
        with pytest.raises(RuntimeError):
            bad()
    with pytest.raises(RuntimeError, match="learned positions"):
        model.build_engine(max_seq_len=cfg["max_positions"] + 1)


@gpu
def test_loader_checks_shapes(tmp_path):
    from pygpukit_amd.llm import load_model_from_safetensors, load_totolorn_from_safetensors

    cfg, W = CONFIGS["odd"], weights(CONFIGS["odd"])
    folder = save(tmp_path, cfg, W)
    m = load_totolorn_from_safetensors(os.path.join(folder, "model.safetensors"), dtype="float32")
    assert m.config.layers[1].num_heads == 7 and m.blocks[0].attn.kv_rank == 10
    other = json.loads(json.dumps(cfg))
    other["layers"][0]["mixer"]["kv_rank"] = 11
    save(tmp_path, other, W)
    with pytest.raises(ValueError, match="dkv"):
        load_model_from_safetensors(folder)
    save(tmp_path, cfg, {k: v for k, v in W.items() if k != "l1.mix.uv"})
    with pytest.raises(ValueError, match="l1.mix.uv"):
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
