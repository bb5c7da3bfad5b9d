"""What the tests of the layer-list models share: checkpoints on disk, arrays on the device, error measure, a recording engine."""

from __future__ import annotations

import json
import os

import numpy as np

from oracle import cpu_ref as O


def bf16(x: np.ndarray) -> np.ndarray:
    """fp32 values rounded to bfloat16."""
    x = np.asarray(x, np.float32)
    return O.bf16_bits_to_f32(O.f32_to_bf16_bits(x)).reshape(x.shape)


def save(folder, cfg, W):
    from pygpukit_amd.llm.safetensors import save_safetensors

    with open(os.path.join(folder, "config.json"), "w", encoding="utf-8") as f:
        json.dump(cfg, f)
    save_safetensors(os.path.join(folder, "model.safetensors"), {k: (np.asarray(v, np.int32), "I32") if np.issubdtype(v.dtype, np.integer) else
                                                                 (O.f32_to_bf16_bits(v).reshape(v.shape), "BF16") for k, v in W.items()})
    return str(folder)


def logit_err(got, want):
    d = np.asarray(got, np.float64) - want
    return float(np.max(np.sqrt(np.mean(d * d, axis=-1)) / np.sqrt(np.mean(want * want))))


def tokens(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def dev(x, dtype):
    from pygpukit_amd.core.factory import from_numpy

    x = np.ascontiguousarray(x, np.float32)
    if dtype == "float32":
        return from_numpy(x)
    return from_numpy(x.astype(np.float16) if dtype == "float16" else O.f32_to_bf16_bits(x).reshape(x.shape))


def host(a):
    h = a.to_numpy()
    return O.bf16_bits_to_f32(h).reshape(h.shape) if h.dtype == np.uint16 else h.astype(np.float32)


def rounded(x, dtype):
    x = np.asarray(x, np.float32)
    if dtype == "bfloat16":
        return O.bf16_bits_to_f32(O.f32_to_bf16_bits(x)).reshape(x.shape)
    return x.astype(np.float16).astype(np.float32) if dtype == "float16" else x


class FakeEngine:
    """Records what the scheduler asks for; the `logits` of a row are (slot, position, token)."""

    def __init__(self, max_batch=3, max_seq_len=20):
        self.max_batch, self.max_seq_len, self.config, self.calls = max_batch, max_seq_len, {"vocab_size": 3}, []

    def prefill_batch(self, prompts, slots, starts, want):
        self.calls.append(("prefill", list(slots), list(starts), [len(p) for p in prompts]))
        return np.array([(s, st + i, p[i]) for p, s, st, w in zip(prompts, slots, starts, want) for i in w], np.float32).reshape(-1, 3)

    def set_state(self, tok, pos):
        self.state = [(i, p, t) for i, (t, p) in enumerate(zip(tok, pos))]

    def decode_step(self, rows):
        self.calls.append(("decode", rows))

    def logits(self, rows):
        state = self.state

        class A:
            @staticmethod
            def to_numpy():
                return np.array(state, np.float32)
        return A()
