"""Batch scheduler over the native engine: sequences come and go, each holds a cache slot while it lives.

`step()` is the one place that drives the engine: new sequences and multi-token portions run as one ragged prompt call, sequences that
go on by one token as one decode step.  `generate()` is continuous batching on top of it - a waiting prompt takes the slot of a
finished sequence - with greedy or in-step stochastic sampling (Engine.set_sampling)."""

from __future__ import annotations

import heapq
from collections.abc import Hashable, Sequence

import numpy as np


class BatchScheduler:
    def __init__(self, engine):
        self.engine = engine
        self._free = list(range(engine.max_batch))       # lowest slot first: live slots stay dense, a decode step runs slots 0 .. highest
        self._slot: dict[Hashable, int] = {}
        self._len: dict[Hashable, int] = {}

    @property
    def live(self) -> tuple[Hashable, ...]:
        return tuple(self._slot)

    def length(self, seq: Hashable) -> int:
        return self._len[seq]

    def release(self, seq: Hashable) -> None:
        heapq.heappush(self._free, self._slot.pop(seq))
        del self._len[seq]

    def _admit(self, seq: Hashable) -> None:
        if not self._free:
            raise RuntimeError(f"no free slot for sequence {seq!r} ({self.engine.max_batch} slots)")
        self._slot[seq] = heapq.heappop(self._free)
        self._len[seq] = 0

    def step(self, entries: Sequence[tuple[Hashable, Sequence[int], Sequence[int]]]) -> list[np.ndarray]:
        """entries: (sequence, its next tokens, which of them want logits).  Unknown sequences are admitted.  Returns one fp32 array
        [len(wanted), V] per entry."""
        if len({s for s, _, _ in entries}) != len(entries):
            raise ValueError("a sequence may appear once per step")
        for s, toks, want in entries:
            if len(toks) < 1 or any(not 0 <= w < len(toks) for w in want):
                raise ValueError(f"sequence {s!r}: empty portion or wanted place outside it")
            if self._len.get(s, 0) + len(toks) > self.engine.max_seq_len:
                raise ValueError(f"sequence {s!r} would exceed {self.engine.max_seq_len} positions")
        new = [s for s, _, _ in entries if s not in self._slot]
        if len(new) > len(self._free):
            raise RuntimeError(f"{len(new)} new sequences but {len(self._free)} free slots")
        for s in new:
            self._admit(s)
        # a decode step runs every slot up to the highest: all live ones must be in it (idle slots take a dummy token at position 0)
        single = [i for i, (s, t, _) in enumerate(entries) if len(t) == 1 and self._len[s] > 0]
        if {entries[i][0] for i in single} != set(self._slot):
            single = []
        out: list[np.ndarray | None] = [None] * len(entries)
        many = [i for i in range(len(entries)) if i not in set(single)]
        if many:
            part = [entries[i] for i in many]
            order = [sorted({int(x) for x in w}) for _, _, w in part]
            got = self.engine.prefill_batch([t for _, t, _ in part], [self._slot[s] for s, _, _ in part], [self._len[s] for s, _, _ in part], want=order)
            at = 0
            for i, o, (_, _, w) in zip(many, order, part):
                out[i] = got[at:at + len(o)][[o.index(int(x)) for x in w]] if len(w) else got[:0]
                at += len(o)
        if single:
            rows = 1 + max(self._slot.values())
            tok, pos = np.zeros(rows, np.int32), np.zeros(rows, np.int32)
            for i in single:
                s = self._slot[entries[i][0]]
                tok[s], pos[s] = entries[i][1][0], self._len[entries[i][0]]
            self.engine.set_state(tok, pos)
            self.engine.decode_step(rows)
            logits = self.engine.logits(rows).to_numpy() if any(len(entries[i][2]) for i in single) else None
            for i in single:
                s, _, w = entries[i]
                out[i] = logits[[self._slot[s]] * len(w)] if len(w) else np.empty((0, self.engine.config["vocab_size"]), np.float32)
        for s, toks, _ in entries:
            self._len[s] += len(toks)
        return out

    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int, *, eos_token_id: int | None = None, temperature: float = 0.0,
                 top_k: int = 0, top_p: float = 1.0, seed: int | None = None) -> list[list[int]]:
        """Prompt + generated tokens of every prompt; temperature 0 is greedy (lowest index on ties)."""
        from pygpukit_amd.llm.sampling import sample_token

        if self._slot:
            raise RuntimeError("generate() needs an idle scheduler")
        rng_state = np.random.get_state()
        if seed is not None:
            np.random.seed(seed)

        def pick(row: np.ndarray) -> int:
            return int(np.argmax(row)) if temperature == 0 else sample_token(row, temperature, top_k, top_p)

        out = [[int(t) for t in p] for p in prompts]
        waiting = list(range(len(prompts)))[::-1]
        done_at = [len(p) + max_new_tokens for p in prompts]
        try:
            active: list[int] = []
            while waiting or active:
                # one decode step for everything that lives, then admit into the slots that are free
                entries = [(i, [out[i][-1]], [0]) for i in active]
                fresh = [waiting.pop() for _ in range(min(len(waiting), len(self._free)))]
                fresh = [i for i in fresh if max_new_tokens > 0]
                if entries:
                    for (i, _, _), lg in zip(entries, self.step(entries)):
                        out[i].append(pick(lg[0]))
                if fresh:
                    for i, lg in zip(fresh, self.step([(i, out[i], [len(out[i]) - 1]) for i in fresh])):
                        out[i].append(pick(lg[0]))
                still = []
                for i in active + fresh:
                    if len(out[i]) >= done_at[i] or (eos_token_id is not None and out[i][-1] == eos_token_id):
                        self.release(i)
                    else:
                        still.append(i)
                active = still
        finally:
            for s in list(self._slot):
                self.release(s)
            if seed is not None:
                np.random.set_state(rng_state)
        return out


__all__ = ["BatchScheduler"]
