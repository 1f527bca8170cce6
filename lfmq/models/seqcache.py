"""Cache and state manager for packed, unequal sequences.

A SequenceCache has `n_slots` slots; a slot holds everything one live
sequence carries from step to step: its length, its previous token, and
what each layer run declares through its mixer's `state_spec` (a ring of
latent rows, keys and values, a recurrent state, ...).  Slots are handed out and given
back; a slot of length 0 is fresh whatever its tensors hold, so giving one
back costs no clearing pass.

A StepBatch describes one step: which slots take part and how many tokens
each brings, packed without padding.  Lengths live on the device (kernels
read them; a captured decode step advances them itself) and are mirrored
on the host for bounds checks.
"""
from __future__ import annotations

from types import SimpleNamespace
from typing import Dict, List, Sequence

import torch


class StepBatch:
    """counts[i] tokens of slot slots[i], rows packed in that order."""

    def __init__(self, slots: Sequence[int], counts: Sequence[int],
                 len0: Sequence[int], device):
        if len(slots) != len(counts) or not slots:
            raise ValueError("a step needs slots, and one count for each")
        if min(counts) < 1:
            raise ValueError("every sequence of a step brings a token")
        if len(set(slots)) != len(slots):
            raise ValueError("a slot may appear once in a step")
        self.device = device
        self.slot_ids, self.counts = list(slots), list(counts)
        self.len0 = list(len0)
        self.b, self.n = len(slots), sum(counts)
        cu, seq = [0], []
        for i, c in enumerate(counts):
            cu.append(cu[-1] + c)
            seq += [i] * c
        self.single = self.n == self.b          # one token each
        self.max_count = max(counts)
        self.last_rows_host = [c - 1 for c in cu[1:]]
        t = self._dev(seq + cu + self.slot_ids)
        self.seq = t[:self.n]
        self.cu = t[self.n:self.n + self.b + 1]
        self.slots = t[self.n + self.b + 1:]
        self._rows: Dict[int, SimpleNamespace] = {}
        self._chunks: Dict[int, tuple] = {}

    def _dev(self, ints) -> torch.Tensor:
        return torch.tensor(ints, dtype=torch.int32).to(self.device)

    def view(self, cache):
        return self.seq, self.cu, self.slots, cache.lens

    def key_rows(self, window: int) -> SimpleNamespace:
        """Layout of a key buffer whose sequences start with the cached
        tokens that the step's windows reach back to:
        own (first own row), prior (cached rows before it), total."""
        r = self._rows.get(window)
        if r is None:
            own, prior, at = [], [], 0
            for c, n0 in zip(self.counts, self.len0):
                p = min(n0, window - 1)
                own.append(at + p)
                prior.append(p)
                at += p + c
            t = self._dev(own + prior)
            r = SimpleNamespace(own=t[:self.b], prior=t[self.b:], total=at,
                                any_prior=any(prior))
            self._rows[window] = r
        return r

    def chunks(self, size: int):
        """(first chunk of every sequence, chunks in all) when sequences
        are cut into chunks of `size` tokens."""
        if size not in self._chunks:
            base, at = [], 0
            for c in self.counts:
                base.append(at)
                at += -(-c // size)
            self._chunks[size] = (self._dev(base), at)
        return self._chunks[size]


class SequenceCache:
    def __init__(self, specs: List[dict], n_slots: int, max_seq: int, device):
        """specs: per layer run, name -> (shape per slot, dtype) and, for
        rows that a position owns and writes before anyone reads them,
        "by_position": nothing of theirs has to be kept apart."""
        self.specs, self.max_seq = specs, max_seq
        self.device = torch.device(device)
        self.n_slots = n_slots
        i32 = dict(dtype=torch.int32, device=self.device)
        self.lens = torch.zeros(n_slots, **i32)
        self.prev = torch.zeros(n_slots, **i32)
        self.turn = torch.zeros(n_slots, **i32)
        self.layers = [{k: torch.zeros((n_slots, *shape), dtype=dt,
                                       device=self.device)
                        for k, (shape, dt, *_) in spec.items()}
                       for spec in specs]
        self.lens_host = [0] * n_slots
        self._free = list(range(n_slots - 1, -1, -1))
        self._decode: Dict[int, StepBatch] = {}

    # ---- slots ----------------------------------------------------------
    def alloc(self) -> int:
        if not self._free:
            raise RuntimeError(f"all {self.n_slots} cache slots are in use")
        return self._free.pop()

    def free(self, slots: Sequence[int]) -> None:
        slots = list(slots)
        for s in slots:
            if s in self._free:
                raise ValueError(f"slot {s} is free already")
            self.lens_host[s] = 0
            self._free.append(s)
        if slots:
            self.lens[torch.tensor(slots, device=self.device)] = 0

    @property
    def free_slots(self) -> int:
        return len(self._free)

    def reserve(self, n_slots: int) -> None:
        """Grow to at least n_slots; live slots keep what they hold."""
        add = n_slots - self.n_slots
        if add <= 0:
            return

        def grown(t):
            new = torch.zeros((n_slots, *t.shape[1:]), dtype=t.dtype,
                              device=t.device)
            new[:t.shape[0]] = t
            return new

        self.lens, self.prev, self.turn = map(
            grown, (self.lens, self.prev, self.turn))
        self.layers = [{k: grown(t) for k, t in st.items()}
                       for st in self.layers]
        self.lens_host += [0] * add
        self._free = list(range(n_slots - 1, self.n_slots - 1, -1)) + self._free
        self.n_slots = n_slots

    # ---- steps ----------------------------------------------------------
    def batch(self, slots: Sequence[int], counts: Sequence[int]) -> StepBatch:
        len0 = [self.lens_host[s] for s in slots]
        for n0, c in zip(len0, counts):
            if n0 + c > self.max_seq:
                raise RuntimeError(
                    f"KV cache overflow: {n0 + c} > {self.max_seq}")
        return StepBatch(slots, counts, len0, self.device)

    def decode_batch(self, b: int) -> StepBatch:
        """One token for each of slots 0..b-1, at addresses that stay the
        same from step to step (hipGraph capture)."""
        if b not in self._decode:
            self._decode[b] = StepBatch(range(b), [1] * b, [1] * b,
                                        self.device)
        return self._decode[b]

    def advance(self, tokens: torch.Tensor, batch: StepBatch) -> None:
        from ..ops import functional as F
        F.seq_advance(tokens, batch, self)
        for s, c in zip(batch.slot_ids, batch.counts):
            self.lens_host[s] += c

    # ---- the equal-batch interface of KVCache ---------------------------
    @property
    def seq_len(self) -> int:
        return max(self.lens_host)

    def reset(self) -> None:
        self.lens.zero_()
        self.lens_host = [0] * self.n_slots
        self._free = list(range(self.n_slots - 1, -1, -1))

    def replayed(self, n: int) -> None:
        """n captured decode steps ran on the device for slots 0..b-1."""
        self.lens_host = [x + n for x in self.lens_host]

    def snapshot(self):
        """Everything a warm-up step would change."""
        return ([t.clone() for t in (self.lens, self.prev, self.turn)],
                [{k: t.clone() for k, t in st.items()
                  if "by_position" not in spec[k][2:]}
                 for spec, st in zip(self.specs, self.layers)],
                list(self.lens_host))

    def restore(self, snap) -> None:
        for t, old in zip((self.lens, self.prev, self.turn), snap[0]):
            t.copy_(old)
        for st, old in zip(self.layers, snap[1]):
            for k in old:
                st[k].copy_(old[k])
        self.lens_host = list(snap[2])
