"""Shared eager autoregressive generation for all model families.

Greedy by default (the BASELINE decode metric is greedy); a
GenerationConfig adds temperature sampling and eos early-stop for
serving (lfmq/obs/serve.py).  The hipGraph decode path
(lfmq/models/graph.py) stays greedy-only — sampling there runs through
the on-device argmax kernel.
"""
from __future__ import annotations

from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import torch

from ..config import GenerationConfig
from ..ops import functional as F


def _next_token(logits_last: torch.Tensor, gc: Optional[GenerationConfig],
                generator: Optional[torch.Generator]) -> torch.Tensor:
    """logits_last [b, vocab] -> token [b, 1]."""
    if gc is None or gc.greedy:
        return F.greedy_sample(logits_last).unsqueeze(1)
    probs = torch.softmax(logits_last.float()
                          / max(gc.temperature, 1e-5), dim=-1)
    return torch.multinomial(probs, 1, generator=generator)


@torch.no_grad()
def autoregressive_generate(model, input_ids: torch.Tensor,
                            max_new_tokens: int = 32, cache=None,
                            gen_cfg: Optional[GenerationConfig] = None,
                            generator: Optional[torch.Generator] = None
                            ) -> torch.Tensor:
    """Prefill + token-by-token decode through model.forward.

    gen_cfg.max_new_tokens overrides max_new_tokens when set;
    gen_cfg.eos_token_id stops early once EVERY row has emitted eos
    (the returned tensor ends at that step — rows that finished earlier
    keep decoding until the slowest row is done, as is standard for
    batched eager generation)."""
    if gen_cfg is not None and gen_cfg.max_new_tokens:
        max_new_tokens = gen_cfg.max_new_tokens
    b, s = input_ids.shape
    if cache is None:
        cache = model.make_cache(b, max_seq=s + max_new_tokens + 8)
    eos = gen_cfg.eos_token_id if gen_cfg is not None else None
    done = torch.zeros(b, dtype=torch.bool, device=input_ids.device)

    logits = model.forward(input_ids, cache)
    out = [input_ids]
    tok = _next_token(logits[:, -1], gen_cfg, generator)
    for _ in range(max_new_tokens - 1):
        out.append(tok)
        if eos is not None:
            done |= (tok.squeeze(1) == eos)
            if bool(done.all()):
                return torch.cat(out, dim=1)
        logits = model.forward(tok, cache)
        tok = _next_token(logits[:, -1], gen_cfg, generator)
    out.append(tok)
    return torch.cat(out, dim=1)


class PackedStepper:
    """Batches requests of unequal length through a packed-batch model: one
    cache, a slot per live request, one model step per call."""

    def __init__(self, model, max_tokens: int, n_slots: int = 1):
        self.model = model
        self.device = model.norm.weight.device
        self.cache = model.make_cache(n_slots, max_seq=max_tokens)
        self.slots: Dict[Hashable, int] = {}

    @torch.no_grad()
    def step(self, entries: Sequence[Tuple[Hashable, Sequence[int],
                                           Sequence[int]]]) -> torch.Tensor:
        """entries: (request id, its next tokens, the places among them
        whose logits are wanted).  Returns the wanted logits, in order."""
        vocab = self.model.cfg.vocab_size
        ids = [e[0] for e in entries]
        if len(set(ids)) != len(ids):
            raise ValueError("a request may appear once in a step")
        flat: List[int] = []
        select: List[int] = []
        for rid, toks, want in entries:
            if not toks:
                raise ValueError(f"request {rid!r} brings no token")
            if min(toks) < 0 or max(toks) >= vocab:
                raise ValueError(f"request {rid!r}: token id out of range")
            if want and (min(want) < 0 or max(want) >= len(toks)):
                raise ValueError(f"request {rid!r}: place out of range")
            select += [len(flat) + w for w in want]
            flat += toks
        new = [r for r in ids if r not in self.slots]
        if len(new) > self.cache.free_slots:
            self.cache.reserve(len(self.slots) + len(new))
        for r in new:
            self.slots[r] = self.cache.alloc()
        batch = self.cache.batch([self.slots[r] for r in ids],
                                 [len(e[1]) for e in entries])
        return self.model.forward_tokens(
            torch.tensor(flat, device=self.device), batch, self.cache,
            torch.tensor(select, dtype=torch.int64, device=self.device))

    def end(self, ids: Sequence[Hashable]) -> None:
        """These requests are finished; their slots are given back."""
        self.cache.free([self.slots.pop(r) for r in ids])


@torch.no_grad()
def generate_batch(model, prompts: Sequence[Sequence[int]],
                   max_new_tokens: int = 32,
                   gen_cfg: Optional[GenerationConfig] = None,
                   generator: Optional[torch.Generator] = None
                   ) -> List[List[int]]:
    """Generate for prompts of unequal length in one batch (models with
    packed batches).  A request that emits eos leaves the batch and gives
    its slot back; the others go on.  Returns prompt + new tokens each."""
    if gen_cfg is not None and gen_cfg.max_new_tokens:
        max_new_tokens = gen_cfg.max_new_tokens
    eos = gen_cfg.eos_token_id if gen_cfg is not None else None
    out = [list(p) for p in prompts]
    st = PackedStepper(model, max(map(len, out)) + max_new_tokens, len(out))
    entries = [(i, p, [len(p) - 1]) for i, p in enumerate(out)]
    for _ in range(max_new_tokens):
        tok = _next_token(st.step(entries), gen_cfg,
                          generator).squeeze(1).tolist()
        done = []
        live = [e[0] for e in entries]
        for i, t in zip(live, tok):
            out[i].append(t)
            if t == eos:
                done.append(i)
        st.end(done)
        entries = [(i, out[i][-1:], [0]) for i in live if i not in done]
        if not entries:
            break
    return out
