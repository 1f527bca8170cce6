"""Base of the models that run packed batches over a SequenceCache: cache
construction, the step function and its captured form.  A model adds

    layer_mixers()     the mixer of every layer run, in order
    _run(tokens, batch, cache, select, trace) -> logits
    norm               a module whose weight names the device
"""
from __future__ import annotations

from typing import Optional, Sequence

import torch
import torch.nn as nn

from ..ops import functional as F
from .seqcache import SequenceCache, StepBatch


class PackedCausalLM(nn.Module):
    packed = True            # takes unequal sequences in one batch

    def __init__(self, cfg, dtype):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype

    def fp32_names(self) -> set:
        """Parameters that keep 32 bits whatever the model's dtype."""
        return {n for n, p in self.named_parameters()
                if p.dtype == torch.float32}

    @torch.no_grad()
    def init_random(self, seed: int = 0):
        g = torch.Generator().manual_seed(seed)
        for p in self.parameters():
            t = torch.randn(p.shape, generator=g, dtype=torch.float32) * 0.02
            # 1-D parameters start at what they stand for (0 or 1)
            p.data.copy_((p.data.float().cpu() + t if p.dim() == 1 else t)
                         .to(p.dtype))
        return self

    def make_cache(self, batch: int, max_seq: Optional[int] = None,
                   device=None) -> SequenceCache:
        dev = device or self.norm.weight.device
        max_seq = max_seq or self.cfg.max_seq
        specs = [m.state_spec(max_seq) for m in self.layer_mixers()]
        return SequenceCache(specs, batch, max_seq, dev)

    def _check(self, tokens: torch.Tensor) -> None:
        if not tokens.is_cuda:
            raise RuntimeError(f"{self.cfg.arch} runs on a GPU device only")

    def forward_tokens(self, tokens: torch.Tensor, batch: StepBatch,
                       cache: SequenceCache, select=None,
                       trace: Optional[list] = None) -> torch.Tensor:
        """One step of packed sequences: tokens [N] -> logits of all rows,
        or of the `select`ed ones (int64 row numbers).  Advances the cache.
        trace collects the residual stream after every layer run."""
        self._check(tokens)
        logits = self._run(tokens, batch, cache, select, trace)
        cache.advance(tokens, batch)
        return logits

    def forward(self, input_ids: torch.Tensor, cache: SequenceCache,
                lengths: Optional[Sequence[int]] = None) -> torch.Tensor:
        """input_ids [b, s] on slots 0..b-1 -> logits [b, s, vocab].  With
        lengths, row i brings its first lengths[i] tokens and the result is
        the last one's logits, [b, 1, vocab]."""
        b, s = input_ids.shape
        if lengths is None:
            batch = cache.batch(range(b), [s] * b)
            return self.forward_tokens(input_ids.reshape(-1).contiguous(),
                                       batch, cache).view(b, s, -1)
        batch = cache.batch(range(b), lengths)
        tok = torch.cat([input_ids[i, :n] for i, n in enumerate(lengths)])
        last = torch.tensor(batch.last_rows_host, device=tok.device)
        return self.forward_tokens(tok, batch, cache, last).unsqueeze(1)

    def forward_decode_step(self, input_ids, cache, state, max_seq):
        """hipGraph-capturable: [b, 1] ids -> [b, 1, vocab].  Positions come
        from the cache's own device lengths (state and max_seq belong to
        the scalar-position models)."""
        batch = cache.decode_batch(input_ids.shape[0])
        tok = input_ids.reshape(-1).contiguous()
        self._check(tok)
        logits = self._run(tok, batch, cache)
        F.seq_advance(tok, batch, cache)
        return logits.unsqueeze(1)

    @torch.no_grad()
    def generate(self, input_ids, max_new_tokens: int = 32, cache=None,
                 gen_cfg=None, generator=None):
        from .generation import autoregressive_generate
        return autoregressive_generate(self, input_ids, max_new_tokens,
                                       cache, gen_cfg, generator)
