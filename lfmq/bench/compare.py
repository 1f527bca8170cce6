"""Throughput of one architecture beside another at equal layer sizes.

bf16 weights on both sides, random; prefill (whole prompt, all logits) and
graph-captured greedy decode at a given context length.  Both models are
resident and timed in turn, `repeats` times each; the best time counts.
"""
from __future__ import annotations

import time

import torch

from ..api import build_model
from ..models.graph import GraphDecoder
from ..models.llama import LlamaConfig
from ..models.rapivik import RapivikConfig
from .decode import _fast_random_init

# width-alike pairs; depth and vocab cut so that a run takes seconds
SIZES = {
    "2k": dict(
        llama=lambda n: LlamaConfig(
            vocab_size=32000, hidden_size=2048, intermediate_size=8192,
            n_layers=n, n_heads=16, n_kv_heads=4, head_dim=128),
        rapivik=lambda n: RapivikConfig.sized_1b(n_layers=n)),
    "4k": dict(
        llama=lambda n: LlamaConfig(
            vocab_size=32000, hidden_size=4096, intermediate_size=14336,
            n_layers=n, n_heads=32, n_kv_heads=8, head_dim=128),
        rapivik=lambda n: RapivikConfig.sized_8b(n_layers=n, vocab=32000)),
    "tiny-debug": dict(
        llama=lambda n: LlamaConfig.tiny(n_layers=n),
        rapivik=lambda n: RapivikConfig.tiny(n_layers=n)),
}
PREFILL = ((1, 2048), (1, 8192), (8, 1024))      # batch, prompt
DECODE = ((1, 1024), (1, 8192), (16, 1024), (64, 2048))


def _build(cfg, device):
    m = build_model(cfg).to_empty(device=device)
    return _fast_random_init(m, 0)


def _timed(fn) -> float:
    torch.cuda.synchronize()
    t = time.perf_counter()
    fn()
    torch.cuda.synchronize()
    return time.perf_counter() - t


@torch.no_grad()
def prefill_tok_s(model, batch: int, prompt: int, repeats: int) -> float:
    ids = torch.randint(0, model.cfg.vocab_size, (batch, prompt),
                        device="cuda")
    cache = model.make_cache(batch, max_seq=prompt + 8, device="cuda")
    best = float("inf")
    for _ in range(repeats + 1):                 # the first one warms up
        cache.reset()
        best = min(best, _timed(lambda: model(ids, cache)))
    return batch * prompt / best


@torch.no_grad()
def decode_tok_s(model, batch: int, context: int, steps: int,
                 repeats: int) -> float:
    total = steps * (repeats + 1)
    dec = GraphDecoder(model, batch, max_seq=context + total + 8,
                       max_new_tokens=total + 4)
    dec.prefill(torch.randint(0, model.cfg.vocab_size, (batch, context),
                              device="cuda"))
    dec.decode(steps)                            # capture and warm-up
    best = min(_timed(lambda: dec.decode(steps)) for _ in range(repeats))
    return batch * steps / best


def compare(size: str, n_layers: int, steps: int = 64, repeats: int = 3,
            prefill=PREFILL, decode=DECODE):
    """Yields one dict per (phase, shape) with both models' tokens/s."""
    models = {k: _build(f(n_layers), "cuda") for k, f in SIZES[size].items()}
    params = {k: sum(p.numel() for n, p in m.named_parameters()
                     if not n.startswith(("embed", "bigram", "lm_head"))) / 1e6
              for k, m in models.items()}          # of the layers
    for phase, shapes in (("prefill", prefill), ("decode", decode)):
        for b, s in shapes:
            row = {"size": size, "layers": n_layers, "phase": phase,
                   "batch": b, "length": s,
                   "mparams": {k: round(v) for k, v in params.items()}}
            for name, m in models.items():
                row[name] = round(
                    prefill_tok_s(m, b, s, repeats) if phase == "prefill"
                    else decode_tok_s(m, b, s, steps, repeats), 1)
                torch.cuda.empty_cache()
            row["ratio"] = round(row["rapivik"] / row["llama"], 3)
            yield row
