"""Throughput of architectures side by side at equal layer sizes.

bf16 weights everywhere, random; prefill (whole prompt, all logits) and
graph-captured greedy decode at a given context length.  All models are
resident and timed in turn, `repeats` times each; the best time counts.
"""
from __future__ import annotations

import time

import torch

from ..api import build_model
from ..models.graph import GraphDecoder
from ..models.llama import LlamaConfig
from ..models.rapivik import RapivikConfig
from ..models.zatasun import ZatasunConfig
from .decode import _fast_random_init

# alike in width and in the parameters a token meets; depth and vocab cut so that a run takes seconds
SIZES = {
    "2k": dict(
        llama=lambda n: LlamaConfig(
            vocab_size=32000, hidden_size=2048, intermediate_size=8192,
            n_layers=n, n_heads=16, n_kv_heads=4, head_dim=128),
        rapivik=lambda n: RapivikConfig.sized_1b(n_layers=n),
        zatasun=lambda n: ZatasunConfig.sized_1b(n_layers=n)),
    "4k": dict(
        llama=lambda n: LlamaConfig(
            vocab_size=32000, hidden_size=4096, intermediate_size=14336,
            n_layers=n, n_heads=32, n_kv_heads=8, head_dim=128),
        rapivik=lambda n: RapivikConfig.sized_8b(n_layers=n, vocab=32000),
        zatasun=lambda n: ZatasunConfig.sized_8b(n_layers=n, vocab=32000)),
    "tiny-debug": dict(
        llama=lambda n: LlamaConfig.tiny(n_layers=n),
        rapivik=lambda n: RapivikConfig.tiny(n_layers=n),
        zatasun=lambda n: ZatasunConfig.tiny(n_layers=n)),
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


def layer_params(model) -> tuple:
    """(all, met by one token) parameters of the layers."""
    total = active = 0
    for name, p in model.named_parameters():
        if name.startswith(("embed", "bigram", "lm_head")):
            continue
        total += p.numel()
        part = 1.0
        if name.endswith((".gate_up", ".down")):     # stacked experts
            moe = model.get_submodule(name.rpartition(".")[0])
            part = moe.top / moe.experts
        active += p.numel() * part
    return total, active


def compare(size: str, n_layers: int, models=("llama", "rapivik"),
            steps: int = 64, repeats: int = 3, prefill=PREFILL,
            decode=DECODE):
    """Yields one dict per (phase, shape) with every model's tokens/s; ratio
    is the last one's to the first one's."""
    built = {k: _build(SIZES[size][k](n_layers), "cuda") for k in models}
    params = {k: [round(v / 1e6) for v in layer_params(m)]
              for k, m in built.items()}
    for phase, shapes in (("prefill", prefill), ("decode", decode)):
        for b, s in shapes:
            row = {"size": size, "layers": n_layers, "phase": phase,
                   "batch": b, "length": s, "mparams_all_active": params}
            for name, m in built.items():
                row[name] = round(
                    prefill_tok_s(m, b, s, repeats) if phase == "prefill"
                    else decode_tok_s(m, b, s, steps, repeats), 1)
                torch.cuda.empty_cache()
            row["ratio"] = round(row[models[-1]] / row[models[0]], 3)
            yield row
