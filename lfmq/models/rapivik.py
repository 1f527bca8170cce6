"""Rapivik: a decoder of recurrent (mLSTM) and windowed latent-attention
layers on an fp32 residual stream, with a hashed bigram embedding.

The configuration lists the layers one by one, each with its mixer's sizes
and an optional feed-forward; a layer may run another layer's weights with
a state of its own.  The model is a list of lfmq.models.mixers blocks over
a SequenceCache, in bf16 or fp32.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Dict, List

import torch
import torch.nn as nn

from ..ops import functional as F
from .mixers import (DenseMLP, LatentAttention, MixerBlock, MLSTMMixer,
                     ResidualNorm)
from .packed import PackedCausalLM
from .seqcache import SequenceCache, StepBatch

MIXER_TYPES = ("mlstm", "latent_attention")


@dataclass
class RapivikConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]
    bigram: dict                     # buckets, mul_prev, mul_cur
    rms_eps: float = 1e-6
    max_seq: int = 131072
    arch: str = "rapivik"

    def __post_init__(self):
        for i, e in enumerate(self.layers):
            if e["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            mlp = e.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp!r}")
            j = self.owner(i)
            if j != i and any(e.get(k) != self.layers[j].get(k)
                              for k in ("type", "mixer", "mlp")):
                raise ValueError(f"layer {i} differs from layer {j}, whose "
                                 "weights it uses")

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i runs with."""
        seen = set()
        while self.layers[i].get("weights_of") is not None:
            if i in seen:
                raise ValueError(f"layer {i}: circular weights_of")
            seen.add(i)
            i = self.layers[i]["weights_of"]
            if not 0 <= i < len(self.layers):
                raise ValueError(f"weights_of names layer {i}")
        return i

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @n_layers.setter
    def n_layers(self, n: int) -> None:
        """Repeat or cut the layer pattern (depth overrides of the tools)."""
        base = [{k: v for k, v in e.items() if k != "weights_of"}
                for e in self.layers]
        self.layers = [copy.deepcopy(base[i % len(base)]) for i in range(n)]

    @classmethod
    def from_dict(cls, d: dict) -> "RapivikConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=copy.deepcopy(d["layers"]),
                   bigram=dict(d["embedding"]["bigram"]),
                   rms_eps=d["norm"]["eps"],
                   **({"max_seq": d["max_seq"]} if "max_seq" in d else {}))

    def to_dict(self) -> dict:
        return {"arch": self.arch, "architecture": "Rapivik",
                "vocab": self.vocab_size, "width": self.hidden_size,
                "layers": copy.deepcopy(self.layers),
                "embedding": {"bigram": dict(self.bigram)},
                "norm": {"eps": self.rms_eps}, "max_seq": self.max_seq}

    @classmethod
    def pattern(cls, width: int, heads: int, dim: int, vdim: int, ff: int,
                lat_heads: int, lat_dim: int, rot: int, lat_vdim: int,
                q_rank: int, kv_rank: int, window: int, vocab: int,
                n_layers: int, **kw) -> "RapivikConfig":
        """mLSTM and latent-attention layers in turn, each with a
        feed-forward."""
        rec = {"type": "mlstm", "mlp": {"kind": "dense", "ff": ff},
               "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                         "gate_cap": 15.0}}
        att = {"type": "latent_attention",
               "mlp": {"kind": "dense", "ff": ff},
               "mixer": {"heads": lat_heads, "dim": lat_dim, "rot_dim": rot,
                         "vdim": lat_vdim, "q_rank": q_rank,
                         "kv_rank": kv_rank, "mask": {"size": window},
                         "rot": {"base": 500000.0, "dims": rot},
                         "scale": (lat_dim + rot) ** -0.5}}
        layers = [copy.deepcopy((rec, att)[i % 2]) for i in range(n_layers)]
        return cls(vocab_size=vocab, hidden_size=width, layers=layers,
                   bigram={"buckets": 4 * vocab - 1, "mul_prev": 1009,
                           "mul_cur": 31}, **kw)

    @classmethod
    def tiny(cls, **kw) -> "RapivikConfig":
        return cls.pattern(**{**dict(
            width=256, heads=2, dim=32, vdim=64, ff=512, lat_heads=2,
            lat_dim=32, rot=32, lat_vdim=64, q_rank=128, kv_rank=64,
            window=40, vocab=512, n_layers=4), **kw})

    @classmethod
    def sized_1b(cls, **kw) -> "RapivikConfig":
        return cls.pattern(**{**dict(
            width=2048, heads=4, dim=256, vdim=512, ff=8192, lat_heads=16,
            lat_dim=128, rot=64, lat_vdim=128, q_rank=768, kv_rank=512,
            window=1024, vocab=32000, n_layers=16), **kw})

    @classmethod
    def sized_8b(cls, **kw) -> "RapivikConfig":
        return cls.pattern(**{**dict(
            width=4096, heads=8, dim=256, vdim=512, ff=14336, lat_heads=32,
            lat_dim=128, rot=64, lat_vdim=128, q_rank=1536, kv_rank=512,
            window=4096, vocab=128256, n_layers=32), **kw})


def _make_mixer(e: dict, width: int, eps: float, dtype) -> nn.Module:
    m = e["mixer"]
    if e["type"] == "mlstm":
        return MLSTMMixer(width, m["heads"], m["dim"], m["vdim"],
                          m["gate_cap"], eps, dtype)
    return LatentAttention(width, m["heads"], m["dim"], m["rot_dim"],
                           m["vdim"], m["q_rank"], m["kv_rank"],
                           m["mask"]["size"], m["scale"], m["rot"]["base"],
                           m["rot"]["dims"], eps, dtype)


class RapivikForCausalLM(PackedCausalLM):
    def __init__(self, cfg: RapivikConfig, dtype=torch.bfloat16):
        super().__init__(cfg, dtype)
        w, eps = cfg.hidden_size, cfg.rms_eps
        self.embed_tokens = nn.Embedding(cfg.vocab_size, w, dtype=dtype)
        # one row per bucket, and one for "no previous token"
        self.bigram = nn.Embedding(cfg.bigram["buckets"] + 1, w, dtype=dtype)
        self.blocks = nn.ModuleDict()
        for i, e in enumerate(cfg.layers):
            if cfg.owner(i) == i:
                mlp = None if e.get("mlp") is None else \
                    DenseMLP(w, e["mlp"]["ff"], dtype)
                self.blocks[f"l{i}"] = MixerBlock(
                    _make_mixer(e, w, eps, dtype), mlp, w, eps, True, dtype)
        self.order = [f"l{cfg.owner(i)}" for i in range(cfg.n_layers)]
        self.norm = ResidualNorm(w, eps, True, dtype)
        self.lm_head = nn.Linear(w, cfg.vocab_size, bias=False, dtype=dtype)

    def layer_mixers(self) -> list:
        return [self.blocks[b].mixer for b in self.order]

    def _run(self, tokens: torch.Tensor, batch: StepBatch,
             cache: SequenceCache, select=None, trace=None) -> torch.Tensor:
        x = F.bigram_embed(tokens, batch, cache, self.embed_tokens.weight,
                           self.bigram.weight, self.cfg.bigram["mul_prev"],
                           self.cfg.bigram["mul_cur"])
        y = None
        for name, state in zip(self.order, cache.layers):
            y = self.blocks[name](x, y, batch, cache, state)
            if trace is not None:
                trace.append(x + y.float())
        h, _ = self.norm(x, y)
        if select is not None:
            h = h[select]
            if h.shape[0] == 0:
                return h.new_empty(0, self.cfg.vocab_size)
        return self.lm_head(h)


# ---------------------------------------------------------------------------
# checkpoint names
# ---------------------------------------------------------------------------

def convert_state(cfg: RapivikConfig, src: Dict[str, torch.Tensor]
                  ) -> Dict[str, torch.Tensor]:
    """Checkpoint tensors (one per matrix) -> module parameters (fused)."""
    src = dict(src)
    out: Dict[str, torch.Tensor] = {}

    def cat(*names):
        return torch.cat([src.pop(n) for n in names])

    try:
        out["embed_tokens.weight"] = src.pop("embed")
        out["bigram.weight"] = src.pop("bigram")
        out["norm.weight"] = src.pop("final.norm")
        out["lm_head.weight"] = src.pop("head")
        for i, e in enumerate(cfg.layers):
            if cfg.owner(i) != i:
                continue
            m, o = f"l{i}.mix.", f"blocks.l{i}."
            out[o + "norm1.weight"] = src.pop(f"l{i}.norm1")
            if e["type"] == "mlstm":
                out[o + "mixer.in_proj.weight"] = cat(
                    m + "q", m + "k", m + "v", m + "g")
                out[o + "mixer.gate_w"] = cat(m + "i", m + "f")
                out[o + "mixer.gate_b"] = cat(m + "i.b", m + "f.b")
                out[o + "mixer.norm_w"] = src.pop(m + "norm")
            else:
                out[o + "mixer.in_proj.weight"] = cat(
                    m + "dq", m + "dkv", m + "g")
                out[o + "mixer.q_norm"] = src.pop(m + "dq.norm")
                out[o + "mixer.kv_norm"] = src.pop(m + "dkv.norm")
                out[o + "mixer.q_up.weight"] = src.pop(m + "uq")
                out[o + "mixer.kv_up"] = cat(m + "uk", m + "uv")
                out[o + "mixer.sink"] = src.pop(m + "sink")
            out[o + "mixer.o_proj.weight"] = src.pop(m + "o")
            if e.get("mlp") is not None:
                p = f"l{i}.mlp."
                out[o + "norm2.weight"] = src.pop(f"l{i}.norm2")
                out[o + "mlp.gate_up_proj.weight"] = cat(p + "gate", p + "up")
                out[o + "mlp.down_proj.weight"] = src.pop(p + "down")
    except KeyError as err:
        raise KeyError(f"checkpoint lacks tensor {err.args[0]!r}") from None
    if src:
        raise KeyError(f"checkpoint has unknown tensors {sorted(src)}")
    return out
