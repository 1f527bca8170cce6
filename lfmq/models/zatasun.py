"""Zatasun: a decoder whose layers run grouped-query attention and a gated
linear recurrence side by side on an fp32 residual stream, with norms on the
sublayers' outputs and dense or mixture-of-experts feed-forwards.

The configuration lists the layers one by one.  The model is a list of
lfmq.models.mixers blocks over a SequenceCache, in bf16 or fp32.  The output
projection is the embedding table.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from ..ops import functional as F
from .mixers import (ClampedGLU, DenseMLP, ExpertMLP, GatedLRU,
                     GroupedAttention, ParallelMixer, PostNorm, PostNormBlock)
from .packed import PackedCausalLM
from .seqcache import SequenceCache, StepBatch

MIXER_TYPES = ("parallel",)
MLP_KINDS = ("dense", "moe")
GLU_ALPHA, GLU_BETA = 1.702, 1.0         # the experts' activation


@dataclass
class ZatasunConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]
    logit_scale: float = 1.0
    rms_eps: float = 1e-5
    max_seq: int = 131072
    arch: str = "zatasun"

    def __post_init__(self):
        if not self.layers:
            raise ValueError("a model needs layers")
        for i, e in enumerate(self.layers):
            if e["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            mlp = e.get("mlp")
            if mlp is not None and mlp.get("kind") not in MLP_KINDS:
                raise ValueError(f"layer {i}: unknown feed-forward {mlp!r}")

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @n_layers.setter
    def n_layers(self, n: int) -> None:
        """Repeat or cut the layer pattern (depth overrides of the tools)."""
        base = self.layers
        self.layers = [copy.deepcopy(base[i % len(base)]) for i in range(n)]

    @classmethod
    def from_dict(cls, d: dict) -> "ZatasunConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=copy.deepcopy(d["layers"]),
                   logit_scale=d["logit_scale"], rms_eps=d["norm"]["eps"],
                   **({"max_seq": d["max_seq"]} if "max_seq" in d else {}))

    def to_dict(self) -> dict:
        return {"arch": self.arch, "architecture": "Zatasun",
                "vocab": self.vocab_size, "width": self.hidden_size,
                "layers": copy.deepcopy(self.layers),
                "logit_scale": self.logit_scale,
                "norm": {"eps": self.rms_eps}, "max_seq": self.max_seq}

    @classmethod
    def pattern(cls, width: int, heads: int, kv_heads: int, dim: int,
                vdim: int, rec_width: int, blocks: int, ff: int, experts: int,
                top: int, expert_ff: int, shared_ff: int, vocab: int,
                n_layers: int, **kw) -> "ZatasunConfig":
        """Dense and expert feed-forwards in turn."""
        mixer = {
            "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim, "scale": dim ** -0.5,
                     "rot": {"base": 500000.0, "dims": dim,
                             "scaling": {"factor": 8.0, "low": 1.0,
                                         "high": 4.0, "original": 8192}}},
            "right": {"width": rec_width, "blocks": blocks, "conv": 4},
            "left_scale": 1.0, "right_scale": 1.0}
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "router": {"experts": experts, "top": top},
               "expert": {"ff": expert_ff, "limit": 7.0},
               "shared": {"ff": shared_ff, "limit": 7.0}}
        layers = [{"type": "parallel", "mixer": copy.deepcopy(mixer),
                   "mlp": copy.deepcopy((dense, moe)[i % 2])}
                  for i in range(n_layers)]
        return cls(vocab_size=vocab, hidden_size=width, layers=layers, **kw)

    @classmethod
    def tiny(cls, **kw) -> "ZatasunConfig":
        return cls.pattern(**{**dict(
            width=256, heads=4, kv_heads=2, dim=32, vdim=64, rec_width=256,
            blocks=2, ff=512, experts=8, top=2, expert_ff=128, shared_ff=256,
            vocab=512, n_layers=4), **kw})

    @classmethod
    def sized_1b(cls, **kw) -> "ZatasunConfig":
        return cls.pattern(**{**dict(
            width=2048, heads=16, kv_heads=4, dim=128, vdim=128,
            rec_width=2048, blocks=8, ff=8192, experts=16, top=2,
            expert_ff=2048, shared_ff=4096, vocab=32000, n_layers=16), **kw})

    @classmethod
    def sized_8b(cls, **kw) -> "ZatasunConfig":
        return cls.pattern(**{**dict(
            width=4096, heads=32, kv_heads=8, dim=128, vdim=128,
            rec_width=4096, blocks=16, ff=14336, experts=16, top=2,
            expert_ff=3584, shared_ff=7168, vocab=128256, n_layers=32), **kw})


def _make_mixer(m: dict, width: int, eps: float, dtype) -> nn.Module:
    a, r = m["left"], m["right"]
    rot = a["rot"]
    left = GroupedAttention(a["heads"], a["kv_heads"], a["dim"], a["vdim"],
                            a["scale"], rot["dims"], rot["base"],
                            rot.get("scaling"), eps, dtype)
    right = GatedLRU(r["width"], r["blocks"], r["conv"], dtype)
    return ParallelMixer(width, {"left": (left, m["left_scale"]),
                                 "right": (right, m["right_scale"])}, dtype)


def _make_mlp(m: Optional[dict], width: int, dtype) -> Optional[nn.Module]:
    if m is None:
        return None
    if m["kind"] == "dense":
        return DenseMLP(width, m["ff"], dtype)
    sh = m.get("shared")
    shared = None if sh is None else ClampedGLU(
        width, sh["ff"], sh["limit"], GLU_ALPHA, GLU_BETA, dtype)
    return ExpertMLP(width, m["router"]["experts"], m["router"]["top"],
                     m["expert"]["ff"], m["expert"]["limit"], GLU_ALPHA,
                     GLU_BETA, shared, dtype)


class ZatasunForCausalLM(PackedCausalLM):
    def __init__(self, cfg: ZatasunConfig, dtype=torch.bfloat16):
        super().__init__(cfg, dtype)
        w, eps = cfg.hidden_size, cfg.rms_eps
        self.embed_tokens = nn.Embedding(cfg.vocab_size, w, dtype=dtype)
        self.embed_norm = PostNorm(w, eps)
        self.blocks = nn.ModuleList(
            PostNormBlock(_make_mixer(e["mixer"], w, eps, dtype),
                          _make_mlp(e.get("mlp"), w, dtype), w, eps)
            for e in cfg.layers)
        self.norm = PostNorm(w, eps)

    def layer_mixers(self) -> list:
        return [b.mixer for b in self.blocks]

    def _run(self, tokens: torch.Tensor, batch: StepBatch,
             cache: SequenceCache, select=None, trace=None) -> torch.Tensor:
        table = self.embed_tokens.weight
        x, h = F.embed_norm(tokens, table, self.embed_norm.weight,
                            self.embed_norm.eps)
        final = len(self.blocks) - 1
        for i, (block, state) in enumerate(zip(self.blocks, cache.layers)):
            last = (self.norm, self.cfg.logit_scale) if i == final \
                else (None, 1.0)
            h = block(x, h, batch, cache, state, last)
            if trace is not None:
                trace.append(x.clone())
        if select is not None:
            h = h[select]
            if h.shape[0] == 0:
                return h.new_empty(0, self.cfg.vocab_size)
        return nn.functional.linear(h, table)


# ---------------------------------------------------------------------------
# checkpoint names
# ---------------------------------------------------------------------------

def convert_state(cfg: ZatasunConfig, src: Dict[str, torch.Tensor]
                  ) -> Dict[str, torch.Tensor]:
    """Checkpoint tensors (one per matrix) -> module parameters (fused)."""
    src = dict(src)
    out: Dict[str, torch.Tensor] = {}

    def cat(*names, dim=0):
        return torch.cat([src.pop(n) for n in names], dim)

    def attention(p, o):
        out[o + "q_norm"] = src.pop(p + "q.norm")
        out[o + "k_norm"] = src.pop(p + "k.norm")
        out[o + "sink"] = src.pop(p + "sink")

    def recurrence(p, o):
        out[o + "y_b"], out[o + "x_b"] = src.pop(p + "y.b"), src.pop(p + "x.b")
        out[o + "conv_w"] = src.pop(p + "conv").t().contiguous()
        out[o + "conv_b"] = src.pop(p + "conv.b")
        out[o + "gate_w"] = torch.stack([src.pop(p + "ra"),
                                         src.pop(p + "ri")], 1)
        out[o + "gate_b"] = torch.stack([src.pop(p + "ra.b"),
                                         src.pop(p + "ri.b")], 1)
        out[o + "lam"] = src.pop(p + "lam")

    def experts(p, o, m):
        names = [f"{p}e{e}." for e in range(m["router"]["experts"])]
        out[o + "gate_up"] = torch.stack([cat(n + "gate", n + "up")
                                          for n in names])
        out[o + "down"] = torch.stack([src.pop(n + "down") for n in names])
        s = p + "shared."
        if m.get("shared") is None:
            out[o + "router"] = src.pop(p + "router")
            return
        out[o + "router"] = cat(p + "router", s + "sg")
        out[o + "shared.gate_up_proj.weight"] = cat(s + "gate", s + "up")
        out[o + "shared.down_proj.weight"] = src.pop(s + "down")

    try:
        out["embed_tokens.weight"] = src.pop("embed")
        out["embed_norm.weight"] = src.pop("embed.norm")
        out["norm.weight"] = src.pop("final.norm")
        for i, e in enumerate(cfg.layers):
            lt, rt = f"l{i}.mix.left.", f"l{i}.mix.right."
            o = f"blocks.{i}."
            out[o + "norm1.weight"] = src.pop(f"l{i}.norm1")
            out[o + "mixer.in_proj.weight"] = cat(
                lt + "q", lt + "k", lt + "v", rt + "y", rt + "x")
            out[o + "mixer.o_proj.weight"] = cat(lt + "o", rt + "o", dim=1)
            attention(lt, o + "mixer.branches.left.")
            recurrence(rt, o + "mixer.branches.right.")
            m, p = e.get("mlp"), f"l{i}.mlp."
            if m is None:
                continue
            out[o + "norm2.weight"] = src.pop(f"l{i}.norm2")
            if m["kind"] == "dense":
                out[o + "mlp.gate_up_proj.weight"] = cat(p + "gate", p + "up")
                out[o + "mlp.down_proj.weight"] = src.pop(p + "down")
            else:
                experts(p, o + "mlp.", m)
    except KeyError as err:
        raise KeyError(f"checkpoint lacks tensor {err.args[0]!r}") from None
    if src:
        raise KeyError(f"checkpoint has unknown tensors {sorted(src)}")
    return out
