"""Model registry: arch name -> configuration, model class, default dtype,
and how a plain (unquantized) checkpoint directory maps onto the model.

A plain directory holds config.json — "arch" or "architecture" picks the
entry — and model.safetensors.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Optional

import torch

from .llama import LlamaConfig, LlamaForCausalLM
from .mixtral import MixtralConfig, MixtralForCausalLM
from .opt import OPTConfig, OPTForCausalLM
from .rapivik import RapivikConfig, RapivikForCausalLM
from .rapivik import convert_state as rapivik_state
from .zatasun import ZatasunConfig, ZatasunForCausalLM
from .zatasun import convert_state as zatasun_state


@dataclass(frozen=True)
class ArchSpec:
    config: type
    model: type
    dtype: torch.dtype
    # (cfg, checkpoint tensors) -> state dict; None: no plain format
    convert: Optional[Callable] = None


ARCHS = {
    "llama": ArchSpec(LlamaConfig, LlamaForCausalLM, torch.bfloat16),
    "opt": ArchSpec(OPTConfig, OPTForCausalLM, torch.float32),
    "mixtral": ArchSpec(MixtralConfig, MixtralForCausalLM, torch.bfloat16),
    "rapivik": ArchSpec(RapivikConfig, RapivikForCausalLM, torch.bfloat16,
                        rapivik_state),
    "zatasun": ArchSpec(ZatasunConfig, ZatasunForCausalLM, torch.bfloat16,
                        zatasun_state),
}


def spec_of(d) -> ArchSpec:
    """Registry entry for a configuration (object or dict)."""
    if isinstance(d, dict):
        arch = d.get("arch") or str(d.get("architecture", "llama")).lower()
    else:
        arch = d.arch
    if arch not in ARCHS:
        raise ValueError(f"unknown arch {arch!r}")
    return ARCHS[arch]


def read_plain_config(path: str) -> Optional[dict]:
    """config.json of a plain checkpoint directory of a registered
    architecture, or None."""
    fn = os.path.join(path, "config.json")
    if not os.path.isfile(fn):
        return None
    with open(fn) as f:
        d = json.load(f)
    name = d.get("arch") or d.get("architecture")
    if not isinstance(name, str):
        return None
    spec = ARCHS.get(name.lower())
    return d if spec is not None and spec.convert is not None else None
