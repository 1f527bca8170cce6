"""Token mixers, feed-forward and norms for packed batches (SequenceCache).

Each mixer takes its sizes and constants as arguments and has one
interface, so that a model is a list of them:

    state_spec(max_seq)          what a cache slot holds for one layer run
    side()                       (weight, bias) of outputs that must stay in
                                 32 bits, computed inside the input norm
    forward(h, side, batch, cache, state) -> sublayer output [N, width]

h [N, width] is the normed input in the model's dtype (bf16 or fp32).
Norm weights, gate biases and sinks are fp32 always.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from ..ops import functional as F


def _fp32(n: int, value: float = 0.0) -> nn.Parameter:
    return nn.Parameter(torch.full((n,), value, dtype=torch.float32))


class ResidualNorm(nn.Module):
    """RMS norm on the fp32 residual stream, fused with adding the previous
    sublayer's output.  centred: the weight is an offset from one."""

    def __init__(self, dim: int, eps: float, centred: bool, out_dtype):
        super().__init__()
        self.weight = _fp32(dim, 0.0 if centred else 1.0)
        self.bias = 1.0 if centred else 0.0
        self.eps, self.out_dtype = eps, out_dtype

    def forward(self, x, y: Optional[torch.Tensor], side=(None, None)):
        return F.add_norm(x, y, self.weight, self.bias, self.eps,
                          self.out_dtype, *side)


class MLSTMMixer(nn.Module):
    """Matrix-memory LSTM with soft-capped exponential gates, a per-head
    output norm and a sigmoid output gate."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int,
                 gate_cap: float, eps: float, dtype):
        super().__init__()
        self.heads, self.dim, self.vdim = heads, dim, vdim
        self.cap, self.eps = gate_cap, eps
        # [q | k | v | output gate]
        self.in_proj = nn.Linear(width, 2 * heads * (dim + vdim), bias=False,
                                 dtype=dtype)
        # [input gate | forget gate], one of each per head
        self.gate_w = nn.Parameter(torch.zeros(2 * heads, width, dtype=dtype))
        self.gate_b = _fp32(2 * heads)
        self.norm_w = _fp32(heads * vdim, 1.0)
        self.o_proj = nn.Linear(heads * vdim, width, bias=False, dtype=dtype)

    def state_spec(self, max_seq: int) -> dict:
        return {"S": ((self.heads, self.dim, self.vdim), torch.float32),
                "nm": ((2, self.heads, self.dim + 1), torch.float32)}

    def side(self):
        return self.gate_w, self.gate_b

    def forward(self, h, side, batch, cache, state):
        p = self.in_proj(h)
        return self.o_proj(F.mlstm(p, side, batch, cache, state["S"],
                                   state["nm"], self.cap, self.norm_w,
                                   self.eps))


class LatentAttention(nn.Module):
    """Latent (low-rank key/value) attention over a sliding window, with a
    shared rotated key part, a softmax sink per head and a sigmoid output
    gate.  The cache keeps one latent row per token, window tokens deep.

    Prompts expand keys and values per head; single-token steps move both
    up-projections to the query and the output and read the cache itself.
    """

    def __init__(self, width: int, heads: int, dim: int, rot_dim: int,
                 vdim: int, q_rank: int, kv_rank: int, window: int,
                 scale: float, rot_base: float, rot_dims: int, eps: float,
                 dtype):
        super().__init__()
        if rot_dims % 2 or rot_dims > rot_dim:
            raise ValueError(f"cannot rotate {rot_dims} of {rot_dim} dimensions")
        self.heads, self.dim, self.rot, self.vdim = heads, dim, rot_dim, vdim
        self.q_rank, self.rank, self.window = q_rank, kv_rank, window
        self.scale, self.eps = scale, eps
        self.rot_base, self.rot_dims = rot_base, rot_dims
        # [query latent | kv latent | rotated key | output gate]
        self.in_proj = nn.Linear(
            width, q_rank + kv_rank + rot_dim + heads * vdim, bias=False,
            dtype=dtype)
        self.q_norm = _fp32(q_rank, 1.0)
        self.kv_norm = _fp32(kv_rank, 1.0)
        self.q_up = nn.Linear(q_rank, heads * (dim + rot_dim), bias=False,
                              dtype=dtype)
        # rows [keys of all heads | values of all heads]
        self.kv_up = nn.Parameter(torch.zeros(heads * (dim + vdim), kv_rank,
                                              dtype=dtype))
        self.sink = _fp32(heads)
        self.o_proj = nn.Linear(heads * vdim, width, bias=False, dtype=dtype)
        self._absorbed = None

    def state_spec(self, max_seq: int) -> dict:
        cap = min(self.window, max_seq)
        return {"ring": ((cap, self.rank + self.rot), self.kv_up.dtype)}

    def side(self):
        return None, None

    def absorbed(self):
        """(W_uk [H, dim, rank], W_uv [H, rank, vdim]) for decode."""
        w = self.kv_up
        key = (w.data_ptr(), w._version)
        if self._absorbed is None or self._absorbed[0] != key:
            k = self.heads * self.dim
            uk = w.detach()[:k].view(self.heads, self.dim, self.rank)
            uv = w.detach()[k:].view(self.heads, self.vdim, self.rank)
            self._absorbed = (key, uk, uv.transpose(1, 2).contiguous())
        return self._absorbed[1:]

    def forward(self, h, side, batch, cache, state):
        p = self.in_proj(h)
        ring = state["ring"]
        gate = p[:, self.q_rank + self.rank + self.rot:]
        inv = F.rope_inv_freq(self.rot_dims, self.rot_base, h.device)
        if batch.single:
            cq = F.latent_prep(p, batch, cache, self.q_norm, self.kv_norm,
                               inv, ring, None, self.eps)
            uk, uv = self.absorbed()
            q = F.latent_absorb(self.q_up(cq), uk, batch, cache, inv, self.rot)
            part = F.attn_window_decode(q, ring, batch, cache, self.rank,
                                        self.window, self.scale)
            return self.o_proj(F.latent_expand(part, self.sink, uv, gate))
        rows = batch.key_rows(self.window)
        lat = torch.empty(rows.total, self.rank + self.rot, dtype=p.dtype,
                          device=p.device)
        cq = F.latent_prep(p, batch, cache, self.q_norm, self.kv_norm, inv,
                           lat, rows.own, self.eps)
        if rows.any_prior:
            F.latent_ring(batch, cache, rows, lat, ring, load=True)
        kv = nn.functional.linear(lat[:, :self.rank], self.kv_up)
        o = F.attn_window_prompt(self.q_up(cq), kv, lat, batch, cache, rows,
                                 inv, self.sink, gate, self.dim, self.rot,
                                 self.vdim, self.window, self.scale)
        F.latent_ring(batch, cache, rows, lat, ring, load=False)
        return self.o_proj(o)


class DenseMLP(nn.Module):
    """down(silu(gate h) * up h), gate and up fused."""

    def __init__(self, width: int, ff: int, dtype):
        super().__init__()
        self.ff = ff
        self.gate_up_proj = nn.Linear(width, 2 * ff, bias=False, dtype=dtype)
        self.down_proj = nn.Linear(ff, width, bias=False, dtype=dtype)

    def forward(self, h):
        return self.down_proj(F.silu_mul_gateup(self.gate_up_proj(h), self.ff))


class MixerBlock(nn.Module):
    """Pre-norm block on the fp32 residual x.  Takes the previous
    sublayer's output y (not yet added) and returns its own last one."""

    def __init__(self, mixer: nn.Module, mlp: Optional[nn.Module], width: int,
                 eps: float, centred: bool, dtype):
        super().__init__()
        self.norm1 = ResidualNorm(width, eps, centred, dtype)
        self.mixer = mixer
        if mlp is not None:
            self.norm2 = ResidualNorm(width, eps, centred, dtype)
        self.mlp = mlp

    def forward(self, x, y, batch, cache, state):
        h, side = self.norm1(x, y, self.mixer.side())
        y = self.mixer(h, side, batch, cache, state)
        if self.mlp is not None:
            h, _ = self.norm2(x, y)
            y = self.mlp(h)
        return y
