"""Token mixers, feed-forward and norms for packed batches (SequenceCache).

Each mixer takes its sizes and constants as arguments and has one
interface, so that a model is a list of them:

    state_spec(max_seq)          what a cache slot holds for one layer run
    side()                       (weight, bias) of outputs that must stay in
                                 32 bits, computed inside the input norm
    forward(h, side, batch, cache, state) -> sublayer output [N, width]

h [N, width] is the sublayer's input in the model's dtype (bf16 or fp32).
Norm weights, gate biases and sinks are fp32 always.

Mixers that can run side by side are written as branches of a
ParallelMixer, which owns one input and one output projection for all:

    rows_in, rows_out            columns of the input projection that the
                                 branch reads, and of its result
    state_spec(max_seq)          as above
    mix(p, out, gain, batch, cache, state)
                                 p [N, rows_in] -> out [N, rows_out], both
                                 column views; the result is times gain
"""
from __future__ import annotations

from typing import Dict, NamedTuple, Optional, Tuple

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


class GroupedAttention(nn.Module):
    """Branch: causal grouped-query attention with RMS norms over the whole
    query and key projections, rotary positions and a softmax sink per head.
    The cache keeps keys (normed and rotated) and values of every token.
    rot_scaling: the wavelength-dependent frequency scaling of
    lfmq.ops.functional.rope_inv_freq."""

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int,
                 scale: float, rot_dims: int, rot_base: float,
                 rot_scaling: Optional[dict], eps: float, dtype):
        super().__init__()
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError(f"cannot rotate {rot_dims} of {dim} dimensions")
        if heads % kv_heads:
            raise ValueError(f"{heads} heads do not share {kv_heads}")
        self.kv_heads, self.dim, self.vdim = kv_heads, dim, vdim
        self.scale, self.eps, self.dtype = scale, eps, dtype
        self.rot = (rot_dims, rot_base, rot_scaling)
        # [queries | keys | values]
        self.rows_in = heads * dim + kv_heads * (dim + vdim)
        self.rows_out = heads * vdim
        self.q_norm = _fp32(heads * dim, 1.0)
        self.k_norm = _fp32(kv_heads * dim, 1.0)
        self.sink = _fp32(heads)

    def state_spec(self, max_seq: int) -> dict:
        # rows of later positions are written before they are read
        return {n: ((max_seq, self.kv_heads, d), self.dtype, "by_position")
                for n, d in (("k", self.dim), ("v", self.vdim))}

    def mix(self, p, out, gain, batch, cache, state):
        dims, base, scaling = self.rot
        inv = F.rope_inv_freq(dims, base, p.device, scaling)
        q = F.qk_prep(p, batch, cache, self.q_norm, self.k_norm, inv,
                      state["k"], state["v"], self.eps)
        F.attn_grouped(q, state["k"], state["v"], batch, cache, self.sink,
                       out, self.scale, gain)


class GatedLRU(nn.Module):
    """Branch: a real-gated linear recurrent unit behind a short causal
    convolution, times a gelu branch.  Both gates of the recurrence are
    block-diagonal; decay = exp(decay_c * r * softplus(lam))."""

    decay_c = -8.0

    def __init__(self, width: int, blocks: int, taps: int, dtype):
        super().__init__()
        if width % blocks:
            raise ValueError(f"{blocks} blocks do not divide width {width}")
        n = width // blocks
        self.width, self.taps = width, taps
        self.rows_in, self.rows_out = 2 * width, width    # [gelu | conv]
        self.y_b, self.x_b = _fp32(width), _fp32(width)
        # rows by age, the current token's last
        self.conv_w = nn.Parameter(torch.zeros(taps, width))
        self.conv_b = _fp32(width)
        # [recurrence gate | input gate] of every block, [out, in]
        self.gate_w = nn.Parameter(torch.zeros(blocks, 2, n, n, dtype=dtype))
        self.gate_b = nn.Parameter(torch.zeros(blocks, 2, n))
        self.lam = _fp32(width)

    def state_spec(self, max_seq: int) -> dict:
        return {"S": ((self.width,), torch.float32),
                "conv": ((self.taps, self.width), torch.float32)}

    def mix(self, p, out, gain, batch, cache, state):
        F.gated_lru(p[:, self.width:], p[:, :self.width], batch, cache,
                    self.x_b, self.y_b, self.conv_w, self.conv_b, self.gate_w,
                    self.gate_b, self.lam, state["conv"], state["S"], out,
                    self.decay_c, gain)


class ParallelMixer(nn.Module):
    """Branches side by side on one input: one projection in, one out, the
    sum of the branches' outputs weighted by their gains."""

    def __init__(self, width: int, branches: Dict[str, Tuple[nn.Module, float]],
                 dtype):
        super().__init__()
        self.branches = nn.ModuleDict({k: b for k, (b, _) in branches.items()})
        self.gains = {k: g for k, (_, g) in branches.items()}
        bs = self.branches.values()
        self.rows_in = sum(b.rows_in for b in bs)
        self.rows_out = sum(b.rows_out for b in bs)
        self.in_proj = nn.Linear(width, self.rows_in, bias=False, dtype=dtype)
        self.o_proj = nn.Linear(self.rows_out, width, bias=False, dtype=dtype)

    def state_spec(self, max_seq: int) -> dict:
        return {f"{n}.{k}": v for n, b in self.branches.items()
                for k, v in b.state_spec(max_seq).items()}

    def side(self):
        return None, None

    def forward(self, h, side, batch, cache, state):
        p = self.in_proj(h)
        out = torch.empty(p.shape[0], self.rows_out, dtype=p.dtype,
                          device=p.device)
        i = o = 0
        for n, b in self.branches.items():
            b.mix(p[:, i:i + b.rows_in], out[:, o:o + b.rows_out],
                  self.gains[n], batch, cache,
                  {k[len(n) + 1:]: t for k, t in state.items()
                   if k.startswith(n + ".")})
            i, o = i + b.rows_in, o + b.rows_out
        return self.o_proj(out)


class DenseMLP(nn.Module):
    """down(silu(gate h) * up h), gate and up fused."""

    def __init__(self, width: int, ff: int, dtype):
        super().__init__()
        self.ff = ff
        self.gate_up_proj = nn.Linear(width, 2 * ff, bias=False, dtype=dtype)
        self.down_proj = nn.Linear(ff, width, bias=False, dtype=dtype)

    def forward(self, h):
        return self.down_proj(F.silu_mul_gateup(self.gate_up_proj(h), self.ff))


class ExpertSum(NamedTuple):
    """A feed-forward's output not yet summed: token t's is the sum of
    rows[pos[t, :]] and, with a shared expert, sgate[t] * shared[t]."""
    rows: torch.Tensor
    pos: torch.Tensor
    shared: Optional[torch.Tensor]
    sgate: Optional[torch.Tensor]


class ClampedGLU(nn.Module):
    """down(g sigmoid(alpha g) (u + beta)), g = min(gate h, limit) and
    u = clamp(up h, -limit, limit)."""

    def __init__(self, width: int, ff: int, limit: float, alpha: float,
                 beta: float, dtype):
        super().__init__()
        self.act = (limit, alpha, beta)
        self.gate_up_proj = nn.Linear(width, 2 * ff, bias=False, dtype=dtype)
        self.down_proj = nn.Linear(ff, width, bias=False, dtype=dtype)

    def forward(self, h):
        return self.down_proj(F.clamped_glu(self.gate_up_proj(h), *self.act))


class ExpertMLP(nn.Module):
    """Mixture of clamped-GLU experts.  A token goes to the `top` experts
    with the largest sigmoid scores; the score (not renormalized) weights
    the expert's input.  A shared expert runs for every token, times the
    sigmoid of one output of its own.  Returns an ExpertSum."""

    def __init__(self, width: int, experts: int, top: int, ff: int,
                 limit: float, alpha: float, beta: float,
                 shared: Optional[ClampedGLU], dtype):
        super().__init__()
        if not 1 <= top <= experts:
            raise ValueError(f"cannot choose {top} of {experts} experts")
        self.experts, self.top = experts, top
        self.act = (limit, alpha, beta)
        # a router row per expert, then the shared expert's gate
        self.router = nn.Parameter(torch.zeros(
            experts + (shared is not None), width, dtype=dtype))
        self.gate_up = nn.Parameter(torch.zeros(experts, 2 * ff, width,
                                                dtype=dtype))
        self.down = nn.Parameter(torch.zeros(experts, width, ff, dtype=dtype))
        self.shared = shared

    def forward(self, h) -> ExpertSum:
        rows, pos, sgate = F.moe(h, self.router, self.gate_up, self.down,
                                 self.top, self.act)
        if self.shared is None:
            return ExpertSum(rows, pos, None, None)
        return ExpertSum(rows, pos, self.shared(h), sgate)


class PostNorm(nn.Module):
    """RMS norm on a sublayer's output, added to the fp32 residual stream."""

    def __init__(self, dim: int, eps: float):
        super().__init__()
        self.weight, self.eps = _fp32(dim, 1.0), eps

    def forward(self, x, y, out: Optional[nn.Module] = None,
                gain: float = 1.0):
        """x += norm(y) in place; returns x in y's dtype, or out's norm of
        it times gain."""
        w_out = None if out is None else out.weight
        if isinstance(y, ExpertSum):
            return F.post_norm_experts(x, y, self.weight, self.eps, w_out,
                                       gain)
        return F.post_norm(x, y, self.weight, self.eps, w_out, gain)


class PostNormBlock(nn.Module):
    """Block whose norms sit on the sublayers' outputs: the sublayers read
    the fp32 residual x itself (h: x in the model's dtype).  Returns the
    next h; last: (the model's output norm, gain) behind the last block."""

    def __init__(self, mixer: nn.Module, mlp: Optional[nn.Module], width: int,
                 eps: float):
        super().__init__()
        self.mixer = mixer
        self.norm1 = PostNorm(width, eps)
        if mlp is not None:
            self.norm2 = PostNorm(width, eps)
        self.mlp = mlp

    def forward(self, x, h, batch, cache, state, last=(None, 1.0)):
        y = self.mixer(h, None, batch, cache, state)
        if self.mlp is None:
            return self.norm1(x, y, *last)
        return self.norm2(x, self.mlp(self.norm1(x, y)), *last)


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
