"""Device-typed op entry points used by the model runtime.

On a CUDA (ROCm) device every call goes to the hand-written gfx950 HIP
kernel — a missing extension raises (lfmq.ops.hip_ext), it never falls
back to eager torch.  On CPU the exact reference twin runs (unit tests +
the OPT int8 CPU decode config).  This is a device split, not a backend
dispatch: per device there is exactly one implementation.
"""
from __future__ import annotations

import math
import os
from typing import Optional

import torch

from . import hip_ext, ref, seq_ext

# Debug numeric guard: LFMQ_NANCHECK=1 asserts every op
# output is finite — catches kernel-layout or quantization bugs at the
# op that produced them instead of 30 layers later.
_NANCHECK = os.environ.get("LFMQ_NANCHECK", "0") == "1"


def _guard(t: torch.Tensor, name: str) -> torch.Tensor:
    if _NANCHECK and not bool(torch.isfinite(t.float()).all()):
        raise FloatingPointError(f"lfmq op {name} produced non-finite values")
    return t


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5,
            residual: Optional[torch.Tensor] = None) -> torch.Tensor:
    if x.is_cuda:
        return hip_ext().rmsnorm(x, weight, eps, residual)
    return ref.rmsnorm(x, weight, eps, residual)


def rmsnorm_residual(x: torch.Tensor, residual: torch.Tensor,
                     weight: torch.Tensor, eps: float = 1e-5):
    """Returns (normed, new_residual = x + residual) in one pass."""
    if x.is_cuda:
        return hip_ext().rmsnorm_residual(x, residual, weight, eps)
    new_res = ref.residual_add(x, residual)
    return ref.rmsnorm(new_res, weight, eps), new_res


_INV_FREQ_CACHE: dict = {}
# zero-initialized arrival tickets for the in-launch attention combine:
# the winning chunk resets its entry, so one buffer per (n, device) stays
# valid across steps and graph replays
_TICKETS_CACHE: dict = {}


def _tickets(n: int, device) -> "torch.Tensor":
    key = (n, str(device))
    t = _TICKETS_CACHE.get(key)
    if t is None:
        t = torch.zeros(n, dtype=torch.int32, device=device)
        _TICKETS_CACHE[key] = t
    return t


def _inv_freq(d: int, theta: float, device) -> torch.Tensor:
    key = (d, theta, str(device))
    t = _INV_FREQ_CACHE.get(key)
    if t is None:
        t = ref.rope_freqs(d, theta).to(device)
        _INV_FREQ_CACHE[key] = t
    return t


def apply_rope(q: torch.Tensor, k: torch.Tensor, positions: torch.Tensor,
               theta: float = 500000.0):
    """q: [b, s, hq, d], k: [b, s, hkv, d] — rotated in place on GPU."""
    if q.is_cuda:
        q = q.contiguous()
        k = k.contiguous()
        hip_ext().rope(q, k, positions.to(torch.int32),
                       _inv_freq(q.shape[-1], theta, q.device))
        return q, k
    return ref.apply_rope(q, positions, theta), ref.apply_rope(k, positions, theta)


def dq_linear(x: torch.Tensor, qweight: torch.Tensor, scales: torch.Tensor,
              qzeros: torch.Tensor, bits: int, group_size: int,
              bias: Optional[torch.Tensor] = None,
              resid: Optional[torch.Tensor] = None,
              rms_eps: float = -1.0) -> torch.Tensor:
    """Fused dequant-GEMM y = x @ dequant(W)^T (+bias) (+residual)
    (rms_eps >= 0: fused-RMSNorm input, decode m<=4 GPU path only)."""
    if x.is_cuda:
        x2 = x.reshape(-1, x.shape[-1])
        r2 = resid.reshape(-1, resid.shape[-1]).contiguous() if resid is not None else None
        y = hip_ext().dq_linear(x2, qweight, scales, qzeros, bits, group_size,
                                bias, r2, rms_eps, 0)
        return _guard(y, "dq_linear").reshape(*x.shape[:-1], y.shape[-1])
    assert resid is None and rms_eps < 0, "fused rms/resid is GPU-only"
    return ref.dq_linear(x, qweight, scales, qzeros, bits, group_size, bias).to(x.dtype)


def silu_mul(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    if gate.is_cuda:
        return hip_ext().silu_mul(gate.contiguous(), up.contiguous())
    return ref.silu_mul(gate, up)


def silu_mul_gateup(gate_up: torch.Tensor, inter: int) -> torch.Tensor:
    """silu(gu[..., :inter]) * gu[..., inter:] without materializing the
    split halves (one fused kernel on GPU)."""
    if gate_up.is_cuda:
        return seq_ext().silu_mul_fused(gate_up.contiguous())
    gate, up = gate_up.split([inter, inter], dim=-1)
    return ref.silu_mul(gate, up)


def attn_decode(q, k_cache, v_cache, seq_len: int, scale: Optional[float] = None):
    if q.is_cuda:
        return _guard(hip_ext().attn_decode(
            q, k_cache, v_cache, seq_len,
            scale or 1.0 / math.sqrt(q.shape[-1]), None), "attn_decode")
    return ref.attn_decode(q, k_cache, v_cache, seq_len, scale)


def attn_prefill(q, k, v, causal: bool = True, scale: Optional[float] = None):
    """Prefill attention. GPU: explicit bf16 matmul chain via rocBLAS (the
    PyTorch-ROCm layer; never SDPA, which can route to aotriton/Triton).
    GQA is handled by folding the q-head repeat into the row dimension
    (no K/V repeat_interleave copies), and the query axis is processed in
    chunks so the fp32 score tile stays bounded (a full 2048-seq layer
    would otherwise materialize a 537 MB score tensor)."""
    if q.is_cuda:
        b, hq, s, d = q.shape
        hkv = k.shape[1]
        rep = hq // hkv
        scale = scale or 1.0 / math.sqrt(d)
        kt = k.transpose(-1, -2)                      # [b, hkv, d, s]
        out = torch.empty_like(q)
        CH = 512 if s > 512 else s
        for q0 in range(0, s, CH):
            q1 = min(s, q0 + CH)
            # [b, hkv, rep*(q1-q0), d]: repeat folded into the row dim
            qc = (q.view(b, hkv, rep, s, d)[:, :, :, q0:q1]
                  .reshape(b, hkv, rep * (q1 - q0), d))
            sc = torch.matmul(qc, kt).float() * scale  # [b,hkv,rep*cq,s]
            if causal:
                t_idx = torch.arange(s, device=q.device)
                rows = torch.arange(q0, q1, device=q.device)
                m = (t_idx[None, :] > rows[:, None])   # [cq, s]
                sc = sc.view(b, hkv, rep, q1 - q0, s).masked_fill(
                    m[None, None, None], float("-inf")).view(
                    b, hkv, rep * (q1 - q0), s)
            p = torch.softmax(sc, dim=-1).to(q.dtype)
            oc = torch.matmul(p, v)                    # [b,hkv,rep*cq,d]
            out.view(b, hkv, rep, s, d)[:, :, :, q0:q1] = (
                oc.view(b, hkv, rep, q1 - q0, d))
        return out
    return ref.attn_prefill(q, k, v, causal, scale)


def attn_prefill_fused(q: torch.Tensor, k_cache: torch.Tensor,
                       v_cache: torch.Tensor, pos0: int,
                       scale: Optional[float] = None) -> torch.Tensor:
    """GPU flash prefill (csrc/attn_prefill.hip): one MFMA kernel instead
    of the rocBLAS matmul chain (measured 3.3-6.3x faster at s 256-2048,
    rel_err ~4e-3 vs fp32; tools/prefill_flash_bench.py).  q [b, s, hq, d]
    already roped (the qkv_rope_append output); caches [b, hkv, Tmax, d]
    hold rows [0, pos0+s).  d == 128 only.  Default GPU prefill path;
    LFMQ_FLASH_PREFILL=0 restores the matmul chain."""
    b, s, hq, d = q.shape
    scale = scale or 1.0 / math.sqrt(d)
    o = _guard(hip_ext().attn_prefill(q.reshape(b, s, hq * d), k_cache,
                                      v_cache, hq, pos0, scale),
               "attn_prefill_fused")
    return o.view(b, s, hq, d)


USE_FLASH_PREFILL = os.environ.get("LFMQ_FLASH_PREFILL", "1") == "1"


def qkv_rope_append(qkv: torch.Tensor, k_cache: torch.Tensor,
                    v_cache: torch.Tensor, positions: torch.Tensor,
                    pos0: int, hq: int, theta: float = 500000.0) -> torch.Tensor:
    """GPU-only fused decode epilogue of the qkv projection: rope(q),
    rope(k)+append, append(v) in one launch.  qkv: [b, s, (hq+2hkv)*d];
    returns q [b, s, hq, d] (== [b, hq, 1, d] layout at s == 1)."""
    d = k_cache.shape[-1]
    return hip_ext().qkv_rope_append(qkv.contiguous(), k_cache, v_cache,
                                     positions.to(torch.int32),
                                     _inv_freq(d, theta, qkv.device), hq,
                                     pos0, None)


def qkv_rope_append_graph(qkv: torch.Tensor, k_cache: torch.Tensor,
                          v_cache: torch.Tensor, state: torch.Tensor,
                          hq: int, theta: float = 500000.0) -> torch.Tensor:
    """hipGraph decode variant: position read from state[0] on device."""
    d = k_cache.shape[-1]
    pos_dev = state[0:1]
    return hip_ext().qkv_rope_append(qkv.contiguous(), k_cache, v_cache,
                                     pos_dev, _inv_freq(d, theta, qkv.device),
                                     hq, 0, pos_dev)


def attn_decode_graph(q, k_cache, v_cache, state, max_t: int, scale: float):
    """hipGraph decode variant: T read from state[1]; grid sized for max_t."""
    return hip_ext().attn_decode(q, k_cache, v_cache, max_t, scale, state[1:2])


def attn_decode_fused(qkv, k_cache, v_cache, state_or_T, max_t: int,
                      scale: float, hq: int, theta: float = 500000.0):
    """One launch: rope(q,k) off the raw qkv buffer, KV-cache append,
    chunked decode attention.  state_or_T: device state tensor (graph
    mode, T = state[1]) or a host int T."""
    d = k_cache.shape[-1]
    inv = _inv_freq(d, theta, qkv.device)
    tk = _tickets(k_cache.shape[0] * hq, qkv.device)
    if torch.is_tensor(state_or_T):
        return hip_ext().attn_decode_fused(qkv.contiguous(), k_cache, v_cache,
                                           max_t, scale, inv, hq,
                                           state_or_T[1:2], tk)
    return hip_ext().attn_decode_fused(qkv.contiguous(), k_cache, v_cache,
                                       int(state_or_T), scale, inv, hq, None,
                                       tk)


def dq_gemv_gateup(x: torch.Tensor, qweight: torch.Tensor,
                   scales: torch.Tensor, qzeros: torch.Tensor, bits: int,
                   group_size: int, rms_eps: float = -1.0) -> torch.Tensor:
    """GPU-only fused gate_up GEMV + silu·mul epilogue (m <= 4);
    rms_eps >= 0 additionally fuses the RMSNorm of the input."""
    x2 = x.reshape(-1, x.shape[-1])
    y = hip_ext().dq_gemv_gateup(x2, qweight, scales, qzeros, bits,
                                 group_size, rms_eps, 0)
    return y.reshape(*x.shape[:-1], y.shape[-1])


def greedy_sample(logits: torch.Tensor) -> torch.Tensor:
    """argmax over the last dim of [b, vocab] logits -> int64 [b]."""
    if logits.is_cuda:
        return seq_ext().greedy_sample(logits.contiguous())
    return logits.argmax(dim=-1)


def kv_append(k_cache, v_cache, k_new, v_new, pos: int) -> None:
    """caches [b, hkv, T_max, d]; k_new/v_new TOKEN-major [b, s, hkv, d]
    (as the qkv split produces them — saves the transpose copies)."""
    if k_cache.is_cuda:
        hip_ext().kv_append(k_cache, v_cache, k_new.contiguous(),
                            v_new.contiguous(), pos)
        return
    ref.kv_append(k_cache, v_cache, k_new.transpose(1, 2), v_new.transpose(1, 2), pos)


# ---------------------------------------------------------------------------
# packed-batch ops (lfmq/models/seqcache.py: StepBatch).  GPU only.
# ---------------------------------------------------------------------------

def bigram_embed(tokens, batch, cache, embed, table, mul_prev: int,
                 mul_cur: int) -> torch.Tensor:
    """fp32 residual rows embed[tok] + table[hash(prev, tok)]; a sequence's
    first token takes the table's last row."""
    return seq_ext().bigram_embed(tokens, *batch.view(cache), cache.prev,
                                  embed, table, mul_prev, mul_cur)


def seq_advance(tokens, batch, cache) -> None:
    """Close a step on the device: lengths, previous tokens, buffer turns."""
    seq_ext().seq_advance(tokens, batch.cu, batch.slots, cache.lens,
                          cache.prev, cache.turn)


def add_norm(x, y, weight, bias: float, eps: float, out_dtype,
             side_w=None, side_b=None):
    """x += y in place (fp32 residual), then h = rms_norm(x) * (bias + w).
    Returns (h, side): side = h @ side_w^T + side_b in fp32."""
    h, side = seq_ext().add_norm(x, y, weight, bias, eps, side_w, side_b,
                                 out_dtype == torch.float32)
    return _guard(h, "add_norm"), side


MLSTM_CHUNK = 128        # tokens a chunk: state traffic against score work


def mlstm(proj, gates, batch, cache, S, nm, cap: float, norm_w, eps: float,
          by_token: bool = False) -> torch.Tensor:
    """Matrix-memory recurrence over the step's rows, each head's output
    normed, weighted and gated: [N, H * vdim].  proj rows are
    [q | k | v | output gate].  Single tokens and 32-bit storage run token
    by token (by_token: everything), prompts by chunks."""
    ext = seq_ext()
    if not (by_token or batch.single) and ext.mlstm_chunk_ok(proj, S):
        base, total = batch.chunks(MLSTM_CHUNK)
        return _guard(ext.mlstm_chunk(
            proj, gates, *batch.view(cache), cache.turn, S, nm, cap, norm_w,
            eps, base, total, MLSTM_CHUNK, max(batch.counts)), "mlstm_chunk")
    o = ext.mlstm_scan(proj, gates, *batch.view(cache), cache.turn, S, nm, cap)
    gate = proj[:, S.shape[1] * (2 * S.shape[2] + S.shape[3]):]
    return head_norm_gate(o, gate, norm_w, eps)


def head_norm_gate(o, gate, weight, eps: float) -> torch.Tensor:
    """o / rms(o) per head (fp32 [N, H, v]), times weight and sigmoid(gate)."""
    return _guard(seq_ext().head_norm_gate(o, gate, weight, eps),
                  "head_norm_gate")


def _scaled_freq(f: float, factor: float, low: float, high: float,
                 original: float) -> float:
    """Context extension by wavelength: short waves keep their frequency,
    long ones are slowed by `factor`, those between are blended."""
    turns = original * f / (2 * math.pi)     # within the original context
    if turns < low:
        return f / factor
    if turns > high:
        return f
    s = (turns - low) / (high - low)
    return (1 - s) * f / factor + s * f


def rope_inv_freq(dims: int, base: float, device,
                  scaling: Optional[dict] = None) -> torch.Tensor:
    """fp32 base^(-2i/dims), i < dims/2, computed in double precision.
    scaling: {factor, low, high, original} of _scaled_freq."""
    key = ("f64", dims, float(base), str(device),
           tuple(sorted(scaling.items())) if scaling else None)
    t = _INV_FREQ_CACHE.get(key)
    if t is None:
        f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
        if scaling:
            f = [_scaled_freq(x, **scaling) for x in f]
        t = torch.tensor(f, dtype=torch.float64).float().to(device)
        _INV_FREQ_CACHE[key] = t
    return t


def latent_prep(proj, batch, cache, q_norm, kv_norm, inv_freq, dst, dst_row,
                eps: float) -> torch.Tensor:
    return seq_ext().latent_prep(proj, *batch.view(cache), q_norm, kv_norm,
                                 inv_freq, dst, dst_row, eps)


def latent_ring(batch, cache, rows, buf, ring, load: bool) -> None:
    seq_ext().latent_ring(*batch.view(cache), rows.own, rows.prior, buf, ring,
                          load)


def latent_absorb(q, w_uk, batch, cache, inv_freq, rot: int) -> torch.Tensor:
    return seq_ext().latent_absorb(q, w_uk, *batch.view(cache), inv_freq, rot)


def latent_expand(part, sink, w_uv, gate) -> torch.Tensor:
    return _guard(seq_ext().latent_expand(part, sink, w_uv, gate),
                  "latent_expand")


def attn_window_prompt(q, kv, lat, batch, cache, rows, inv_freq, sink, gate,
                       d1: int, d2: int, dv: int, window: int, scale: float,
                       general: bool = False) -> torch.Tensor:
    """Sliding-window attention with a sink and an output gate over the
    step's key buffer (q's second part is rotated inside).  general: the
    any-size kernel also where the matrix-core one applies."""
    return _guard(seq_ext().attn_window_prompt(
        q, kv, lat, *batch.view(cache), rows.own, inv_freq, sink, gate, d1,
        d2, dv, window, scale, max(batch.counts), general),
        "attn_window_prompt")


def attn_window_decode(q, ring, batch, cache, rank: int, window: int,
                       scale: float, general: bool = False) -> torch.Tensor:
    """Absorbed queries over the latent ring (one token per sequence):
    partial results of a split key range.  general: the any-size kernel
    also where the matrix-core one applies."""
    reach = min(window, ring.shape[1])
    # enough key ranges to fill the chip, none shorter than two key tiles
    groups = -(-q.shape[1] // 32) * q.shape[0]
    splits = max(1, min(-(-reach // 64), -(-512 // groups), 64))
    return seq_ext().attn_window_decode(q, ring, *batch.view(cache), rank,
                                        window, splits, scale, general)


def embed_norm(tokens, table, weight, eps: float):
    """(x, h): normed embedding rows as the fp32 residual, and in the
    table's dtype."""
    return seq_ext().embed_norm(tokens, table, weight, eps)


def post_norm(x, y, weight, eps: float, w_out=None, gain: float = 1.0):
    """x += rms_norm(y) * weight in place (fp32 residual).  Returns x in y's
    dtype (x itself in 32 bit) or, given w_out, rms_norm(x) * w_out * gain."""
    return _guard(seq_ext().post_norm(x, y, weight, eps, w_out, gain),
                  "post_norm")


def post_norm_experts(x, y, weight, eps: float, w_out=None,
                      gain: float = 1.0):
    """post_norm of a lfmq.models.mixers.ExpertSum."""
    return _guard(seq_ext().post_norm_experts(
        x, y.rows, y.pos, y.shared, y.sgate, weight, eps, w_out, gain),
        "post_norm_experts")


def qk_prep(proj, batch, cache, q_norm, k_norm, inv_freq, kc, vc,
            eps: float) -> torch.Tensor:
    """[q | k | v] columns: norms over all of q and all of k, rotation; keys
    and values go to the cache, queries [N, heads * dim] are returned."""
    return seq_ext().qk_prep(proj, *batch.view(cache), q_norm, k_norm,
                             inv_freq, kc, vc, eps)


def attn_grouped(q, kc, vc, batch, cache, sink, out, scale: float,
                 gain: float = 1.0, general: bool = False) -> None:
    """Causal grouped-query attention with a sink over the cache, written to
    out's columns.  general: the any-size kernel also where a matrix-core
    one applies."""
    seq_ext().attn_grouped(q, kc, vc, *batch.view(cache), sink, out, scale,
                           gain, batch.max_count, general)
    _guard(out, "attn_grouped")


LRU_TILE = 64            # tokens a tile of the prompt kernels


def gated_lru(x, y, batch, cache, x_b, y_b, conv_w, conv_b, gate_w, gate_b,
              lam, ring, S, out, c: float, gain: float = 1.0,
              general: bool = False) -> None:
    """Convolution, gates, linear recurrence and gelu branch over the step's
    rows (csrc/gated_lru.hip), written to out's columns."""
    base, total = (None, 0) if batch.single else batch.chunks(LRU_TILE)
    seq_ext().gated_lru(x, y, *batch.view(cache), x_b, y_b, conv_w, conv_b,
                        gate_w, gate_b, lam, ring, S, out, c, gain, base,
                        total, batch.max_count, general)
    _guard(out, "gated_lru")


def clamped_glu(gate_up, limit: float, alpha: float, beta: float):
    return seq_ext().clamped_glu(gate_up, limit, alpha, beta)


def moe(h, router, gate_up, down, top: int, act, general: bool = False):
    """Router, sort by expert and expert products: (rows [N * top, width],
    pos [N, top] row of a token's choice, the shared expert's gate [N] if
    the router has its row).  Stays on the device."""
    ext = seq_ext()
    E, ff2, width = gate_up.shape
    aligned = not general and h.dtype == torch.bfloat16 and \
        width % 8 == 0 and ff2 % 16 == 0
    bm = ext.moe_tile(h.shape[0] * top, E, aligned)
    src, weight, pos, tiles, sgate = ext.moe_route(h, router, E, top, bm)
    a = ext.moe_glu(h, gate_up, src, weight, tiles, *act, bm)
    return _guard(ext.moe_down(a, down, tiles, bm), "moe"), pos, sgate
