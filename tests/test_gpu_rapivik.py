"""Rapivik on the GPU against the plain oracle: every mechanism alone, then
whole models — prompts, portions, decoding, unequal batches, slots used
again, window edges, generation."""
import io
import json
import math

import numpy as np
import pytest
import torch

import rapivik_oracle as oracle
import rapivik_util as util

pytestmark = pytest.mark.gpu
DEV = "cuda"
D = torch.float64
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-5, torch.bfloat16: 4e-2}


def F():
    from lfmq.ops import functional
    return functional


def gen(seed=0):
    return torch.Generator().manual_seed(seed)


def randn(*shape, g, scale=1.0, dtype=torch.float32):
    """Values that the dtype holds exactly, on the CPU in fp32."""
    return (torch.randn(*shape, generator=g) * scale).to(dtype).float()


def make_cache(spec, lens, max_seq=1 << 16):
    """A cache whose slots hold lens[i] tokens already."""
    from lfmq.models.seqcache import SequenceCache
    c = SequenceCache([spec], len(lens), max_seq, DEV)
    c.lens_host = list(lens)
    c.lens.copy_(torch.tensor(lens, dtype=torch.int32))
    return c


def close(got, want, tol):
    want = want.double()
    err = (got.double().cpu() - want).abs().max() / want.abs().max()
    assert math.isfinite(float(err)) and float(err) < tol, float(err)


# ---------------------------------------------------------------------------
# mechanisms
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
def test_bigram_embedding_and_step_end(dtype):
    """Unequal sequences, fresh and continued; the previous token is part
    of the slot's state."""
    g = gen()
    V, W, B = 50, 37, 23
    e, t = (randn(n, W, g=g, dtype=dtype) for n in (V, B + 1))
    toks = [[3, 49, 7], [5], [8, 8]]
    c = make_cache({}, [0, 4, 9])
    c.prev.copy_(torch.tensor([11, 21, 0], dtype=torch.int32))
    b = c.batch([0, 1, 2], [3, 1, 2])
    flat = torch.tensor(sum(toks, []), device=DEV)
    x = F().bigram_embed(flat, b, c, e.to(DEV, dtype), t.to(DEV, dtype), 17, 3)
    want = [e[ts].double() + t[oracle.bigram_rows(ts, B, 17, 3, p)].double()
            for ts, p in zip(toks, (None, 21, 0))]
    close(x, torch.cat(want), 1e-6)
    c.advance(flat, b)
    assert c.lens.tolist() == [3, 5, 11] == c.lens_host
    assert c.prev.tolist() == [7, 5, 8] and c.turn.tolist() == [1, 1, 1]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,side", [
    (1, 64, 6), (5, 51, 0), (3, 2052, 3), (2049, 96, 7), (2050, 53, 2)])
def test_add_norm(dtype, rows, width, side):
    g = gen(rows)
    x, y = randn(rows, width, g=g), randn(rows, width, g=g, dtype=dtype)
    w = randn(width, g=g, scale=0.3)
    sw = randn(side, width, g=g, dtype=dtype) if side else None
    sb = randn(side, g=g) if side else None
    for bias in (1.0, 0.0):
        xd = x.to(DEV)
        h, s = F().add_norm(xd, y.to(DEV, dtype), w.to(DEV), bias, 1e-3, dtype,
                            None if sw is None else sw.to(DEV, dtype),
                            None if sb is None else sb.to(DEV))
        r = x.double() + y.double()
        want = oracle.rms(r, 1e-3) * (bias + w.double())
        close(xd, r, 1e-6)
        close(h, want, 1e-5 if dtype == torch.float32 else 5e-3)
        if side:       # 32-bit outputs of the unrounded row
            close(s, want @ sw.double().t() + sb.double(), 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,v", [(3, 21), (2, 64), (5, 136)])
def test_head_norm_gate(dtype, H, v):
    g = gen(v)
    o, w = randn(7, H, v, g=g), randn(H * v, g=g)
    gate = randn(7, 9 + H * v, g=g, dtype=dtype)
    y = F().head_norm_gate(o.to(DEV), gate.to(DEV, dtype)[:, 9:], w.to(DEV),
                           1e-2)
    want = oracle.rms(o.double(), 1e-2).reshape(7, -1) * w.double() \
        * oracle.sigmoid(gate[:, 9:].double())
    close(y, want, 1e-5 if dtype == torch.float32 else 5e-3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_shared_small_ops_any_size(dtype):
    g = gen()
    gu = randn(5, 2 * 33, g=g, dtype=dtype)
    y = F().silu_mul_gateup(gu.to(DEV, dtype), 33)
    a = gu[:, :33].double()
    close(y, a * oracle.sigmoid(a) * gu[:, 33:].double(), 1e-2)
    lg = randn(4, 1001, g=g)
    lg[1, 1000] = lg[2, 0] = 99.0
    lg[3, 7] = lg[3, 500] = 99.0        # ties go to the lowest index
    got = F().greedy_sample(lg.to(DEV, dtype)).cpu()
    assert torch.equal(got, lg.to(dtype).float().argmax(-1))
    assert got[1:].tolist() == [1000, 0, 7]


def mlstm_oracle(proj, gates, H, dk, dv, cap, state, norm_w, eps):
    """One sequence from state (S, n, m) per head: normed and gated rows."""
    T = proj.shape[0]
    p = proj.double()
    q = p[:, :H * dk].view(T, H, dk) * dk ** -0.5
    k = p[:, H * dk:2 * H * dk].view(T, H, dk)
    v = p[:, 2 * H * dk:2 * H * dk + H * dv].view(T, H, dv)
    gate = p[:, 2 * H * dk + H * dv:]
    i = oracle.soft_cap(gates[:, :H].double(), cap)
    f = oracle.log_sigmoid(oracle.soft_cap(gates[:, H:].double(), cap))
    o, out = torch.zeros(T, H, dv, dtype=D), []
    for h in range(H):
        st = state[h]
        for t in range(T):
            o[t, h], st = oracle.mlstm_cell(q[t, h], k[t, h], v[t, h],
                                            float(i[t, h]), float(f[t, h]),
                                            st)
        out.append(st)
    return oracle.rms(o, eps).reshape(T, -1) * norm_w.double() \
        * oracle.sigmoid(gate), out


@pytest.mark.parametrize("dtype,by_token", [(torch.float32, True),
                                            (torch.bfloat16, True),
                                            (torch.bfloat16, False)])
@pytest.mark.parametrize("H,dk,dv,counts,lens,forget", [
    (2, 32, 64, [70, 2], [0, 5], 4.0),
    (1, 40, 136, [129, 64, 3], [7, 0, 0], 2.0),
    (3, 16, 24, [1, 1, 1], [0, 3, 9], 0.0),
    (1, 256, 72, [131], [4], 9.0)])
def test_mlstm(dtype, by_token, H, dk, dv, counts, lens, forget):
    """Token by token and by chunks, fresh slots (whatever they hold) and
    continued ones, slow and fast forgetting, gates beyond the cap."""
    g = gen(dk)
    n, cap, eps = sum(counts), 6.0, 1e-4
    proj = randn(n, 2 * H * (dk + dv), g=g, dtype=dtype)
    gates = randn(n, 2 * H, g=g, scale=3.0)
    gates[:, H:] += forget
    gates[n // 2, 0] = 40.0
    w = randn(H * dv, g=g)
    c = make_cache({"S": ((H, dk, dv), torch.float32),
                    "nm": ((2, H, dk + 1), torch.float32)}, lens)
    S0, nm0 = randn(len(lens), H, dk, dv, g=g), randn(len(lens), 2, H, dk + 1,
                                                     g=g)
    c.layers[0]["S"].copy_(S0)
    c.layers[0]["nm"].copy_(nm0)
    c.turn[0] = 1                       # slots may be at different turns
    turn = c.turn.tolist()
    b = c.batch(range(len(lens)), counts)
    y = F().mlstm(proj.to(DEV, dtype), gates.to(DEV), b, c,
                  c.layers[0]["S"], c.layers[0]["nm"], cap, w.to(DEV), eps,
                  by_token=by_token)
    at = 0
    for s, cnt in enumerate(counts):
        if lens[s] == 0:
            st = [(torch.zeros(dk, dv, dtype=D), torch.zeros(dk, dtype=D),
                   0.0) for _ in range(H)]
        else:
            st = [(S0[s, h].double(), nm0[s, turn[s], h, :dk].double(),
                   float(nm0[s, turn[s], h, dk])) for h in range(H)]
        want, st = mlstm_oracle(proj[at:at + cnt], gates[at:at + cnt], H, dk,
                                dv, cap, st, w, eps)
        close(y[at:at + cnt], want,
              2e-4 if dtype == torch.float32 else 1e-2)
        for h in range(H):
            close(c.layers[0]["S"][s, h], st[h][0], 2e-5)
            close(c.layers[0]["nm"][s, 1 - turn[s], h],
                  torch.cat([st[h][1], torch.tensor([st[h][2]], dtype=D)]),
                  2e-5)
        at += cnt


def test_mlstm_long_memory_survives_chunks():
    """A key written once, long ago, with a gate that stands out: its value
    comes back many chunks later, and the denominator's floor holds."""
    H, dk, dv, T = 1, 32, 64, 700
    g = gen(3)
    proj = randn(T, 2 * (dk + dv), g=g, scale=0.05, dtype=torch.bfloat16)
    gates = torch.zeros(T, 2)
    gates[:, 0], gates[:, 1] = -9.0, 20.0        # write little, keep all
    proj[3, dk:2 * dk] = proj[T - 1, :dk] = \
        randn(dk, g=g, dtype=torch.bfloat16)
    proj[3, 2 * dk:2 * dk + dv] = randn(dv, g=g, dtype=torch.bfloat16)
    gates[3, 0] = 8.0
    w = torch.ones(dv)
    for dtype, by_token in ((torch.float32, True), (torch.bfloat16, False)):
        c = make_cache({"S": ((H, dk, dv), torch.float32),
                        "nm": ((2, H, dk + 1), torch.float32)}, [0])
        y = F().mlstm(proj.to(DEV, dtype), gates.to(DEV), c.batch([0], [T]),
                      c, c.layers[0]["S"], c.layers[0]["nm"], 10.0,
                      w.to(DEV), 1e-6, by_token=by_token)
        st = [(torch.zeros(dk, dv, dtype=D), torch.zeros(dk, dtype=D), 0.0)]
        want, _ = mlstm_oracle(proj, gates, H, dk, dv, 10.0, st, w, 1e-6)
        # rows whose query is all but orthogonal to the one key that counts
        # are normed back to full size: those rows magnify any rounding
        assert float((y.cpu() - want).norm() / want.norm()) < 5e-3
        close(y[-1:], want[-1:], 5e-3)
        # without that token's value the last row is another one
        proj2 = proj.clone()
        proj2[3, 2 * dk:2 * dk + dv] = 0.0
        st = [(torch.zeros(dk, dv, dtype=D), torch.zeros(dk, dtype=D), 0.0)]
        other, _ = mlstm_oracle(proj2, gates, H, dk, dv, 10.0, st, w, 1e-6)
        assert util.rel(other[-1:], want[-1:]) > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_rank,rank,rot,dims", [(27, 19, 6, 6),
                                                  (56, 48, 16, 8),
                                                  (300, 72, 8, 8)])
def test_latent_prep_and_ring(dtype, q_rank, rank, rot, dims):
    """Both latent norms, the rotation at every position, ring rows modulo
    the capacity, and the way from ring to key buffer and back."""
    g = gen(rank)
    cap, lens, counts = 6, [0, 17, 4], [9, 1, 3]
    n = sum(counts)
    p = randn(n, q_rank + rank + rot + 5, g=g, dtype=dtype)
    wq, wk = randn(q_rank, g=g), randn(rank, g=g)
    eps, base = 1e-3, 700.0
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    inv = F().rope_inv_freq(dims, base, DEV)
    cq_want = oracle.rms(p[:, :q_rank].double(), eps) * wq.double()
    lat_want = []
    at = 0
    for l0, cnt in zip(lens, counts):
        for t in range(cnt):
            r = p[at, q_rank:q_rank + rank + rot].double()
            lat_want.append(torch.cat([
                oracle.rms(r[:rank], eps) * wk.double(),
                oracle.rotate(r[rank:], l0 + t, base, dims)]))
            at += 1
    lat_want = torch.stack(lat_want)

    c = make_cache({"ring": ((cap, rank + rot), dtype)}, lens)
    ring = c.layers[0]["ring"]
    old = randn(3, cap, rank + rot, g=g, dtype=dtype)
    ring.copy_(old)
    b = c.batch([0, 1, 2], counts)
    rows = b.key_rows(cap)
    buf = torch.zeros(rows.total, rank + rot, dtype=dtype, device=DEV)
    cq = F().latent_prep(p.to(DEV, dtype), b, c, wq.to(DEV), wk.to(DEV), inv,
                         buf, rows.own, eps)
    close(cq, cq_want, tol)
    F().latent_ring(b, c, rows, buf, ring, load=True)
    prior = [0, 5, 4]
    at, row = 0, 0
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        for j in range(l0 - prior[s], l0):         # cached rows, in order
            assert torch.equal(buf[row].float().cpu(), old[s, j % cap])
            row += 1
        close(buf[row:row + cnt], lat_want[at:at + cnt], tol)
        row += cnt
        at += cnt
    F().latent_ring(b, c, rows, buf, ring, load=False)
    at = 0
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        for j in range(max(0, cnt - cap), cnt):
            close(ring[s, (l0 + j) % cap], lat_want[at + j], tol)
        at += cnt
    keep = ring[2, (4 + 3) % cap].clone()          # not yet overwritten
    assert torch.equal(keep.float().cpu(), old[2, (4 + 3) % cap])
    # single tokens go straight into the ring
    c.lens_host = [3, 17, 4]
    c.lens.copy_(torch.tensor(c.lens_host, dtype=torch.int32))
    b1 = c.batch([1], [1])
    ring.copy_(old)
    F().latent_prep(p[9:10].to(DEV, dtype), b1, c, wq.to(DEV), wk.to(DEV),
                    inv, ring, None, eps)
    close(ring[1, 17 % cap], lat_want[9], tol)
    assert torch.equal(ring[0].float().cpu(), old[0])


def attention_oracle(q, kn, kr, v, pos0, window, scale, sink, rot_base,
                     rot_dims):
    """q [T, H, d1 + d2] unrotated at positions pos0..; keys 0.. rotated
    already."""
    T, H, _ = q.shape
    d1 = kn.shape[-1]
    o = torch.zeros(T, H, v.shape[-1], dtype=D)
    for t in range(T):
        p = pos0 + t
        lo = max(0, p - window + 1)
        for h in range(H):
            qr = oracle.rotate(q[t, h, d1:], p, rot_base, rot_dims)
            s = (kn[lo:p + 1, h] @ q[t, h, :d1] + kr[lo:p + 1] @ qr) * scale
            o[t, h] = oracle.sink_attend(s, v[lo:p + 1, h], sink[h])
    return o


@pytest.mark.parametrize("dtype,general", [(torch.float32, True),
                                           (torch.bfloat16, True),
                                           (torch.bfloat16, False)])
@pytest.mark.parametrize("H,d1,d2,dv,window,lens,counts", [
    (3, 24, 8, 40, 12, [0, 0], [70, 3]),
    (2, 128, 64, 128, 65, [0, 100], [66, 5]),
    (1, 16, 16, 24, 1, [0, 9], [5, 64]),
    (2, 8, 8, 8, 5000, [0], [150]),
    (1, 200, 56, 256, 33, [31], [40])])
def test_window_attention_prompt(dtype, general, H, d1, d2, dv, window, lens,
                                 counts):
    """A key at the window's last place outscores all others; one token
    further out it must be gone, and the sink always counts."""
    g = gen(d1)
    scale, base = (d1 + d2) ** -0.5, 300.0
    n = sum(counts)
    q = randn(n, H, d1 + d2, g=g, dtype=dtype)
    sink = randn(H, g=g, scale=2.0)
    gate = randn(n, H * dv, g=g, dtype=dtype)
    c = make_cache({}, lens)
    b = c.batch(range(len(lens)), counts)
    rows = b.key_rows(window)
    kv = torch.zeros(rows.total, H * (d1 + dv))
    lat = torch.zeros(rows.total, 5 * 8 + d2)
    want, at, row = [], 0, 0
    for l0, cnt in zip(lens, counts):
        kn = randn(l0 + cnt, H, d1, g=g, dtype=dtype)
        kr = randn(l0 + cnt, d2, g=g, dtype=dtype)
        v = randn(l0 + cnt, H, dv, g=g, dtype=dtype)
        # the last query's favourite is at the window's edge, the one
        # before it has its favourite just outside
        for t in (cnt - 1, cnt - 2):
            p, far = l0 + t, l0 + cnt - 1 - window + 1
            if t >= 0 and 0 <= far <= p:
                kn[far] = q[at + t, :, :d1] * 3.0
                kn[far] = kn[far].to(dtype).float()
        want.append(attention_oracle(
            q[at:at + cnt].double(), kn.double(), kr.double(), v.double(),
            l0, window, scale, sink.double(), base, d2))
        p0 = min(l0, window - 1)
        m = p0 + cnt
        kv[row:row + m, :H * d1] = kn[l0 - p0:].reshape(m, -1)
        kv[row:row + m, H * d1:] = v[l0 - p0:].reshape(m, -1)
        lat[row:row + m, -d2:] = kr[l0 - p0:]
        row += m
        at += cnt
    want = torch.cat(want).reshape(n, -1) * oracle.sigmoid(gate.double())
    y = F().attn_window_prompt(
        q.reshape(n, -1).to(DEV, dtype), kv.to(DEV, dtype),
        lat.to(DEV, dtype), b, c, rows, F().rope_inv_freq(d2, base, DEV),
        sink.to(DEV), gate.to(DEV, dtype), d1, d2, dv, window, scale,
        general=general)
    close(y, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype,general", [(torch.float32, True),
                                           (torch.bfloat16, True),
                                           (torch.bfloat16, False)])
@pytest.mark.parametrize("H,dim,rot,rank,dv,window,lens", [
    (3, 24, 8, 48, 40, 12, [0, 10, 11, 12, 13, 100]),
    (20, 16, 16, 160, 24, 200, [0, 198, 199, 200, 450]),
    (2, 128, 64, 512, 128, 333, [332, 700]),
    (1, 9, 6, 19, 11, 1, [0, 5]),
    (33, 8, 8, 64, 8, 64, [63, 64, 1000])])
def test_window_attention_decode(dtype, general, H, dim, rot, rank, dv,
                                 window, lens):
    """Absorbed single-token attention over a wrapped ring, with a key that
    stands out just inside and just outside the window."""
    g = gen(rank)
    scale, base = (dim + rot) ** -0.5, 300.0
    cap, nb = window, len(lens)
    c = make_cache({"ring": ((cap, rank + rot), dtype)}, lens)
    uk = randn(H, dim, rank, g=g, scale=rank ** -0.5, dtype=dtype)
    uv = randn(H, rank, dv, g=g, scale=rank ** -0.5, dtype=dtype)
    q = randn(nb, H, dim + rot, g=g, dtype=dtype)
    gate, sink = randn(nb, H * dv, g=g, dtype=dtype), randn(H, g=g)
    want = []
    for s, p in enumerate(lens):
        lat = randn(p + 1, rank + rot, g=g, dtype=dtype)
        qa = torch.einsum("d,dr->r", q[s, 0, :dim], uk[0])
        for far, gain in ((p - window + 1, 3.0), (p - window, 9.0)):
            if 0 <= far < p:
                lat[far, :rank] = (qa * gain * (dim + rot) ** 0.5
                                   / qa.norm()).to(dtype).float()
        for j in range(max(0, p + 1 - cap), p + 1):
            c.layers[0]["ring"][s, j % cap] = lat[j].to(DEV, dtype)
        kn = torch.einsum("tr,hdr->thd", lat[:, :rank].double(), uk.double())
        v = torch.einsum("tr,hrv->thv", lat[:, :rank].double(), uv.double())
        want.append(attention_oracle(q[s:s + 1].double(), kn,
                                     lat[:, rank:].double(), v, p, window,
                                     scale, sink.double(), base, rot))
    b = c.batch(range(nb), [1] * nb)
    qa = F().latent_absorb(q.reshape(nb, -1).to(DEV, dtype), uk.to(DEV, dtype),
                           b, c, F().rope_inv_freq(rot, base, DEV), rot)
    part = F().attn_window_decode(qa, c.layers[0]["ring"], b, c, rank, window,
                                  scale, general=general)
    y = F().latent_expand(part, sink.to(DEV), uv.to(DEV, dtype),
                          gate.to(DEV, dtype))
    want = torch.cat(want).reshape(nb, -1) * oracle.sigmoid(gate.double())
    close(y, want, 3e-5 if dtype == torch.float32 else 3e-2)


# ---------------------------------------------------------------------------
# models
# ---------------------------------------------------------------------------

_MODELS = {}


def model(name, dtype, tmp_path_factory=None):
    """(loaded model, configuration, weights), made once."""
    import lfmq
    key = (name, dtype)
    if key not in _MODELS:
        import tempfile
        cfg = util.CONFIGS[name]
        w = util.weights(cfg, seed=len(name))
        with tempfile.TemporaryDirectory() as d:
            m = lfmq.load(util.write_checkpoint(d, cfg, w), device=DEV,
                          dtype=dtype)
        _MODELS[key] = (m, cfg, w)
    return _MODELS[key]


def stepper(m, max_tokens=4096, n=1):
    from lfmq.models.generation import PackedStepper
    return PackedStepper(m, max_tokens, n)


def run(m, toks, cuts=(), st=None, rid="r"):
    """All logits of one sequence, fed in portions that end at `cuts`."""
    st = st or stepper(m)
    out, ends = [], [c for c in cuts if c < len(toks)] + [len(toks)]
    a = 0
    for e in ends:
        out.append(st.step([(rid, toks[a:e], list(range(e - a)))]))
        a = e
    st.end([rid])
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(util.CONFIGS))
def test_prompt_matches_oracle(name, dtype):
    m, cfg, w = model(name, dtype)
    for n in (1, 2, 37, 150):
        t = util.tokens(cfg, n, n)
        assert util.rel(run(m, t), util.expected(w, cfg, t)) < TOL[dtype], n


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_after_every_layer_run(dtype):
    m, cfg, w = model("mixed", dtype)
    t = util.tokens(cfg, 30)
    want, got = [], []
    oracle.forward(w, cfg, t, want)
    c = m.make_cache(1, max_seq=64)
    with torch.no_grad():
        m.forward_tokens(torch.tensor(t, device=DEV), c.batch([0], [30]), c,
                         trace=got)
    assert len(got) == len(want) == 6
    for a, b in zip(got, want):
        assert a.dtype == torch.float32
        assert util.rel(a, b) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "attention_first", "odd"])
def test_decode_token_by_token(name, dtype):
    m, cfg, w = model(name, dtype)
    t = util.tokens(cfg, 60, 5)
    want = util.expected(w, cfg, t)
    assert util.rel(run(m, t, range(1, 60)), want) < TOL[dtype]
    assert util.rel(run(m, t, range(20, 60)), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [2, 3, 7, 32, 65])
def test_portions(size, dtype):
    """However a prompt is cut, and with single tokens in between."""
    for name in ("mixed", "odd"):
        m, cfg, w = model(name, dtype)
        t = util.tokens(cfg, 140, 6)
        want = util.expected(w, cfg, t)
        assert util.rel(run(m, t, range(size, 140, size)), want) < TOL[dtype]
        cuts = sorted({*range(size, 140, size), *range(size + 1, 140, size)})
        assert util.rel(run(m, t, cuts), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd", "wide_window"])
def test_unequal_batch_and_slots_used_again(name, dtype):
    """Requests of several lengths together, decoded together while the
    short ones end; their slots serve the next batch."""
    m, cfg, w = model(name, dtype)
    st = stepper(m, 400, 2)
    for rnd in range(3):
        lens = [1, 9, 70, 33] if rnd % 2 == 0 else [40, 2, 5]
        tail = [6, 3, 20, 11]
        req = [util.tokens(cfg, n + k, 10 * rnd + n)
               for n, k in zip(lens, tail)]
        want = [util.expected(w, cfg, t) for t in req]
        at = list(lens)
        lg = st.step([(i, t[:n], list(range(n)))
                      for i, (t, n) in enumerate(zip(req, lens))])
        assert util.rel(lg, torch.cat([x[:n] for x, n in zip(want, lens)])) \
            < TOL[dtype]
        live = list(range(len(req)))
        while live:
            lg = st.step([(i, [req[i][at[i]]], [0]) for i in live])
            assert util.rel(lg, torch.stack([want[i][at[i]] for i in live])) \
                < TOL[dtype]
            for i in live:
                at[i] += 1
            done = [i for i in live if at[i] == len(req[i])]
            st.end(done)
            live = [i for i in live if i not in done]
        assert st.cache.free_slots == st.cache.n_slots


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_step_of_prompts_and_single_tokens(dtype):
    """A step may bring portions for some sequences, one token for others."""
    m, cfg, w = model("mixed", dtype)
    a, b, c = (util.tokens(cfg, n, n) for n in (50, 61, 4))
    wa, wb, wc = (util.expected(w, cfg, t) for t in (a, b, c))
    st = stepper(m)
    st.step([("a", a[:49], []), ("b", b[:30], [])])
    lg = st.step([("b", b[30:], list(range(31))), ("a", a[49:], [0]),
                  ("c", c, [0, 3])])
    want = torch.cat([wb[30:], wa[49:], wc[:1], wc[3:]])
    assert util.rel(lg, want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_through_the_ring(dtype):
    """The rings of 5 and 12 rows wrap many times."""
    m, cfg, w = model("mixed", dtype)
    t = util.tokens(cfg, 300, 3)
    want = util.expected(w, cfg, t)
    assert util.rel(run(m, t, range(4, 300)), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_window_edge_in_the_model(dtype):
    """One latent layer: a token whose key stands out is seen by the query
    window - 1 tokens later and not by the one after it."""
    import copy
    import tempfile

    import lfmq
    W = 9
    cfg = util.config([util.latent(heads=2, dim=16, rot=8, vdim=32,
                                   kv_rank=32, window=W, base=1e6)])
    w = util.weights(cfg, 9)
    w = copy.deepcopy(w)
    w["l0.mix.uq"] *= 2.5
    w["l0.mix.o"] *= 3
    with tempfile.TemporaryDirectory() as d:
        m = lfmq.load(util.write_checkpoint(d, cfg, w), device=DEV,
                      dtype=dtype)
    t = util.tokens(cfg, 2 * W + 20, 2)
    t2 = list(t)
    t2[5] = (t[5] + 1) % cfg["vocab"]          # another key at position 5
    want, want2 = util.expected(w, cfg, t), util.expected(w, cfg, t2)
    edge = 5 + W - 1
    seen = float((want[edge] - want2[edge]).abs().max())
    assert seen > 1e-2
    # token 6 differs too (its bigram), so the last one touched is edge + 1
    assert float((want[edge + 2] - want2[edge + 2]).abs().max()) < 1e-12
    for cuts in ((), range(4, len(t)), (6, 12, 14, 20)):
        a, b = run(m, t, cuts), run(m, t2, cuts)
        assert util.rel(a, want) < TOL[dtype]
        assert util.rel(b, want2) < TOL[dtype]
        assert float((a[edge] - b[edge]).abs().max()) > 0.5 * seen
        assert float((a[edge + 2:] - b[edge + 2:]).abs().max()) < 1e-5


def greedy(w, cfg, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(util.expected(w, cfg, t)[-1].argmax()))
    return t


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(name):
    """generate(), generate_batch() and the captured graph agree with the
    oracle, in 32 bits."""
    from lfmq.models.generation import generate_batch
    from lfmq.models.graph import GraphDecoder
    m, cfg, w = model(name, torch.float32)
    prompts = [util.tokens(cfg, n, n) for n in (3, 17, 17)]
    want = [greedy(w, cfg, p, 20) for p in prompts]
    assert generate_batch(m, prompts, 20) == want
    same = torch.tensor(prompts[1:], device=DEV)
    assert m.generate(same, max_new_tokens=20).tolist() == want[1:]
    # replays with eager work and new prompts in between
    dec = GraphDecoder(m, 3, max_seq=80, max_new_tokens=64)
    pad = torch.zeros(3, 17, dtype=torch.int64)
    for i, p in enumerate(prompts):
        pad[i, :len(p)] = torch.tensor(p)
    for _ in range(3):
        dec.prefill(pad, lengths=[3, 17, 17])
        got = torch.cat([dec.decode(7), dec.decode(13)], dim=1).cpu()
        torch.cuda.synchronize()
        for i, p in enumerate(prompts):
            assert got[i].tolist() == want[i][len(p):]
        assert generate_batch(m, prompts[:1], 4)[0] == want[0][:7]


def test_graph_equals_eager_in_16_bits():
    from lfmq.models.graph import GraphDecoder
    m, cfg, _ = model("mixed", torch.bfloat16)
    ids = torch.tensor([util.tokens(cfg, 30, 1), util.tokens(cfg, 30, 2)],
                       device=DEV)
    dec = GraphDecoder(m, 2, max_seq=100, max_new_tokens=64)
    dec.prefill(ids)
    got = dec.decode(40)
    assert torch.equal(torch.cat([ids, got], 1),
                       m.generate(ids, max_new_tokens=40))


def test_sampling_and_eos():
    import lfmq
    from lfmq.models.generation import generate_batch
    m, cfg, w = model("mixed", torch.float32)
    p = [util.tokens(cfg, 3, 3), util.tokens(cfg, 8, 8)]
    full = generate_batch(m, p, 12)
    eos = full[0][5]
    gc = lfmq.GenerationConfig(max_new_tokens=12, eos_token_id=eos)
    cut = generate_batch(m, p, gen_cfg=gc)
    assert cut[0] == full[0][:full[0].index(eos, 3) + 1]
    gc = lfmq.GenerationConfig(max_new_tokens=5, greedy=False,
                               temperature=0.8)
    a, b = (generate_batch(m, p, gen_cfg=gc, generator=torch.Generator(
        device=DEV).manual_seed(4)) for _ in range(2))
    assert a == b and all(len(x) == len(y) + 5 for x, y in zip(a, p))


def test_server_and_cli(tmp_path):
    from fastapi.testclient import TestClient
    from typer.testing import CliRunner
    from lfmq.cli import app as cli
    from lfmq.obs.serve import make_app
    m, cfg, w = model("mixed", torch.float32)
    p = [util.tokens(cfg, 3, 3), util.tokens(cfg, 8, 8)]
    want = [greedy(w, cfg, x, 6) for x in p]
    http = TestClient(make_app(m))
    for ids, out in (([p[0]], [want[0]]), (p, want)):
        r = http.post("/generate", json={"input_ids": ids,
                                         "max_new_tokens": 6})
        assert r.status_code == 200 and r.json()["output_ids"] == out
    path = util.write_checkpoint(tmp_path / "m", cfg, w)
    r = CliRunner().invoke(cli, [
        "generate", "--ckpt", path, "--dtype", "float32",
        "--max-new-tokens", "6"] + [a for x in p for a in
                                    ("--prompt", ",".join(map(str, x)))])
    assert r.exit_code == 0, r.output
    assert [x for x in r.output.split("\n") if "," in x] == \
        [",".join(map(str, x)) for x in want]


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_runner(tmp_path, monkeypatch, capsys, dtype):
    from lfmq import replay
    cfg = util.CONFIGS["mixed"]
    w = util.weights(cfg, 1)
    path = util.write_checkpoint(tmp_path / "m", cfg, w)
    (tmp_path / "out").mkdir()
    a, b = util.tokens(cfg, 20, 1), util.tokens(cfg, 9, 2)
    steps = [{"step": 0, "end": [],
              "entries": [{"id": "a", "tokens": a[:18], "want": [4, 17]},
                          {"id": "b", "tokens": b[:8], "want": []}]},
             {"step": 1, "end": ["b"],
              "entries": [{"id": "b", "tokens": b[8:], "want": [0]},
                          {"id": "a", "tokens": a[18:19], "want": [0]}]},
             {"step": 2, "end": ["a"],
              "entries": [{"id": "a", "tokens": a[19:], "want": [0]}]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "".join(json.dumps(s) + "\n" for s in steps)))
    assert replay.main(["--model", path, "--dtype", str(dtype).split(".")[1],
                        "--out", str(tmp_path / "out"), "--max-tokens",
                        "40"]) == 0
    assert [x for x in capsys.readouterr().out.split("\n") if x] == \
        ["done 0", "done 1", "done 2"]
    wa, wb = util.expected(w, cfg, a), util.expected(w, cfg, b)
    for n, want in enumerate(([wa[4], wa[17]], [wb[8], wa[18]], [wa[19]])):
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{n}.f32",
                                           dtype="<f4"))
        want = torch.stack(want)
        assert util.rel(got.view(want.shape), want) < TOL[dtype]


def test_quantized_round_trip(tmp_path):
    """RTN swaps the projections for packed ones; saved and loaded, it
    gives the same logits, near the 16-bit model's."""
    import lfmq
    from lfmq.models.qlinear import QLinear
    cfg = lfmq.models.registry.RapivikConfig.tiny()
    base = lfmq.build_model(cfg, seed=0)
    for p in base.parameters():
        if p.dim() == 2:
            p.data.mul_(2.0)
    base = base.to(DEV)
    ids = torch.randint(0, cfg.vocab_size, (2, 40), generator=gen()).to(DEV)
    with torch.no_grad():
        ref = base(ids, base.make_cache(2, max_seq=64)).float()
    qc = lfmq.QuantConfig(scheme="rtn", bits=8, group_size=64)
    q = lfmq.quantize(base, qc)
    assert isinstance(q.blocks["l0"].mixer.in_proj, QLinear)
    with torch.no_grad():
        a = q(ids, q.make_cache(2, max_seq=64)).float()
    assert float((a - ref).norm() / ref.norm()) < 0.1
    lfmq.save(q, str(tmp_path), qc)
    q2 = lfmq.load(str(tmp_path), device=DEV)
    with torch.no_grad():
        b = q2(ids, q2.make_cache(2, max_seq=64)).float()
    assert torch.equal(a, b)
    out = q2.generate(ids, max_new_tokens=6)
    assert out.shape == (2, 46)
