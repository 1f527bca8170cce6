"""Zatasun on the GPU against the plain oracle: every mechanism alone, then
whole models — prompts, portions, decoding, unequal batches, slots used
again, far keys, generation."""
import io
import json

import numpy as np
import pytest
import torch

import zatasun_oracle as oracle
import zatasun_util as util
from test_gpu_rapivik import (DEV, DTYPES, F, close, gen, make_cache, randn,
                              run, stepper)

pytestmark = pytest.mark.gpu
D = torch.float64
TOL = {torch.float32: 3e-5, torch.bfloat16: 4e-2}
SMALL = {torch.float32: 1e-5, torch.bfloat16: 5e-3}


def empty_view(n, cols, pad, dtype):
    """Columns pad.. of a wider buffer, as the mixers write them."""
    return torch.full((n, cols + pad), 7.0, dtype=dtype, device=DEV)[:, pad:]


# ---------------------------------------------------------------------------
# mechanisms
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 64), (3, 51), (2051, 96),
                                        (5, 2052), (2050, 53)])
def test_embed_and_post_norm(dtype, rows, width):
    g = gen(rows + width)
    table, y = (randn(n, width, g=g, dtype=dtype) for n in (40, rows))
    w, we, wo = (randn(width, g=g) for _ in range(3))
    tok = torch.randint(0, 40, (rows,), generator=g)
    eps = 1e-2
    x, h = F().embed_norm(tok.to(DEV), table.to(DEV, dtype), we.to(DEV), eps)
    want = oracle.rms(table[tok].double(), eps) * we.double()
    close(x, want, 1e-6)
    assert x.dtype == torch.float32 and h.dtype == dtype
    assert torch.equal(h, x.to(dtype))
    x0 = x.clone()
    h = F().post_norm(x, y.to(DEV, dtype), w.to(DEV), eps)
    want = x0.cpu().double() + oracle.rms(y.double(), eps) * w.double()
    close(x, want, 1e-6)
    assert torch.equal(h, x.to(dtype))
    x = x0.clone()
    h = F().post_norm(x, y.to(DEV, dtype), w.to(DEV), eps, wo.to(DEV), 0.3)
    close(x, want, 1e-6)
    close(h, oracle.rms(want, eps) * wo.double() * 0.3, SMALL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,width,top,shared", [
    (1, 64, 1, True), (7, 51, 3, False), (2100, 40, 2, True)])
def test_post_norm_of_a_sum_of_experts(dtype, n, width, top, shared):
    from lfmq.models.mixers import ExpertSum
    g = gen(n)
    rows, sh = (randn(k, width, g=g, dtype=dtype) for k in (n * top, n))
    x, w, sg = randn(n, width, g=g), randn(width, g=g), randn(n, g=g)
    pos = torch.randperm(n * top, generator=g).view(n, top)
    y = rows[pos].double().sum(1)
    if shared:
        y = y + sg[:, None].double() * sh.double()
    parts = ExpertSum(rows.to(DEV, dtype), pos.int().to(DEV),
                      sh.to(DEV, dtype) if shared else None,
                      sg.to(DEV) if shared else None)
    xd = x.to(DEV)
    h = F().post_norm_experts(xd, parts, w.to(DEV), 1e-3)
    close(xd, x.double() + oracle.rms(y, 1e-3) * w.double(), 1e-5)
    assert torch.equal(h, xd.to(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,dv,dims", [(4, 2, 32, 40, 32),
                                             (3, 1, 13, 9, 6),
                                             (6, 6, 24, 72, 8)])
def test_qk_prep(dtype, H, G, dim, dv, dims):
    """Norms over the whole projections, rotation at every position, keys
    and values at their positions in the cache and nowhere else."""
    g = gen(dim)
    lens, counts, cap, eps, base = [0, 40, 3], [5, 1, 2], 44, 1e-2, 300.0
    n, cols = sum(counts), H * dim + G * (dim + dv)
    p = randn(n, cols + 3, g=g, dtype=dtype)
    wq, wk = randn(H * dim, g=g), randn(G * dim, g=g)
    c = make_cache({"k": ((cap, G, dim), dtype), "v": ((cap, G, dv), dtype)},
                   lens, cap)
    kc, vc = c.layers[0]["k"], c.layers[0]["v"]
    b = c.batch([0, 1, 2], counts)
    inv = F().rope_inv_freq(dims, base, DEV, util.SCALING)
    q = F().qk_prep(p.to(DEV, dtype)[:, 2:2 + cols], b, c, wq.to(DEV),
                    wk.to(DEV), inv, kc, vc, eps)
    f = oracle.frequencies(dims, base, util.SCALING)
    p = p[:, 2:2 + cols].double()
    qw = (oracle.rms(p[:, :H * dim], eps) * wq.double()).view(n, H, dim)
    kw = (oracle.rms(p[:, H * dim:H * dim + G * dim], eps)
          * wk.double()).view(n, G, dim)
    at, used = 0, torch.zeros(3, cap, dtype=torch.bool)
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        for t in range(cnt):
            close(q[at].view(H, dim), oracle.rotate(qw[at], l0 + t, f),
                  SMALL[dtype])
            close(kc[s, l0 + t], oracle.rotate(kw[at], l0 + t, f),
                  SMALL[dtype])
            assert torch.equal(vc[s, l0 + t].float().cpu().reshape(-1),
                               p[at, -G * dv:].float())
            used[s, l0 + t] = True
            at += 1
    assert float(kc[~used.to(DEV)].abs().max()) == 0.0
    assert float(vc[~used.to(DEV)].abs().max()) == 0.0


def filled_attention(H, G, dim, dv, lens, counts, dtype, g, cap):
    """Cache holding every position up to lens + counts, ready queries."""
    c = make_cache({"k": ((cap, G, dim), dtype), "v": ((cap, G, dv), dtype)},
                   lens, cap)
    k, v = (randn(len(lens), cap, G, d, g=g, dtype=dtype) for d in (dim, dv))
    q = randn(sum(counts), H, dim, g=g, dtype=dtype)
    sink = randn(H, g=g)
    return c, q, k, v, sink


def attention_want(q, k, v, sink, lens, counts, scale, gain):
    H, G = q.shape[1], k.shape[2]
    out, at = [], 0
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        for t in range(cnt):
            p = l0 + t + 1
            out.append(torch.cat([oracle.sink_attend(
                (k[s, :p, h // (H // G)].double() @ q[at, h].double())
                * scale, v[s, :p, h // (H // G)].double(), sink[h].double())
                for h in range(H)]))
            at += 1
    return gain * torch.stack(out)


@pytest.mark.parametrize("dtype,general", [(torch.float32, True),
                                           (torch.bfloat16, True),
                                           (torch.bfloat16, False)])
@pytest.mark.parametrize("H,G,dim,dv,lens,counts", [
    (4, 2, 24, 40, [0, 0], [70, 3]),
    (8, 1, 128, 128, [0, 100], [66, 5]),
    (3, 3, 16, 24, [0, 9], [5, 64]),
    (2, 1, 8, 8, [31], [130]),
    (2, 2, 200, 256, [31], [40]),
    # one token each: the decode kernel, key ranges of many sizes
    (4, 2, 24, 40, [0, 1, 31, 32], [1, 1, 1, 1]),
    (8, 2, 128, 128, [129, 700], [1, 1]),
    (18, 2, 40, 72, [63, 64, 300], [1, 1, 1]),
    (5, 5, 16, 256, [511], [1]),
    (32, 1, 256, 64, [257], [1])])
def test_grouped_attention(dtype, general, H, G, dim, dv, lens, counts):
    """Far, first and last keys that outscore all others, in every place
    of a key tile; rows past a sequence's end hold garbage."""
    g = gen(dim + dv)
    cap = max(a + b for a, b in zip(lens, counts)) + 37
    c, q, k, v, sink = filled_attention(H, G, dim, dv, lens, counts, dtype, g,
                                        cap)
    scale, at = dim ** -0.5, 0
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        k[s, l0 + cnt:], v[s, l0 + cnt:] = 1e4, 1e4
        for t in range(cnt):
            j = (0, l0 + t, (l0 + t) // 2, max(0, l0 + t - 1))[t % 4]
            h = t % H
            d = k[s, j, h // (H // G)]
            q[at, h] = (8 * d / d.norm() * dim ** 0.5).to(dtype).float() \
                / max(float(d.norm()), 1e-3) * 2
            at += 1
        sink[t % H] = 9.0
    q = q.to(dtype).float()
    c.layers[0]["k"].copy_(k)
    c.layers[0]["v"].copy_(v)
    b = c.batch(range(len(lens)), counts)
    out = empty_view(sum(counts), H * dv, 5, dtype)
    F().attn_grouped(q.to(DEV, dtype).view(len(q), -1), c.layers[0]["k"],
                     c.layers[0]["v"], b, c, sink.to(DEV), out, scale, 0.7,
                     general=general)
    close(out, attention_want(q, k, v, sink, lens, counts, scale, 0.7),
          2e-5 if dtype == torch.float32 else 1e-2)
    assert float(out._base[:, :5].min()) == 7.0


def lru_inputs(C, blocks, taps, n, dtype, g):
    nb = C // blocks
    return dict(
        proj=randn(n, 2 * C + 3, g=g, dtype=dtype), xb=randn(C, g=g),
        yb=randn(C, g=g), cw=randn(C, taps, g=g), cb=randn(C, g=g),
        gw=randn(blocks, 2, nb, nb, g=g, scale=nb ** -0.5, dtype=dtype),
        gb=randn(blocks, 2, nb, g=g), lam=randn(C, g=g, scale=2.0) - 3)


def lru_run(a, c, b, C, dtype, gain, general=False):
    dev = {k: v.to(DEV) for k, v in a.items()}
    p = a["proj"].to(DEV, dtype)
    out = empty_view(b.n, C, 3, dtype)
    st = c.layers[0]
    F().gated_lru(p[:, C + 1:2 * C + 1], p[:, 1:C + 1], b, c, dev["xb"],
                  dev["yb"], dev["cw"].t().contiguous(), dev["cb"],
                  dev["gw"].to(dtype), dev["gb"], dev["lam"], st["conv"],
                  st["S"], out, -8.0, gain, general=general)
    return out


def lru_want(a, rows, C, S, past, dtype):
    p = a["proj"][rows].double()
    x = p[:, C + 1:2 * C + 1] + a["xb"].double()
    u = oracle.causal_conv(x, a["cw"].double(), a["cb"].double(),
                           past.double())
    u = u.to(dtype).double()       # the convolution's output may round
    d, z = oracle.lru_gates(u, a["gw"][:, 0].double(),
                            a["gb"][:, 0].double(), a["gw"][:, 1].double(),
                            a["gb"][:, 1].double(), a["lam"].double())
    out, S = oracle.lru(d, z, S.double())
    y = oracle.gelu_tanh(p[:, 1:C + 1] + a["yb"].double())
    return out * y, S, x


@pytest.mark.parametrize("dtype,general", [(torch.float32, True),
                                           (torch.bfloat16, True),
                                           (torch.bfloat16, False)])
@pytest.mark.parametrize("C,blocks,taps,counts,lens", [
    (64, 4, 4, [70, 2, 1], [0, 5, 0]),
    (80, 2, 4, [129, 64, 3], [7, 0, 2]),
    (48, 1, 2, [1, 1, 1], [0, 3, 9]),
    (32, 2, 1, [65, 1], [0, 4]),
    (96, 3, 7, [4, 66], [2, 3]),
    (768, 1, 4, [66], [9]),
    (640, 1, 4, [1] * 18, [0, 1, 2, 3, 4, 50] * 3),
    (35, 5, 3, [9, 1], [1, 0])])
def test_gated_lru(dtype, general, C, blocks, taps, counts, lens):
    """Prompts, portions and single tokens; fresh slots (whatever they
    hold) and continued ones; the state and the convolution's inputs."""
    g = gen(C)
    n, gain = sum(counts), 0.6
    a = lru_inputs(C, blocks, taps, n, dtype, g)
    c = make_cache({"S": ((C,), torch.float32),
                    "conv": ((taps, C), torch.float32)}, lens)
    S0, ring0 = randn(len(lens), C, g=g), randn(len(lens), taps, C, g=g)
    c.layers[0]["S"].copy_(S0)
    c.layers[0]["conv"].copy_(ring0)
    b = c.batch(range(len(lens)), counts)
    out = lru_run(a, c, b, C, dtype, gain, general)
    at, tol = 0, 2e-5 if dtype == torch.float32 else 1e-2
    for s, (l0, cnt) in enumerate(zip(lens, counts)):
        past = torch.zeros(taps - 1, C)
        for j in range(1, taps):
            if l0 - j >= 0:
                past[taps - 1 - j] = ring0[s, (l0 - j) % taps]
        S = S0[s] if l0 else torch.zeros(C)
        want, S, x = lru_want(a, slice(at, at + cnt), C, S, past, dtype)
        close(out[at:at + cnt], gain * want, tol)
        # a 16-bit step on the convolution's output moves the state a bit
        close(c.layers[0]["S"][s], S, 2e-5 if dtype == torch.float32 else 4e-3)
        for i in range(max(0, cnt - taps), cnt):
            close(c.layers[0]["conv"][s, (l0 + i) % taps], x[i], 1e-6)
        at += cnt
    assert float(out._base[:, :3].min()) == 7.0


@pytest.mark.parametrize("dtype", DTYPES)
def test_gated_lru_long_memory_and_decay_near_one(dtype):
    """One input that stands out is still in the state hundreds of tokens
    and many tiles later, where a is all but one and sqrt(1 - a^2) tiny."""
    C, T = 64, 700
    g = gen(4)
    a = lru_inputs(C, 2, 4, T, dtype, g)
    a["proj"] *= 0.02
    a["proj"] = a["proj"].to(dtype).float()
    a["xb"] *= 0.02
    a["cb"] *= 0.02
    a["lam"] = torch.linspace(-16, -8, C)
    a["proj"][5, C + 1:2 * C + 1] = 40.0
    base = lru_want(a, slice(0, T), C, torch.zeros(C), torch.zeros(3, C),
                    dtype)[0]
    b = {**a, "proj": a["proj"].clone()}
    b["proj"][5, C + 1:2 * C + 1] = 0.0
    other = lru_want(b, slice(0, T), C, torch.zeros(C), torch.zeros(3, C),
                     dtype)[0]
    assert util.rel(other[-1:], base[-1:]) > 0.3
    for cuts in ((), (64,), (3, 6, 8, 400)):
        c = make_cache({"S": ((C,), torch.float32),
                        "conv": ((4, C), torch.float32)}, [0])
        got, at = [], 0
        for e in (*cuts, T):
            bt = c.batch([0], [e - at])
            got.append(lru_run({**a, "proj": a["proj"][at:e]}, c, bt, C,
                               dtype, 1.0).cpu())
            c.advance(torch.zeros(e - at, dtype=torch.int64, device=DEV), bt)
            at = e
        got = torch.cat(got).double()
        assert float((got - base).norm() / base.norm()) < \
            (1e-4 if dtype == torch.float32 else 1e-2)
        assert util.rel(got[-1:], base[-1:]) < 1e-2


@pytest.mark.parametrize("dtype,general", [(torch.float32, True),
                                           (torch.bfloat16, True),
                                           (torch.bfloat16, False)])
@pytest.mark.parametrize("n,width,E,top,ff,shared", [
    (1, 64, 7, 2, 40, True), (3, 96, 3, 3, 24, False),
    (17, 64, 100, 5, 32, True), (40, 72, 2, 1, 136, True),
    (300, 128, 4, 2, 200, False), (1, 1032, 8, 4, 1040, True),
    (700, 64, 70, 1, 48, False), (9, 51, 6, 2, 21, True)])
def test_experts(dtype, general, n, width, E, top, ff, shared):
    """Router choices, scores and the shared gate; every expert's rows for
    the tokens that chose it, weighted on the way in; crowded, single and
    unused experts."""
    g = gen(n + E)
    lim, alpha, beta = 0.6, 1.702, 1.0
    h = randn(n, width, g=g, dtype=dtype)
    r = randn(E + shared, width, g=g, scale=3 * width ** -0.5, dtype=dtype)
    if E > 4:
        r[1] = r[0] * 0.0 - 1e-3        # an expert of middling scores
    gu = randn(E, 2 * ff, width, g=g, scale=1.5 * width ** -0.5, dtype=dtype)
    down = randn(E, width, ff, g=g, scale=ff ** -0.5, dtype=dtype)
    rows, pos, sg = F().moe(h.to(DEV, dtype), r.to(DEV, dtype),
                            gu.to(DEV, dtype), down.to(DEV, dtype), top,
                            (lim, alpha, beta), general=general)
    assert sorted(pos.flatten().tolist()) == list(range(n * top))
    got = rows[pos.long()].cpu()
    w = {f"e{e}.{k}": t.double() for e in range(E) for k, t in
         (("gate", gu[e, :ff]), ("up", gu[e, ff:]), ("down", down[e]))}
    z = (h.double() @ r[:E].double().t()).sort(-1, descending=True)[0]
    clear = z[:, top - 1] - (z[:, top] if top < E else -99.0) > 1e-4
    want, have = [], []
    for t in range(n):
        if not clear[t]:
            continue
        ids, ss = oracle.route(h[t].double(), r[:E].double(), top)
        y = sum(oracle.expert(s * h[t].double(), w[f"e{e}.gate"],
                              w[f"e{e}.up"], w[f"e{e}.down"], lim)
                for e, s in zip(ids, ss))
        want.append(y)
        have.append(got[t].double().sum(0))
    assert len(want) > 0.9 * n
    close(torch.stack(have), torch.stack(want),
          1e-5 if dtype == torch.float32 else 2e-2)
    if shared:
        close(sg, oracle.sigmoid(h.double() @ r[E].double()), 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [33, 64])
def test_clamped_glu(dtype, ff):
    g = gen(ff)
    gu = randn(9, 2 * ff, g=g, scale=2.0, dtype=dtype)
    y = F().clamped_glu(gu.to(DEV, dtype), 1.5, 1.702, 1.0)
    a = torch.clamp(gu[:, :ff].double(), max=1.5)
    u = torch.clamp(gu[:, ff:].double(), -1.5, 1.5)
    close(y, a * oracle.sigmoid(1.702 * a) * (u + 1), SMALL[dtype])


# ---------------------------------------------------------------------------
# whole models
# ---------------------------------------------------------------------------

_MODELS = {}


def model(name, dtype):
    """(loaded model, configuration, weights), made once."""
    import tempfile

    import lfmq
    key = (name, dtype)
    if key not in _MODELS:
        cfg = util.CONFIGS[name]
        w = util.weights(cfg, seed=len(name))
        with tempfile.TemporaryDirectory() as d:
            m = lfmq.load(util.write_checkpoint(d, cfg, w), device=DEV,
                          dtype=dtype)
        _MODELS[key] = (m, cfg, w)
    return _MODELS[key]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(util.CONFIGS))
def test_prompt_matches_oracle(name, dtype):
    m, cfg, w = model(name, dtype)
    for n in (1, 2, 37, 150):
        t = util.tokens(cfg, n, n)
        assert util.rel(run(m, t), util.expected(w, cfg, t)) < TOL[dtype], n


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_after_every_layer(dtype):
    m, cfg, w = model("mixed", dtype)
    t = util.tokens(cfg, 30)
    want, got = [], []
    oracle.forward(w, cfg, t, want)
    c = m.make_cache(1, max_seq=64)
    with torch.no_grad():
        m.forward_tokens(torch.tensor(t, device=DEV), c.batch([0], [30]), c,
                         trace=got)
    assert len(got) == len(want) == 4
    for a, b in zip(got, want):
        assert a.dtype == torch.float32
        assert util.rel(a, b) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "experts_first", "odd"])
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
@pytest.mark.parametrize("name", ["mixed", "odd"])
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
def test_batch_equals_alone(dtype):
    """A request's logits do not depend on its neighbours."""
    m, cfg, _ = model("mixed", dtype)
    req = [util.tokens(cfg, n, n) for n in (3, 64, 21)]
    st = stepper(m)
    both = st.step([(i, t, list(range(len(t)))) for i, t in enumerate(req)])
    alone = torch.cat([run(m, t) for t in req])
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert float((both - alone).float().norm() / alone.float().norm()) < tol


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
def test_long_decoding(dtype):
    m, cfg, w = model("mixed", dtype)
    t = util.tokens(cfg, 300, 3)
    want = util.expected(w, cfg, t)
    assert util.rel(run(m, t, range(4, 300)), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_token_in_the_model(dtype):
    """One layer whose recurrence forgets at once: what a far token changes
    comes through attention, in prompts, portions and decoding."""
    import tempfile

    import lfmq
    cfg = util.config([util.layer(heads=4, kv=2, dim=32, vdim=32, rot=8,
                                  scale=0.4)])
    w = util.weights(cfg, 9)
    w["l0.mix.right.lam"] = torch.full_like(w["l0.mix.right.lam"], 6.0)
    # token 96 is token 95 negated and queries are keys negated: its query
    # is the key of 95, and its own key is as far off as can be
    w["embed"][96] = -w["embed"][95]
    w["l0.mix.left.q"] = -w["l0.mix.left.k"].view(2, 1, 32, -1).expand(
        2, 2, 32, cfg["width"]).reshape(128, -1)
    w["l0.mix.left.q.norm"] *= 2
    w["l0.mix.left.sink"] = w["l0.mix.left.sink"] * 0 + 4
    with tempfile.TemporaryDirectory() as d:
        m = lfmq.load(util.write_checkpoint(d, cfg, w), device=DEV,
                      dtype=dtype)
    t = [x % 90 for x in util.tokens(cfg, 260, 2)]
    t[3], t[250] = 95, 96
    t2 = list(t)
    t2[3] = 94
    want, want2 = util.expected(w, cfg, t), util.expected(w, cfg, t2)
    seen = float((want[250] - want2[250]).abs().max())
    assert seen > 0.1
    for cuts in ((), range(240, 260), (64, 129, 250)):
        a, b = run(m, t, cuts), run(m, t2, cuts)
        assert util.rel(a, want) < TOL[dtype]
        assert util.rel(b, want2) < TOL[dtype]
        assert float((a[250] - b[250]).abs().max()) > 0.5 * seen


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
    want = [greedy(w, cfg, p, 12) for p in prompts]
    assert generate_batch(m, prompts, 12) == want
    same = torch.tensor(prompts[1:], device=DEV)
    assert m.generate(same, max_new_tokens=12).tolist() == want[1:]
    # replays with eager work and new prompts in between
    dec = GraphDecoder(m, 3, max_seq=80, max_new_tokens=64)
    pad = torch.zeros(3, 17, dtype=torch.int64)
    for i, p in enumerate(prompts):
        pad[i, :len(p)] = torch.tensor(p)
    for _ in range(3):
        dec.prefill(pad, lengths=[3, 17, 17])
        got = torch.cat([dec.decode(5), dec.decode(7)], dim=1).cpu()
        torch.cuda.synchronize()
        for i, p in enumerate(prompts):
            assert got[i].tolist() == want[i][len(p):]
        assert generate_batch(m, prompts[:1], 4)[0] == want[0][:7]


def test_graph_equals_eager_in_16_bits():
    from lfmq.models.graph import GraphDecoder
    m, cfg, _ = model("mixed", torch.bfloat16)
    ids = torch.tensor([util.tokens(cfg, 30, 1), util.tokens(cfg, 30, 2)],
                       device=DEV)
    # the same capacity, hence the same key ranges
    want = m.generate(ids, max_new_tokens=40,
                      cache=m.make_cache(2, max_seq=100))
    dec = GraphDecoder(m, 2, max_seq=100, max_new_tokens=64)
    for _ in range(2):
        dec.prefill(ids)
        assert torch.equal(torch.cat([ids, dec.decode(40)], 1), want)


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
    """RTN swaps the projections for packed ones (experts stay as they
    are); saved and loaded, it gives the same logits."""
    import lfmq
    from lfmq.models.qlinear import QLinear
    cfg = lfmq.models.registry.ARCHS["zatasun"].config.tiny()
    base = lfmq.build_model(cfg, seed=0).to(DEV)
    ids = torch.randint(0, cfg.vocab_size, (2, 40), generator=gen()).to(DEV)
    with torch.no_grad():
        ref = base(ids, base.make_cache(2, max_seq=64)).float()
    qc = lfmq.QuantConfig(scheme="rtn", bits=8, group_size=64)
    q = lfmq.quantize(base, qc)
    assert isinstance(q.blocks[0].mixer.in_proj, QLinear)
    with torch.no_grad():
        a = q(ids, q.make_cache(2, max_seq=64)).float()
    assert float((a - ref).norm() / ref.norm()) < 0.1
    lfmq.save(q, str(tmp_path), qc)
    q2 = lfmq.load(str(tmp_path), device=DEV)
    with torch.no_grad():
        b = q2(ids, q2.make_cache(2, max_seq=64)).float()
    assert torch.equal(a, b)
    assert q2.generate(ids, max_new_tokens=6).shape == (2, 46)
