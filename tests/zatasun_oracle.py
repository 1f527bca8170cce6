"""Plain Zatasun on the CPU, one function per mechanism, token by token where
the mechanism is a recurrence.  Double precision throughout; shares nothing
with the product.

Equations (h: a sublayer's input, p: a token's position):
  stream      x <- x + N1(mix(x)); x <- x + N2(ff(x)), N an RMS norm
  attention   out = sum_j e^{s_j} v_j / (e^{sink} + sum_j e^{s_j}), j <= p
  recurrence  S <- a S + sqrt(1 - a^2) i u, a = exp(-8 r softplus(lam))
  experts     y = sum over the chosen of E(s h), s the router's sigmoid
"""
import math

import torch

D = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


# ---- positions --------------------------------------------------------------

def frequencies(dims, base, scaling=None):
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            n, lo, hi, org = (scaling[k] for k in
                              ("factor", "low", "high", "original"))
            wave = 2 * math.pi / f
            if wave > org / lo:
                f = f / n
            elif wave >= org / hi:
                s = (org / wave - lo) / (hi - lo)
                f = (1 - s) * f / n + s * f
        out.append(f)
    return out


def rotate(x, pos, freqs):
    """x [..., dim] at position(s) pos (a number, or one per leading index):
    pairs (i, i + len(freqs)) turn by pos * freqs[i]."""
    n, f = len(freqs), torch.tensor(freqs, dtype=x.dtype)
    p = torch.as_tensor(pos, dtype=x.dtype)
    a = p.reshape(p.shape + (1,) * (x.dim() - p.dim())) * f
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a),
                      v * torch.cos(a) + u * torch.sin(a), x[..., 2 * n:]], -1)


# ---- attention -----------------------------------------------------------------

def sink_attend(scores, values, sink):
    """One query: scores [n], values [n, dv]."""
    top = torch.maximum(scores.max(), sink)
    e = torch.exp(scores - top)
    return (e @ values) / (e.sum() + torch.exp(sink - top))


def attention(q, k, v, wq, wk, sink, m, eps):
    """Projections [T, ...] of one whole sequence -> [T, heads * vdim]."""
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    f = frequencies(m["rot"]["dims"], m["rot"]["base"],
                    m["rot"].get("scaling"))
    T = q.shape[0]
    q = (rms(q, eps) * wq).view(T, H, d)
    k = (rms(k, eps) * wk).view(T, G, d)
    v = v.view(T, G, dv)
    pos = torch.arange(T)
    q, k = rotate(q, pos, f), rotate(k, pos, f)
    out = torch.empty(T, H, dv, dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * m["scale"]
        for t in range(T):
            out[t, h] = sink_attend(s[t, :t + 1], v[:t + 1, g], sink[h])
    return out.reshape(T, H * dv)


# ---- gated linear recurrence -----------------------------------------------------

def causal_conv(x, w, b, past=None):
    """x [T, C], w [C, taps] whose last column meets the current token."""
    taps = w.shape[1]
    if past is None:
        past = torch.zeros(taps - 1, x.shape[1], dtype=x.dtype)
    z = torch.cat([past, x])
    return torch.stack([sum(w[:, j] * z[t + j] for j in range(taps)) + b
                        for t in range(x.shape[0])])


def lru_gates(u, ra, ra_b, ri, ri_b, lam):
    """u [T, C] -> decay a and input sqrt(1 - a^2) i u."""
    B, n = ra.shape[0], ra.shape[1]
    r, i = [], []
    for b in range(B):
        ub = u[:, b * n:(b + 1) * n]
        r.append(sigmoid(ub @ ra[b].t() + ra_b[b]))
        i.append(sigmoid(ub @ ri[b].t() + ri_b[b]))
    log_a = -8 * torch.cat(r, 1) * softplus(lam)
    return torch.exp(log_a), \
        torch.sqrt(1 - torch.exp(2 * log_a)) * torch.cat(i, 1) * u


def lru(a, z, S=None):
    S = torch.zeros(a.shape[1], dtype=a.dtype) if S is None else S
    out = []
    for t in range(a.shape[0]):
        S = a[t] * S + z[t]
        out.append(S)
    return torch.stack(out), S


# ---- feed-forward -------------------------------------------------------------------

def dense_mlp(h, gate, up, down):
    z = h @ gate.t()
    return (z * sigmoid(z) * (h @ up.t())) @ down.t()


def expert(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.t(), max=limit)
    u = torch.clamp(h @ up.t(), min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ down.t()


def route(h, router, top):
    """One token: the chosen experts and their scores."""
    z = router @ h
    ids = sorted(range(len(z)), key=lambda e: (-float(z[e]), e))[:top]
    return ids, [sigmoid(z[e]) for e in ids]


def moe(h, w, p, mlp):
    lim = mlp["expert"]["limit"]
    out = []
    for x in h:
        y = torch.zeros_like(x)
        ids, ss = route(x, w[p + "router"], mlp["router"]["top"])
        for e, s in zip(ids, ss):
            q = f"{p}e{e}."
            y = y + expert(s * x, w[q + "gate"], w[q + "up"], w[q + "down"],
                           lim)
        if mlp.get("shared") is not None:
            q = p + "shared."
            y = y + sigmoid(w[q + "sg"][0] @ x) * expert(
                x, w[q + "gate"], w[q + "up"], w[q + "down"],
                mlp["shared"]["limit"])
        out.append(y)
    return torch.stack(out)


# ---- the model ------------------------------------------------------------------------

def parallel(h, w, p, m, eps):
    lt, rt = p + "left.", p + "right."
    left = attention(h @ w[lt + "q"].t(), h @ w[lt + "k"].t(),
                     h @ w[lt + "v"].t(), w[lt + "q.norm"], w[lt + "k.norm"],
                     w[lt + "sink"], m["left"], eps) @ w[lt + "o"].t()
    y = gelu_tanh(h @ w[rt + "y"].t() + w[rt + "y.b"])
    u = causal_conv(h @ w[rt + "x"].t() + w[rt + "x.b"], w[rt + "conv"],
                    w[rt + "conv.b"])
    a, z = lru_gates(u, w[rt + "ra"], w[rt + "ra.b"], w[rt + "ri"],
                     w[rt + "ri.b"], w[rt + "lam"])
    right = (lru(a, z)[0] * y) @ w[rt + "o"].t()
    return m["left_scale"] * left + m["right_scale"] * right


def forward(w, cfg, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence."""
    w = {k: t.to(D) for k, t in w.items()}
    eps = cfg["norm"]["eps"]
    x = rms(w["embed"][torch.tensor(tokens)], eps) * w["embed.norm"]
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = parallel(x, w, p + "mix.", e["mixer"], eps)
        x = x + rms(y, eps) * w[p + "norm1"]
        mlp = e.get("mlp")
        if mlp is not None:
            q = p + "mlp."
            y = moe(x, w, q, mlp) if mlp["kind"] == "moe" else \
                dense_mlp(x, w[q + "gate"], w[q + "up"], w[q + "down"])
            x = x + rms(y, eps) * w[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["embed"].t() \
        * cfg["logit_scale"]
