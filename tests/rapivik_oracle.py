"""Plain, slow Rapivik: the tests' oracle.

One function per mechanism, written token by token from the equations in
double precision.  Shares no code with the lfmq package; tensors come as
a flat dict with the checkpoint's names, the configuration as the parsed
config.json.
"""
import math

import torch

D = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """RMS norm whose weight is stored as an offset from one."""
    return rms(x, eps) * (1 + w)


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def log_sigmoid(x):
    return -(torch.clamp(-x, min=0) + torch.log1p(torch.exp(-x.abs())))


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def bigram_rows(tokens, buckets, mul_prev, mul_cur, prev=None):
    """Hash-table row of every token; the row after the buckets has no
    previous token."""
    rows = []
    for t in tokens:
        rows.append(buckets if prev is None
                    else (prev * mul_prev + t * mul_cur) % buckets)
        prev = t
    return rows


def embed(w, cfg, tokens):
    b = cfg["embedding"]["bigram"]
    rows = bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])
    return w["embed"][tokens] + w["bigram"][rows]


def rotate(x, pos, base, dims):
    """x [..., n]; the first `dims` entries turn, halves paired."""
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=D) / dims)
    c, s = torch.cos(pos * f), torch.sin(pos * f)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def mlstm_cell(q, k, v, i, f, state):
    """One token, one head.  q, k [dim], v [vdim], log gates i, f;
    state (S [dim, vdim], n [dim], m).  Returns (o [vdim], state)."""
    S, n, m = state
    m2 = max(f + m, i)
    a, b = math.exp(f + m - m2), math.exp(i - m2)
    S = a * S + b * torch.outer(k, v)
    n = a * n + b * k
    den = max(abs(float(n @ q)), math.exp(-m2)) + 1e-6
    return (S.t() @ q) / den, (S, n, m2)


def mlstm_gates(w, p, c, h):
    i = soft_cap(h @ w[p + "i"].t() + w[p + "i.b"], c["gate_cap"])
    f = log_sigmoid(soft_cap(h @ w[p + "f"].t() + w[p + "f.b"],
                             c["gate_cap"]))
    return i, f


def mlstm(w, p, c, h, eps):
    """h [T, width] -> [T, width]; p is the tensor prefix."""
    T, H, dk, dv = h.shape[0], c["heads"], c["dim"], c["vdim"]
    q = (h @ w[p + "q"].t()).view(T, H, dk) * dk ** -0.5
    k = (h @ w[p + "k"].t()).view(T, H, dk)
    v = (h @ w[p + "v"].t()).view(T, H, dv)
    i, f = mlstm_gates(w, p, c, h)
    o = torch.zeros(T, H, dv, dtype=D)
    for hd in range(H):
        st = (torch.zeros(dk, dv, dtype=D), torch.zeros(dk, dtype=D), 0.0)
        for t in range(T):
            o[t, hd], st = mlstm_cell(q[t, hd], k[t, hd], v[t, hd],
                                      float(i[t, hd]), float(f[t, hd]), st)
    o = rms(o, eps).reshape(T, H * dv) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].t())) @ w[p + "o"].t()


def sink_attend(scores, values, sink):
    """scores [n] and values [n, v] of the visible keys; the sink joins
    the denominator only."""
    m = max(float(scores.max()), float(sink))
    e = torch.exp(scores - m)
    return (e @ values) / (e.sum() + math.exp(float(sink) - m))


def latent_attention(w, p, c, h, eps):
    T, H, dn, dr = h.shape[0], c["heads"], c["dim"], c["rot_dim"]
    dv, R, rot = c["vdim"], c["kv_rank"], c["rot"]
    cq = rms(h @ w[p + "dq"].t(), eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].t()).view(T, H, dn + dr)
    lat = h @ w[p + "dkv"].t()
    ckv = rms(lat[:, :R], eps) * w[p + "dkv.norm"]
    kr = torch.stack([rotate(lat[t, R:], t, rot["base"], rot["dims"])
                      for t in range(T)])
    kn = (ckv @ w[p + "uk"].t()).view(T, H, dn)
    v = (ckv @ w[p + "uv"].t()).view(T, H, dv)
    o = torch.zeros(T, H, dv, dtype=D)
    for t in range(T):
        lo = max(0, t - c["mask"]["size"] + 1)
        for hd in range(H):
            qr = rotate(q[t, hd, dn:], t, rot["base"], rot["dims"])
            s = (kn[lo:t + 1, hd] @ q[t, hd, :dn]
                 + kr[lo:t + 1] @ qr) * c["scale"]
            o[t, hd] = sink_attend(s, v[lo:t + 1, hd], w[p + "sink"][hd])
    return (o.reshape(T, H * dv) * sigmoid(h @ w[p + "g"].t())) \
        @ w[p + "o"].t()


def dense_ff(w, p, h):
    g = h @ w[p + "gate"].t()
    return (g * sigmoid(g) * (h @ w[p + "up"].t())) @ w[p + "down"].t()


def forward(w, cfg, tokens, layers_out=None):
    """tokens: list of ints -> logits [T, vocab] in double precision."""
    w = {k: v.to(D) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = embed(w, cfg, tokens)
    for i, e in enumerate(cfg["layers"]):
        p = f"l{e.get('weights_of', i)}."
        mix = {"mlstm": mlstm, "latent_attention": latent_attention}[e["type"]]
        x = x + mix(w, p + "mix.", e["mixer"],
                    centred_norm(x, w[p + "norm1"], eps), eps)
        if e["mlp"] is not None:
            x = x + dense_ff(w, p + "mlp.",
                             centred_norm(x, w[p + "norm2"], eps))
        if layers_out is not None:
            layers_out.append(x)
    return centred_norm(x, w["final.norm"], eps) @ w["head"].t()
