"""Small Rapivik models for the tests: configurations of many shapes,
random weights under the checkpoint's names, and the oracle's answers."""
import json
import os

import torch
from safetensors.torch import save_file

import rapivik_oracle as oracle


def mlstm(heads=2, dim=24, vdim=40, cap=9.0, ff=None, **kw):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim,
                                       "vdim": vdim, "gate_cap": cap},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}, **kw}


def latent(heads=3, dim=24, rot=8, vdim=40, q_rank=56, kv_rank=48, window=12,
           base=5000.0, scale=None, ff=72, **kw):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot,
                      "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "mask": {"size": window},
                      "rot": {"base": base, "dims": rot},
                      "scale": scale or 1.3 * (dim + rot) ** -0.5},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}, **kw}


def config(layers, vocab=97, width=64, buckets=89, eps=1e-5, mul_prev=31,
           mul_cur=5):
    return {"architecture": "Rapivik", "vocab": vocab, "width": width,
            "layers": layers, "norm": {"eps": eps},
            "embedding": {"bigram": {"buckets": buckets,
                                     "mul_prev": mul_prev,
                                     "mul_cur": mul_cur}}}


# aligned sizes (matrix-core kernels), odd ones (general kernels), orders,
# shared weights, missing and extra feed-forwards, windows of 1 and beyond
# every prompt
CONFIGS = {
    "mixed": config([mlstm(), latent(), mlstm(ff=48), latent(window=5),
                     mlstm(weights_of=0), latent(weights_of=1)]),
    "attention_first": config(
        [latent(heads=5, dim=16, rot=16, vdim=24, kv_rank=40, window=33,
                ff=None), latent(window=1, base=100.0),
         mlstm(heads=1, dim=64, vdim=32, cap=3.0)], width=96, vocab=130),
    "odd": config([mlstm(heads=3, dim=11, vdim=21, ff=35),
                   latent(heads=3, dim=13, rot=6, vdim=11, q_rank=27,
                          kv_rank=19, window=9, ff=33),
                   mlstm(heads=2, dim=5, vdim=7)], width=51, vocab=101,
                  buckets=7),
    "wide_window": config([latent(heads=17, dim=8, rot=8, vdim=8, q_rank=16,
                                  kv_rank=16, window=5000),
                           mlstm(heads=4, dim=40, vdim=136)], width=80),
    "recurrent_only": config([mlstm(heads=2, dim=32, vdim=64, ff=64),
                              mlstm(weights_of=0, heads=2, dim=32, vdim=64,
                                    ff=64)], width=64),
}


def weights(cfg, seed=0):
    """Random bf16 tensors under the checkpoint's names, scaled so that
    scores, gates and sinks all matter."""
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, n, mean=0.0, std=0.2):
        w[name] = mean + std * torch.randn(n, generator=g)

    mat("embed", cfg["vocab"], width, width ** 0.5)
    mat("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, width,
        width ** 0.5)
    for i, e in enumerate(cfg["layers"]):
        if e.get("weights_of") is not None:
            continue
        m, p = e["mixer"], f"l{i}."
        H, dv = m["heads"], m["vdim"]
        vec(p + "norm1", width)
        if e["type"] == "mlstm":
            for n, k in (("q", m["dim"]), ("k", m["dim"]), ("v", dv),
                         ("g", dv)):
                mat(p + "mix." + n, H * k, width, 1.5)
            vec(p + "mix.norm", H * dv, 1.0)
            mat(p + "mix.i", H, width, 2.0)
            vec(p + "mix.i.b", H, -0.5, 1.0)
            mat(p + "mix.f", H, width, 1.0)
            vec(p + "mix.f.b", H, 3.5, 1.0)
        else:
            mat(p + "mix.dq", m["q_rank"], width)
            vec(p + "mix.dq.norm", m["q_rank"], 1.0)
            mat(p + "mix.uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], 2.0)
            mat(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], width, 1.5)
            vec(p + "mix.dkv.norm", m["kv_rank"], 1.0)
            mat(p + "mix.uk", H * m["dim"], m["kv_rank"], 1.5)
            mat(p + "mix.uv", H * dv, m["kv_rank"])
            vec(p + "mix.sink", H, 0.5, 1.0)
            mat(p + "mix.g", H * dv, width)
        mat(p + "mix.o", width, H * dv)
        if e["mlp"] is not None:
            vec(p + "norm2", width)
            mat(p + "mlp.gate", e["mlp"]["ff"], width, 1.5)
            mat(p + "mlp.up", e["mlp"]["ff"], width)
            mat(p + "mlp.down", width, e["mlp"]["ff"])
    vec("final.norm", width)
    mat("head", cfg["vocab"], width)
    return {k: v.bfloat16() for k, v in w.items()}


def write_checkpoint(path, cfg, w):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(path, "model.safetensors"))
    return str(path)


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def expected(w, cfg, toks):
    return oracle.forward(w, cfg, toks)


def rel(got, want):
    """Error of the logits relative to their size.  32-bit results: the
    worst row.  16-bit ones: over all rows — a head whose output nearly
    cancels is normed back to full size, rounding included, so that single
    rows of a random model may be several times worse than the rest."""
    got16 = got.dtype == torch.bfloat16
    got, want = got.double().cpu(), want.double().cpu()
    e = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    if got16:
        assert float(e.max()) < 0.4, float(e.max())
        return float(e.pow(2).mean().sqrt())
    return float(e.max())
