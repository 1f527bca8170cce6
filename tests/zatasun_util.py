"""Small Zatasun models for the tests: configurations of many shapes, random
weights under the checkpoint's names, and the oracle's answers."""
import torch

import zatasun_oracle as oracle
from rapivik_util import rel, tokens, write_checkpoint  # noqa: F401

SCALING = {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 64}


def layer(heads=6, kv=2, dim=24, vdim=40, rot=16, base=900.0, scaling=SCALING,
          scale=None, rec=64, blocks=4, taps=4, gains=(0.7, 1.3), mlp=None):
    r = {"base": base, "dims": rot}
    if scaling is not None:
        r["scaling"] = dict(scaling)
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                 "rot": r, "scale": scale or 1.4 * dim ** -0.5},
        "right": {"width": rec, "blocks": blocks, "conv": taps},
        "left_scale": gains[0], "right_scale": gains[1]}}


def dense(ff=48):
    return {"kind": "dense", "ff": ff}


def moe(experts=7, top=2, ff=40, limit=0.8, shared=(56, 1.1)):
    m = {"kind": "moe", "router": {"experts": experts, "top": top},
         "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        m["shared"] = {"ff": shared[0], "limit": shared[1]}
    return m


def config(layers, vocab=97, width=64, eps=1e-5, logit_scale=0.35):
    return {"architecture": "Zatasun", "vocab": vocab, "width": width,
            "layers": layers, "norm": {"eps": eps},
            "logit_scale": logit_scale}


# aligned sizes (matrix-core kernels), odd ones (general kernels), every
# order of feed-forwards, one and many of heads, blocks, taps and experts
CONFIGS = {
    "mixed": config([layer(mlp=dense()), layer(mlp=moe()),
                     layer(kv=6, gains=(1.0, 0.6)),
                     layer(kv=1, blocks=1, taps=2,
                           mlp=moe(top=1, shared=None))]),
    "experts_first": config(
        [layer(heads=5, kv=5, dim=16, vdim=24, rot=8, scaling=None, rec=96,
               blocks=2, taps=1, mlp=moe(experts=3, top=3)),
         layer(heads=18, kv=2, dim=40, vdim=72, rot=40, rec=80, blocks=2,
               taps=5, mlp=dense(72))], width=96, vocab=130,
        logit_scale=1.0),
    "odd": config([layer(heads=3, kv=3, dim=13, vdim=11, rot=6, rec=35,
                         blocks=5, taps=3, mlp=moe(ff=21, shared=(19, 0.5))),
                   layer(heads=4, kv=2, dim=7, vdim=21, rot=2, rec=33,
                         blocks=1, mlp=dense(33))], width=51, vocab=101,
                  logit_scale=2.0),
    "bare": config([layer(heads=1, kv=1, dim=8, vdim=8, rot=8, rec=16,
                          blocks=2)], width=16, vocab=40),
}


def weights(cfg, seed=0):
    """Random bf16 tensors under the checkpoint's names, scaled so that
    scores, gates, sinks and clamps all matter.

    Rounding must not choose experts: routers read the first CODE
    dimensions only, no sublayer writes there, and every token's code keeps
    the last chosen expert well ahead of the first one left out."""
    g = torch.Generator().manual_seed(seed)
    w, width = {}, cfg["width"]

    def mat(name, out, inp, gain=1.0):
        w[name] = torch.randn(out, inp, generator=g) * gain * inp ** -0.5

    def vec(name, *shape, mean=0.0, std=0.2):
        w[name] = mean + std * torch.randn(*shape, generator=g)

    def glu(p, ff):
        mat(p + "gate", ff, width, 1.5)
        mat(p + "up", ff, width)
        mat(p + "down", width, ff)

    mat("embed", cfg["vocab"], width, width ** 0.5)
    vec("embed.norm", width, mean=1.0)
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        a, r = e["mixer"]["left"], e["mixer"]["right"]
        H, G, n = a["heads"], a["kv_heads"], r["width"] // r["blocks"]
        q, C = p + "mix.left.", r["width"]
        vec(p + "norm1", width, mean=1.0)
        for name, rows in (("q", H * a["dim"]), ("k", G * a["dim"]),
                           ("v", G * a["vdim"])):
            mat(q + name, rows, width)
        vec(q + "q.norm", H * a["dim"], mean=1.3)
        vec(q + "k.norm", G * a["dim"], mean=1.3)
        vec(q + "sink", H, mean=0.5, std=1.0)
        mat(q + "o", width, H * a["vdim"])
        q = p + "mix.right."
        for name in "yx":
            mat(q + name, C, width)
            vec(f"{q}{name}.b", C)
        vec(q + "conv", C, r["conv"], std=r["conv"] ** -0.5)
        vec(q + "conv.b", C)
        for name in ("ra", "ri"):
            vec(q + name, r["blocks"], n, n, std=n ** -0.5)
            vec(f"{q}{name}.b", r["blocks"], n, std=0.5)
        vec(q + "lam", C, mean=-3.0, std=1.5)
        mat(q + "o", width, C)
        m = e.get("mlp")
        if m is None:
            continue
        p += "mlp."
        vec(f"l{i}.norm2", width, mean=1.0)
        if m["kind"] == "dense":
            glu(p, m["ff"])
            continue
        mat(p + "router", m["router"]["experts"], width,
            3.0 * (width / CODE) ** 0.5)
        w[p + "router"][:, CODE:] = 0
        for x in range(m["router"]["experts"]):
            glu(f"{p}e{x}.", m["expert"]["ff"])
        if m.get("shared") is not None:
            glu(p + "shared.", m["shared"]["ff"])
            mat(p + "shared.sg", 1, width)
    vec("final.norm", width, mean=1.0)
    w = {k: v.bfloat16() for k, v in w.items()}
    routers = [(w[f"l{i}.mlp.router"].double(), e["mlp"]["router"]["top"])
               for i, e in enumerate(cfg["layers"])
               if (e.get("mlp") or {}).get("kind") == "moe"]
    routers = [(r, k) for r, k in routers if k < len(r)]
    for k in w if routers else ():
        if k.endswith(("norm1", "norm2")):
            w[k][:CODE] = 0
    for t in range(cfg["vocab"]):
        while not all(clear(w, cfg, t, r, k) for r, k in routers):
            w["embed"][t] = torch.randn(width, generator=g).bfloat16()
    return w


CODE = 16


def clear(w, cfg, t, router, top):
    x = oracle.rms(w["embed"][t].double(), cfg["norm"]["eps"]) \
        * w["embed.norm"].double()
    z = (router @ x).sort(descending=True)[0]
    return float(z[top - 1] - z[top]) > 0.15


def expected(w, cfg, toks):
    return oracle.forward(w, cfg, toks)
