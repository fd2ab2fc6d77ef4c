"""Small configurations and random weights of the Rivudra design for its tests, in the checkpoint's layout."""
from __future__ import annotations

import torch

from tests.gisitar_cases import tokens, write_folder  # noqa: F401  (the formats are the same)


def layer(heads, kv_heads, dim, vdim, window, rot=None, base=10000.0, scale=None, mlp=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                      "rot": {"base": base, "dims": dim if rot is None else rot}, "scale": dim ** -0.5 if scale is None else scale},
            "mlp": mlp}


def moe(experts, top, ff, limit=2.0, groups=1, keep=1, scale=1.0, shared=None, shared_limit=2.0):
    m = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}},
         "expert": {"ff": ff, "limit": limit}}
    if shared is not None:
        m["shared"] = {"ff": shared, "limit": shared_limit}
    return m


def config(layers, width=48, vocab=97, eps=1e-5, scale=3.0):
    return {"architecture": "Rivudra", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": layers}


CONFIGS = {
    # aligned widths; windows of several sizes; the first layer without a feed-forward
    "plain": config([layer(4, 2, 16, 16, 24),
                     layer(6, 3, 32, 24, 40, base=5000.0, mlp=moe(8, 2, 32, 1.0, 4, 2, 1.5, shared=40, shared_limit=0.5)),
                     layer(2, 2, 64, 64, 64, rot=32, mlp=moe(6, 3, 24, 1.5, 2, 1, 2.5, shared=24))]),
    # nothing a multiple of 8 or 4; an odd vocabulary; partly rotated heads
    "odd": config([layer(3, 1, 10, 13, 19, rot=6, mlp=moe(9, 2, 21, 0.8, 3, 2, 0.7, shared=13, shared_limit=3.0)),
                   layer(6, 2, 7, 30, 33, rot=2, base=100.0, scale=0.9, mlp=moe(5, 4, 11, shared=27)),
                   layer(5, 5, 22, 9, 101, rot=22, mlp=None)], width=53, vocab=101, eps=1e-3, scale=7.5),
    # one head, one expert, one group of each expert, a window of one token, nothing rotated, no shared expert
    "edges": config([layer(1, 1, 16, 16, 1, scale=1.0, mlp=moe(1, 1, 16)),
                     layer(2, 1, 16, 16, 2, rot=0, mlp=moe(4, 1, 8, 1.0, 4, 1, 3.0)),
                     layer(2, 2, 16, 16, 1000, mlp=moe(4, 4, 16, 1.0, 2, 2, shared=8))], width=16, vocab=40, scale=1.0),
    # many query heads per key/value head, wide heads, many experts in few and in many groups
    "wide": config([layer(34, 2, 8, 8, 30, mlp=moe(130, 3, 16, groups=10, keep=4)),
                    layer(2, 1, 136, 72, 50, rot=64, mlp=moe(70, 5, 24, groups=70, keep=9, shared=16)),
                    layer(1, 1, 248, 40, 20, mlp=moe(300, 2, 8, groups=3, keep=1)),
                    layer(3, 1, 72, 232, 45, mlp=None)], width=160, vocab=64),
}


def weights(cfg, seed=0, dtype=torch.float32):
    """{checkpoint name: tensor}; linear weights N(0, 1/in) (routers three times as large: few close calls), norm weights
    around 0.  Values are representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, out, inn, scale=1.0):
        w[name] = torch.randn(out, inn, generator=g) * scale / inn ** 0.5

    def norm(name, n):
        w[name] = 0.2 * torch.randn(n, generator=g)

    def mlp(name, ff):
        lin(name + ".gate", ff, W)
        lin(name + ".up", ff, W)
        lin(name + ".down", W, ff)

    W, V = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(V, W, generator=g) / cfg["embedding"]["scale"]
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        norm(p + "norm1", W)
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv), ("g", H * dv)):
            lin(p + "mix." + n, rows, W)
        lin(p + "mix.o", W, H * dv)
        if l["mlp"] is not None:
            r = l["mlp"]["router"]
            lin(p + "mlp.router", r["experts"], W, 3.0)
            for e in range(r["experts"]):
                mlp(f"{p}mlp.e{e}", l["mlp"]["expert"]["ff"])
            if "shared" in l["mlp"]:
                mlp(p + "mlp.shared", l["mlp"]["shared"]["ff"])
    norm("final.norm", W)
    lin("head", V, W)
    return {n: t.to(torch.bfloat16).to(dtype) for n, t in w.items()}
