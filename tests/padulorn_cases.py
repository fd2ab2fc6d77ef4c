"""Small configurations and random weights of the Padulorn design for its tests, in the checkpoint's layout."""
from __future__ import annotations

import torch

from tests.gisitar_cases import tokens, write_folder  # noqa: F401  (the formats are the same)


def yarn(factor=4.0, original=40, fast=3.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attention(heads, kv_heads, dim, vdim, window, first=0, rot=None, base=10000.0, scaling=None, scale=None, v_mix=False, mlp=None):
    r = {"base": base, "dims": dim if rot is None else rot}
    if scaling is not None:
        r["scaling"] = scaling
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window, "keep_first": first},
                      "rot": r, "scale": dim ** -0.5 if scale is None else scale, "v_mix": v_mix},
            "mlp": mlp}


def retention(heads, dim, vdim, decay=None, rot=None, base=10000.0, mlp=None):
    return {"type": "retention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": dim if rot is None else rot},
                      "decay": [1.0 - 2.0 ** -(2 + 2 * h) for h in range(heads)] if decay is None else decay},
            "mlp": mlp}


def moe(experts, top, ff, groups=1, keep=1):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}, "expert": {"ff": ff}}


def config(layers, width=48, vocab=97, eps=1e-5, scale=3.0, mult=0.4, logit_scale=0.5):
    return {"architecture": "Padulorn", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "residual_mult": mult, "logit_scale": logit_scale, "layers": layers}


CONFIGS = {
    # aligned widths; two layers whose values mix with a first one's, one between them that does not
    "plain": config([attention(4, 2, 16, 16, 24, 5, v_mix=True, scaling=yarn(), mlp=moe(8, 2, 32, 4, 2)),
                     retention(3, 32, 24, mlp=moe(6, 3, 24, 2, 1)),
                     attention(4, 1, 32, 16, 40, 8, base=500.0, mlp=moe(12, 2, 16, 3, 2)),
                     attention(4, 2, 64, 16, 64, 70, rot=32, v_mix=True, scaling=yarn(2.5, 100, 8.0, 1.0)),
                     retention(2, 64, 64, rot=32),
                     attention(8, 2, 128, 16, 33, 1, rot=16, v_mix=True, mlp=moe(4, 1, 40, 2, 1))]),
    # nothing a multiple of 8 or 4; an odd vocabulary; partly rotated heads
    "odd": config([retention(3, 10, 13, rot=6, base=50.0, mlp=moe(9, 2, 21, 3, 2)),
                   attention(6, 2, 7, 30, 33, 3, rot=2, base=100.0, scale=0.9, v_mix=True, mlp=moe(5, 4, 11)),
                   attention(3, 1, 22, 60, 19, 7, scaling=yarn(1.7, 300, 16.0, 2.0), v_mix=True, mlp=moe(15, 3, 13, 5, 3)),
                   retention(5, 22, 9, decay=[0.6, 1.0, 0.999, 0.75, 0.9])], width=53, vocab=101, eps=1e-3, scale=7.5, mult=0.83,
                  logit_scale=1.9),
    # one head, one expert, groups of one expert, a window of one token, nothing kept, nothing rotated, all factors 1
    "edges": config([attention(1, 1, 16, 16, 1, 0, scale=1.0, mlp=moe(1, 1, 16)),
                     retention(1, 16, 16, rot=0, decay=[0.5], mlp=moe(4, 1, 8, 4, 1)),
                     attention(2, 1, 16, 16, 1, 3, rot=0, v_mix=True, mlp=moe(4, 4, 16, 2, 2)),
                     attention(2, 2, 16, 16, 1000, 2, mlp=moe(6, 2, 8, 3, 3))], width=16, vocab=40, scale=1.0, mult=1.0, logit_scale=1.0),
    # many query heads per key/value head, wide heads, many experts in few and in many groups
    "wide": config([attention(34, 2, 8, 8, 30, 9, mlp=moe(130, 3, 16, 10, 4)),
                    retention(2, 136, 72, rot=64, mlp=moe(70, 5, 24, 70, 9)),
                    attention(1, 1, 248, 40, 20, 2, scaling=yarn(8.0, 30, 2.0, 0.25), mlp=moe(300, 2, 8, 3, 1)),
                    retention(1, 40, 232), attention(3, 1, 72, 232, 45, 45, rot=70)], width=160, vocab=64),
}


def weights(cfg, seed=0, dtype=torch.float32):
    """{checkpoint name: tensor}; linear weights N(0, 1/in) (routers so large that few choices are close), norm weights around
    1.  Values are representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, out, inn, scale=1.0):
        w[name] = torch.randn(out, inn, generator=g) * scale / inn ** 0.5

    def norm(name, n):
        w[name] = 1.0 + 0.2 * torch.randn(n, generator=g)

    W, V = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(V, W, generator=g) / cfg["embedding"]["scale"]
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        H, G, dk, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
        norm(p + "norm1", W)
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            lin(p + "mix." + n, rows, W)
        if l["type"] == "attention":
            norm(p + "mix.q.norm", H * dk)
            norm(p + "mix.k.norm", G * dk)
            if m["v_mix"]:
                w[p + "mix.vmix"] = 0.2 + 0.6 * torch.rand((), generator=g)
        else:
            lin(p + "mix.g", H * dv, W)
        lin(p + "mix.o", W, H * dv)
        if l["mlp"] is not None:
            norm(p + "norm2", W)
            r, ff = l["mlp"]["router"], l["mlp"]["expert"]["ff"]
            lin(p + "mlp.router", r["experts"], W, 2.0)
            for e in range(r["experts"]):
                lin(f"{p}mlp.e{e}.up", ff, W, 2.0)
                lin(f"{p}mlp.e{e}.down", W, ff)
    norm("final.norm", W)
    lin("head", V, W)
    return {n: t.to(torch.bfloat16).to(dtype) for n, t in w.items()}
