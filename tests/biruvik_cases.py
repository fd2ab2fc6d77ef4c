"""Small configurations and random weights of the Biruvik design for its tests, in the checkpoint's layout."""
from __future__ import annotations

import torch

from tests.gisitar_cases import tokens, write_folder  # noqa: F401  (the formats are the same)


def dense(ff):
    return {"kind": "dense", "ff": ff}


def attention(heads, kv_heads, dim, vdim, diff=0.3, coef=0.4, every=16, scale=None, mlp=None):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
                      "q_temp": {"coef": coef, "every": every}, "scale": dim ** -0.5 if scale is None else scale}, "mlp": mlp}


def latent(heads, dim, vdim, kv_rank, window, scale=None, mlp=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
                      "scale": dim ** -0.5 if scale is None else scale}, "mlp": mlp}


def hgrn2(heads, dim, vdim, mlp=None):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp}


def config(layers, width=48, vocab=97, eps=1e-5, scale=3.0, cap=9.0):
    return {"architecture": "Biruvik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "logit_softcap": cap, "layers": layers}


CONFIGS = {
    # aligned widths; every pair of key maps as wide as its values once in 64 and once in 128 columns
    "plain": config([attention(6, 3, 32, 64, mlp=dense(96)), hgrn2(3, 32, 24, mlp=dense(64)), latent(4, 16, 24, 32, 24, mlp=dense(40)),
                     attention(2, 1, 64, 128, diff=0.8, every=50), latent(2, 64, 64, 128, 64), hgrn2(2, 64, 64, mlp=dense(48))]),
    # nothing a multiple of 8 or 4; an odd vocabulary
    "odd": config([hgrn2(3, 10, 13, mlp=dense(21)), attention(6, 2, 7, 30, diff=0.1, coef=0.6, every=9, scale=0.5, mlp=dense(50)),
                   latent(3, 22, 11, 19, 30, scale=0.6, mlp=dense(37)), hgrn2(5, 22, 9), latent(5, 9, 50, 37, 19),
                   attention(3, 3, 21, 13, diff=0.65, coef=0.2, every=33, mlp=dense(11))], width=53, vocab=101, eps=1e-3, scale=7.5, cap=3.5),
    # one head, one column too few or many, a window of one token, a temperature that grows with every token, factors of 1
    "edges": config([attention(1, 1, 8, 8, diff=0.0, coef=1.0, every=1, scale=1.0, mlp=dense(8)), latent(1, 16, 16, 16, 1, scale=1.0),
                     hgrn2(1, 16, 16, mlp=dense(16)), latent(2, 16, 16, 16, 1000, mlp=dense(24)), attention(2, 2, 16, 8, coef=0.0, every=7)],
                    width=16, vocab=40, scale=1.0, cap=1.0),
    # many query heads per key/value head, wide heads, wide latents
    "wide": config([attention(34, 2, 8, 24, mlp=dense(200)), hgrn2(2, 136, 72, mlp=dense(8)), latent(17, 16, 8, 264, 33),
                    attention(1, 1, 136, 200, every=100), hgrn2(1, 104, 232), latent(1, 248, 40, 520, 45, mlp=dense(300))], width=160, vocab=64),
}


def weights(cfg, seed=0, dtype=torch.float32):
    """{checkpoint name: tensor}; linear weights N(0, 1/in), norm weights around 1, gates between nearly closed and nearly open.
    Values are representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def rand(name, *shape, scale=1.0, at=0.0):
        w[name] = at + torch.randn(shape, generator=g) * scale

    def lin(name, out, inn, scale=1.0):
        rand(name, out, inn, scale=scale / inn ** 0.5)

    W, V = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(V, W, generator=g) / cfg["embedding"]["scale"]
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] is not None else ()):
            rand(p + n, scale=0.2, at=1.0)
        if l["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", 2 * H * dk), ("k", 2 * G * dk), ("v", G * dv)):
                lin(p + "mix." + n, rows, W)
                rand(f"{p}mix.{n}.b", rows, scale=0.3)
            for n in ("q.norm", "k.norm"):
                rand(p + "mix." + n, dk, scale=0.4, at=1.3)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                rand(p + "mix." + n, dk, scale=0.7 / dk ** 0.5)
        elif l["type"] == "latent_attention":
            lin(p + "mix.q", H * dk, W, 2.0)
            lin(p + "mix.dkv", m["kv_rank"], W)
            rand(p + "mix.dkv.norm", m["kv_rank"], scale=0.2, at=1.0)
            lin(p + "mix.uk", H * dk, m["kv_rank"])
            lin(p + "mix.uv", H * dv, m["kv_rank"])
            lin(p + "mix.g", H, W, 2.0)
        else:
            lin(p + "mix.q", H * dk, W)
            lin(p + "mix.f", H * dk, W)
            rand(p + "mix.f.b", H * dk, scale=2.5, at=2.0)
            w[p + "mix.lower"] = (torch.rand(H * dk, generator=g) - 0.2).clamp(min=0.0)
            lin(p + "mix.v", H * dv, W)
            rand(p + "mix.norm", dv, scale=0.2, at=1.0)
        lin(p + "mix.o", W, H * dv)
        if l["mlp"] is not None:
            lin(p + "mlp.up", l["mlp"]["ff"], W)
            lin(p + "mlp.down", W, l["mlp"]["ff"])
    rand("final.norm", scale=0.2, at=1.0)
    lin("head", V, W, 2.0)
    return {n: t.to(torch.bfloat16).to(dtype) for n, t in w.items()}
