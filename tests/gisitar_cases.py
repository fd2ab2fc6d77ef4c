"""Small configurations and random weights of the Gisitar design for its tests, in the checkpoint's layout."""
from __future__ import annotations

import json
import os
import struct

import torch


def latent(heads, dim, vdim, q_rank, kv_rank, scale=None, ff=48):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": dim ** -0.5 if scale is None else scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def lightning(heads, dim, vdim, decay, ff=48):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, width=48, vocab=97, eps=1e-5):
    return {"architecture": "Gisitar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # aligned widths, the two kinds alternating, lightning first
    "alternating": config([lightning(3, 16, 24, (0.9, 0.5, 0.99)), latent(3, 32, 16, 24, 40), lightning(1, 32, 32, (0.7,)),
                           latent(5, 16, 48, 56, 32)]),
    # nothing a multiple of 8 or 4; an odd vocabulary; layers without a feed-forward
    "odd": config([latent(3, 10, 13, 21, 27, ff=51), lightning(2, 11, 9, (0.97, 0.3), ff=None), latent(1, 7, 30, 9, 19, ff=None),
                   lightning(3, 5, 21, (0.2, 0.999, 0.8), ff=35)], width=53, vocab=101, eps=1e-3),
    # one head, equal widths, decays of exactly 0 and 1, a scale that is not dim^-1/2
    "edges": config([latent(1, 16, 16, 16, 16, scale=1.0, ff=16), lightning(2, 16, 16, (1.0, 0.0), ff=16)], width=16, vocab=40),
    # wide heads and latents: other tile sizes
    "wide": config([latent(2, 136, 72, 96, 136), lightning(1, 136, 72, (0.95,)), lightning(2, 72, 136, (0.6, 0.98)),
                    latent(17, 8, 8, 16, 264)], width=160, vocab=64),
}


def weights(cfg, seed=0, dtype=torch.float32):
    """{checkpoint name: tensor}; linear weights N(0, 1/in), norm weights around 1.  Values are representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, out, inn):
        w[name] = torch.randn(out, inn, generator=g) / inn ** 0.5

    def norm(name, n):
        w[name] = 1.0 + 0.2 * torch.randn(n, generator=g)

    W, V = cfg["width"], cfg["vocab"]
    w["embed"] = torch.randn(V, W, generator=g)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        for n in ("norm1", "norm1b"):
            norm(p + n, W)
        if l["type"] == "latent_attention":
            lin(p + "mix.dq", m["q_rank"], W)
            norm(p + "mix.dq.norm", m["q_rank"])
            lin(p + "mix.uq", H * dk, m["q_rank"])
            lin(p + "mix.dkv", m["kv_rank"], W)
            norm(p + "mix.dkv.norm", m["kv_rank"])
            lin(p + "mix.uk", H * dk, m["kv_rank"])
            lin(p + "mix.uv", H * dv, m["kv_rank"])
        else:
            lin(p + "mix.q", H * dk, W)
            lin(p + "mix.k", H * dk, W)
            lin(p + "mix.v", H * dv, W)
            norm(p + "mix.norm", H * dv)
        lin(p + "mix.g", H * dv, W)
        lin(p + "mix.o", W, H * dv)
        if l["mlp"] is not None:
            for n in ("norm2", "norm2b"):
                norm(p + n, W)
            ff = l["mlp"]["ff"]
            lin(p + "mlp.gate", ff, W)
            lin(p + "mlp.up", ff, W)
            lin(p + "mlp.down", W, ff)
    norm("final.norm", W)
    lin("head", V, W)
    return {n: t.to(torch.bfloat16).to(dtype) for n, t in w.items()}


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def write_folder(folder, cfg, w):
    """config.json and model.safetensors (bf16) in `folder`."""
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blob = {}, b""
    for n, t in w.items():
        raw = t.to(torch.bfloat16).reshape(-1).view(torch.uint8).numpy().tobytes()
        header[n] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + blob)
