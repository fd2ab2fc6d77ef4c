"""Plain restatement of the Rivudra decoder (test infrastructure only): one function per mechanism, loops where a loop
says it best, double precision by default, nothing shared with the product path.

A sequence is a (T, width) tensor; batches are lists of sequences.  Weights are a flat {name: tensor} dictionary in
the checkpoint's layout: every linear weight [out, in], applied as W x; layer i under ``l<i>.``.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

Tensor = torch.Tensor


def rms_norm(x: Tensor, w: Tensor, eps: float) -> Tensor:
    """The weight is stored around zero: x / rms(x) * (1 + w)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * (1.0 + w)


def sigmoid(z: Tensor) -> Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def linear(x: Tensor, w: Tensor) -> Tensor:
    return x @ w.T


def rotate(x: Tensor, base: float, dims: int, first: int = 0) -> Tensor:
    """Rotary positions on (T, dim) rows of one head at positions first, first + 1, ...: neighbours (2i, 2i + 1) among the
    first `dims` columns turn by position * base^(-2i / dims)."""
    y = x.clone()
    position = torch.arange(first, first + x.shape[0], dtype=torch.float64)
    for i in range(dims // 2):
        angle = position * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(angle).to(x.dtype), torch.sin(angle).to(x.dtype)
        u, v = x[:, 2 * i], x[:, 2 * i + 1]
        y[:, 2 * i] = u * c - v * s
        y[:, 2 * i + 1] = v * c + u * s
    return y


def window_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, window: int) -> Tensor:
    """One head: query i sees keys i - window + 1 .. i; a sink of score 0 without a value takes its share."""
    out = []
    for i in range(q.shape[0]):
        lo = max(0, i - window + 1)
        s = (k[lo: i + 1] @ q[i]) * scale
        m = torch.clamp(s.max(), min=0.0)
        e = torch.exp(s - m)
        out.append((e / (torch.exp(-m) + e.sum())) @ v[lo: i + 1])
    return torch.stack(out)


def attention(h: Tensor, p: Dict[str, Tensor], cfg: dict) -> Tensor:
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    base, dims = cfg["rot"]["base"], cfg["rot"]["dims"]
    q, k, v = linear(h, p["q"]), linear(h, p["k"]), linear(h, p["v"])
    ks = [rotate(k[:, g * dim:(g + 1) * dim], base, dims) for g in range(G)]
    heads = []
    for a in range(H):
        g = a // (H // G)
        heads.append(window_attention(rotate(q[:, a * dim:(a + 1) * dim], base, dims), ks[g],
                                      v[:, g * vdim:(g + 1) * vdim], cfg["scale"], cfg["mask"]["size"]))
    return linear(torch.cat(heads, -1) * sigmoid(linear(h, p["g"])), p["o"])


def clamped_mlp(h: Tensor, p: Dict[str, Tensor], limit: float) -> Tensor:
    g = torch.clamp(linear(h, p["gate"]), max=limit)
    u = torch.clamp(linear(h, p["up"]), min=-limit, max=limit)
    return linear(g * sigmoid(1.702 * g) * (u + 1.0), p["down"])


def route(z: Tensor, cfg: dict):
    """Router logits of ONE token -> (chosen experts, their weights)."""
    e = torch.exp(z - z.max())
    s = (e / e.sum()).tolist()
    n = len(s)
    groups = cfg["groups"]["count"]
    size = n // groups
    best = [max(s[g * size:(g + 1) * size]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-best[g], g))[: cfg["groups"]["keep"]]
    allowed = [i for i in range(n) if i // size in kept]
    chosen = sorted(allowed, key=lambda i: (-s[i], i))[: cfg["top"]]
    total = sum(s[i] for i in chosen) + 1e-20
    return chosen, [s[i] / total * cfg["scale"] for i in chosen]


def mixture(h: Tensor, p: Dict[str, Tensor], cfg: dict) -> Tensor:
    z = linear(h, p["router"])
    out = []
    for t in range(h.shape[0]):
        row = h[t:t + 1]
        y = torch.zeros_like(row)
        for i, w in zip(*route(z[t], cfg["router"])):
            y = y + w * clamped_mlp(row, below(p, f"e{i}."), cfg["expert"]["limit"])
        out.append(y)
    y = torch.cat(out)
    if cfg.get("shared") is not None:
        y = y + clamped_mlp(h, below(p, "shared."), cfg["shared"]["limit"])
    return y


def below(weights: Dict[str, Tensor], prefix: str) -> Dict[str, Tensor]:
    return {n[len(prefix):]: t for n, t in weights.items() if n.startswith(prefix)}


def layer(x: Tensor, w: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    """Both sublayers read the one norm: x + (mixer(h) + ff(h))."""
    h = rms_norm(x, w["norm1"], eps)
    y = attention(h, below(w, "mix."), cfg["mixer"])
    if cfg["mlp"] is not None:
        y = y + mixture(h, below(w, "mlp."), cfg["mlp"])
    return x + y


def forward(weights: Dict[str, Tensor], config: dict, tokens, layers_out: Optional[List[Tensor]] = None,
            dtype: torch.dtype = torch.float64) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    for i, cfg in enumerate(config["layers"]):
        x = layer(x, below(w, f"l{i}."), cfg, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return linear(rms_norm(x, w["final.norm"], eps), w["head"])


def greedy(weights: Dict[str, Tensor], config: dict, prompt, new_tokens: int) -> List[int]:
    ids = [int(t) for t in prompt]
    for _ in range(new_tokens):
        ids.append(int(forward(weights, config, ids)[-1].argmax()))
    return ids
