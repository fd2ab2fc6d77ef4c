"""Plain restatement of the Padulorn decoder (test infrastructure only): one function per mechanism, loops where a loop says
it best, double precision by default, nothing shared with the product path.

A sequence is a (T, width) tensor; batches are lists of sequences.  Weights are a flat {name: tensor} dictionary in the
checkpoint's layout: every linear weight [out, in], applied as W x; layer i under ``l<i>.``.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

Tensor = torch.Tensor


def rms_norm(x: Tensor, w: Optional[Tensor], eps: float) -> Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def sigmoid(z: Tensor) -> Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: Tensor) -> Tensor:
    return z * sigmoid(z)


def gelu(z: Tensor) -> Tensor:
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def linear(x: Tensor, w: Tensor) -> Tensor:
    return x @ w.T


def below(weights: Dict[str, Tensor], prefix: str) -> Dict[str, Tensor]:
    return {n[len(prefix):]: t for n, t in weights.items() if n.startswith(prefix)}


# ---- rotary positions -----------------------------------------------------------------------------
def frequencies(rot: dict):
    """-> (angle per position of every pair, factor on cosine and sine)."""
    base, dims, s = float(rot["base"]), rot["dims"], rot.get("scaling")
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if s is None:
        return plain, 1.0

    def where(turns):   # the (fractional) pair that turns so often within the original length
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(where(s["fast"])), 0)
    hi = min(math.ceil(where(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(x: Tensor, rot: dict, layout: str, first: int = 0) -> Tensor:
    """(T, dim) rows of one head at positions first, first + 1, ...  layout "pairs": columns 2i and 2i + 1 turn together;
    "halves": columns i and i + dims / 2."""
    y = x.clone()
    freq, factor = frequencies(rot)
    position = torch.arange(first, first + x.shape[0], dtype=torch.float64)
    half = rot["dims"] // 2
    for i in range(half):
        a, b = (2 * i, 2 * i + 1) if layout == "pairs" else (i, i + half)
        angle = position * freq[i]
        c, s = (factor * torch.cos(angle)).to(x.dtype), (factor * torch.sin(angle)).to(x.dtype)
        y[:, a] = x[:, a] * c - x[:, b] * s
        y[:, b] = x[:, b] * c + x[:, a] * s
    return y


# ---- mixers ---------------------------------------------------------------------------------------
def visible(i: int, size: int, keep_first: int) -> List[int]:
    return [j for j in range(i + 1) if i - j < size or j < keep_first]


def window_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, size: int, keep_first: int) -> Tensor:
    """One head over a whole sequence."""
    out = []
    for i in range(q.shape[0]):
        see = visible(i, size, keep_first)
        s = (k[see] @ q[i]) * scale
        e = torch.exp(s - s.max())
        out.append((e / e.sum()) @ v[see])
    return torch.stack(out)


def mix_values(v: Tensor, first: Tensor, lam: Tensor) -> Tensor:
    return (1.0 - lam) * v + lam * first


def attention(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float, v_first: Optional[Tensor] = None):
    """-> (output, the values before any mixing).  v_first: the values to mix in (None: none)."""
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = rms_norm(linear(h, p["q"]), p["q.norm"], eps)
    k = rms_norm(linear(h, p["k"]), p["k.norm"], eps)
    own = v = linear(h, p["v"])
    if v_first is not None:
        v = mix_values(own, v_first, p["vmix"])
    heads = []
    for a in range(H):
        g = a // (H // G)
        heads.append(window_attention(rotate(q[:, a * dim:(a + 1) * dim], cfg["rot"], "pairs"),
                                      rotate(k[:, g * dim:(g + 1) * dim], cfg["rot"], "pairs"),
                                      v[:, g * vdim:(g + 1) * vdim], cfg["scale"], cfg["mask"]["size"], cfg["mask"]["keep_first"]))
    return linear(torch.cat(heads, -1), p["o"]), own


def recurrence(q: Tensor, k: Tensor, v: Tensor, decay: float, state: Optional[Tensor] = None) -> Tensor:
    """One head: S <- decay S + k v^T, o = S^T q.  A given state is advanced in place."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state
    out = []
    for t in range(q.shape[0]):
        S.mul_(decay).add_(torch.outer(k[t], v[t]))
        out.append(S.T @ q[t])
    return torch.stack(out)


def retention(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = linear(h, p["q"]), linear(h, p["k"]), linear(h, p["v"])
    heads = []
    for a in range(H):
        qa = rotate(q[:, a * dim:(a + 1) * dim], cfg["rot"], "halves")
        ka = rotate(k[:, a * dim:(a + 1) * dim], cfg["rot"], "halves") * dim ** -0.5
        heads.append(rms_norm(recurrence(qa, ka, v[:, a * vdim:(a + 1) * vdim], cfg["decay"][a]), None, eps))
    return linear(torch.cat(heads, -1) * silu(linear(h, p["g"])), p["o"])


# ---- feed-forward ---------------------------------------------------------------------------------
def route(z: Tensor, cfg: dict):
    """Router logits of ONE token -> (chosen experts, their weights)."""
    s = sigmoid(z).tolist()
    n, groups = len(s), cfg["groups"]["count"]
    size = n // groups
    score = [sum(sorted(s[g * size:(g + 1) * size], reverse=True)[:2]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-score[g], g))[: cfg["groups"]["keep"]]
    allowed = [i for i in range(n) if i // size in kept]
    chosen = sorted(allowed, key=lambda i: (-s[i], i))[: cfg["top"]]
    return chosen, [s[i] for i in chosen]


def expert(h: Tensor, p: Dict[str, Tensor]) -> Tensor:
    return linear(gelu(linear(h, p["up"])), p["down"])


def mixture(h: Tensor, p: Dict[str, Tensor], cfg: dict) -> Tensor:
    z = linear(h, p["router"])
    picks = [route(z[t], cfg["router"]) for t in range(h.shape[0])]
    y = torch.zeros_like(h)
    for e in range(cfg["router"]["experts"]):
        rows = [t for t, (chosen, _) in enumerate(picks) if e in chosen]
        if rows:
            w = torch.tensor([picks[t][1][picks[t][0].index(e)] for t in rows], dtype=h.dtype)
            y[rows] += w[:, None] * expert(h[rows], below(p, f"e{e}."))
    return y


# ---- the model ------------------------------------------------------------------------------------
def forward(weights: Dict[str, Tensor], config: dict, tokens, layers_out: Optional[List[Tensor]] = None,
            dtype: torch.dtype = torch.float64) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps, m = config["norm"]["eps"], config["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    v_first = None
    for i, cfg in enumerate(config["layers"]):
        p = below(w, f"l{i}.")
        if cfg["type"] == "attention":
            mixes = bool(cfg["mixer"].get("v_mix"))
            y, own = attention(x, below(p, "mix."), cfg["mixer"], eps, v_first if mixes else None)
            if mixes and v_first is None:
                v_first = own
        else:
            y = retention(x, below(p, "mix."), cfg["mixer"], eps)
        x = x + m * rms_norm(y, p["norm1"], eps)
        if cfg["mlp"] is not None:
            x = x + m * rms_norm(mixture(x, below(p, "mlp."), cfg["mlp"]), p["norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return linear(rms_norm(x, w["final.norm"], eps), w["head"]) * config["logit_scale"]


def greedy(weights: Dict[str, Tensor], config: dict, prompt, new_tokens: int) -> List[int]:
    ids = [int(t) for t in prompt]
    for _ in range(new_tokens):
        ids.append(int(forward(weights, config, ids)[-1].argmax()))
    return ids
