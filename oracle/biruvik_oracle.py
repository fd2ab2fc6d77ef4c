"""Plain restatement of the Biruvik decoder (test infrastructure only): one function per mechanism, loops where a loop says
it best, double precision by default, nothing shared with the product path.

A sequence is a (T, width) tensor; batches are lists of sequences.  Weights are a flat {name: tensor} dictionary in the
checkpoint's layout: every linear weight [out, in], applied as W x; layer i under ``l<i>.``.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

Tensor = torch.Tensor


def rms(x: Tensor, eps: float) -> Tensor:
    """Every row over its root mean square."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z: Tensor) -> Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: Tensor) -> Tensor:
    return z * sigmoid(z)


def linear(x: Tensor, w: Tensor, b: Optional[Tensor] = None) -> Tensor:
    y = x @ w.T
    return y if b is None else y + b


def below(weights: Dict[str, Tensor], prefix: str) -> Dict[str, Tensor]:
    return {n[len(prefix):]: t for n, t in weights.items() if n.startswith(prefix)}


# ---- differential attention -----------------------------------------------------------------------
def temperature(position: int, coef: float, every: int) -> float:
    """Factor on the query of a position: grows with the logarithm of how many spans of `every` tokens lie behind it."""
    return 1.0 + coef * math.log(math.floor((position + 1) / every) + 1)


def softmax_attention(q: Tensor, k: Tensor, v: Tensor, scale: float, size: Optional[int] = None) -> Tensor:
    """One head over a whole sequence: query i sees keys up to its own, with `size` only the last `size` of them."""
    out = []
    for i in range(q.shape[0]):
        lo = 0 if size is None else max(0, i - size + 1)
        s = (k[lo:i + 1] @ q[i]) * scale
        e = torch.exp(s - s.max())
        out.append((e / e.sum()) @ v[lo:i + 1])
    return torch.stack(out)


def difference_weight(p: Dict[str, Tensor], diff: float) -> Tensor:
    """Weight of the second map, one number."""
    return torch.exp((p["lq1"] * p["lk1"]).sum()) - torch.exp((p["lq2"] * p["lk2"]).sum()) + diff


def differential_head(a1: Tensor, a2: Tensor, lam: Tensor, diff: float, eps: float) -> Tensor:
    return rms(a1 - lam * a2, eps) * (1.0 - diff)


def attention(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    H, G, dim, vdim, T = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"], h.shape[0]
    q = (rms(linear(h, p["q"], p["q.b"]).view(T, H, 2, dim), eps) * p["q.norm"])
    k = (rms(linear(h, p["k"], p["k.b"]).view(T, G, 2, dim), eps) * p["k.norm"])
    v = linear(h, p["v"], p["v.b"]).view(T, G, vdim)
    temp = torch.tensor([temperature(i, cfg["q_temp"]["coef"], cfg["q_temp"]["every"]) for i in range(T)], dtype=h.dtype)
    q = q * temp[:, None, None, None]
    lam = difference_weight(p, cfg["diff"])
    heads = []
    for a in range(H):
        g = a // (H // G)
        a1, a2 = (softmax_attention(q[:, a, m], k[:, g, m], v[:, g], cfg["scale"]) for m in (0, 1))
        heads.append(differential_head(a1, a2, lam, cfg["diff"], eps))
    return linear(torch.cat(heads, -1), p["o"])


# ---- latent attention -----------------------------------------------------------------------------
def latent_attention(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = linear(h, p["q"])
    c = rms(linear(h, p["dkv"]), eps) * p["dkv.norm"]
    k, v = linear(c, p["uk"]), linear(c, p["uv"])
    gate = sigmoid(linear(h, p["g"]))
    heads = []
    for a in range(H):
        o = softmax_attention(q[:, a * dim:(a + 1) * dim], k[:, a * dim:(a + 1) * dim], v[:, a * vdim:(a + 1) * vdim], cfg["scale"],
                              cfg["mask"]["size"])
        heads.append(o * gate[:, a:a + 1])
    return linear(torch.cat(heads, -1), p["o"])


# ---- gated linear attention (HGRN2) ---------------------------------------------------------------
def forget(z: Tensor, lower: Tensor) -> Tensor:
    return lower + (1.0 - lower) * sigmoid(z)


def recurrence(q: Tensor, f: Tensor, v: Tensor, state: Optional[Tensor] = None) -> Tensor:
    """One head: row d of S decays by f_d and takes (1 - f_d) v; o = S^T q.  A given state is advanced in place."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype) if state is None else state
    out = []
    for t in range(q.shape[0]):
        S.mul_(f[t][:, None]).add_(torch.outer(1.0 - f[t], v[t]))
        out.append(S.T @ q[t])
    return torch.stack(out)


def hgrn2(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q, v = silu(linear(h, p["q"])), linear(h, p["v"])
    f = forget(linear(h, p["f"], p["f.b"]), p["lower"])
    heads = []
    for a in range(H):
        d, e = slice(a * dim, (a + 1) * dim), slice(a * vdim, (a + 1) * vdim)
        heads.append(rms(recurrence(q[:, d], f[:, d], v[:, e]), eps) * p["norm"])
    return linear(torch.cat(heads, -1), p["o"])


MIXERS = {"attention": attention, "latent_attention": latent_attention, "hgrn2": hgrn2}


# ---- feed-forward, output -------------------------------------------------------------------------
def mlp(h: Tensor, p: Dict[str, Tensor]) -> Tensor:
    return linear(torch.clamp(linear(h, p["up"]), min=0.0) ** 2, p["down"])


def softcap(x: Tensor, cap: float) -> Tensor:
    return cap * torch.tanh(x / cap)


# ---- the model ------------------------------------------------------------------------------------
def forward(weights: Dict[str, Tensor], config: dict, tokens, layers_out: Optional[List[Tensor]] = None,
            dtype: torch.dtype = torch.float64) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    for i, cfg in enumerate(config["layers"]):
        p = below(w, f"l{i}.")
        x = x + rms(MIXERS[cfg["type"]](rms(x, eps) * p["norm1"], below(p, "mix."), cfg["mixer"], eps), eps) * p["norm1b"]
        if cfg["mlp"] is not None:
            x = x + rms(mlp(rms(x, eps) * p["norm2"], below(p, "mlp.")), eps) * p["norm2b"]
        if layers_out is not None:
            layers_out.append(x.clone())
    return softcap(linear(rms(x, eps) * w["final.norm"], w["head"]), config["logit_softcap"])


def greedy(weights: Dict[str, Tensor], config: dict, prompt, new_tokens: int) -> List[int]:
    ids = [int(t) for t in prompt]
    for _ in range(new_tokens):
        ids.append(int(forward(weights, config, ids)[-1].argmax()))
    return ids
