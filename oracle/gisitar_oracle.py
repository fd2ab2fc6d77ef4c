"""Plain restatement of the Gisitar decoder (test infrastructure only): one function per mechanism, loops where a
loop says it best, double precision by default, nothing shared with the product path.

A sequence is a (T, width) tensor; batches are lists of sequences.  Weights are a flat {name: tensor} dictionary in
the checkpoint's layout: every linear weight [out, in], applied as W x; layer i under ``l<i>.``.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

Tensor = torch.Tensor


def layer_norm(x: Tensor, w: Tensor, eps: float) -> Tensor:
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * w"""
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w


def rms_norm(x: Tensor, w: Tensor, eps: float) -> Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(z: Tensor) -> Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: Tensor) -> Tensor:
    return z * sigmoid(z)


def linear(x: Tensor, w: Tensor) -> Tensor:
    return x @ w.T


def softmax_attention(q: Tensor, k: Tensor, v: Tensor, scale: float) -> Tensor:
    """q (T, dim), k (T, dim), v (T, vdim) of one head; query i sees keys 0 .. i."""
    out = []
    for i in range(q.shape[0]):
        s = (k[: i + 1] @ q[i]) * scale
        e = torch.exp(s - s.max())
        out.append((e / e.sum()) @ v[: i + 1])
    return torch.stack(out)


def latent_attention(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    """Low-rank queries, keys and values expanded from one normalised latent per token, sigmoid output gate."""
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = linear(rms_norm(linear(h, p["dq"]), p["dq.norm"], eps), p["uq"])
    c = rms_norm(linear(h, p["dkv"]), p["dkv.norm"], eps)
    k, v = linear(c, p["uk"]), linear(c, p["uv"])
    heads = [softmax_attention(q[:, a * dim:(a + 1) * dim], k[:, a * dim:(a + 1) * dim],
                               v[:, a * vdim:(a + 1) * vdim], cfg["scale"]) for a in range(H)]
    return linear(torch.cat(heads, -1) * sigmoid(linear(h, p["g"])), p["o"])


def decayed_recurrence(q: Tensor, k: Tensor, v: Tensor, decay: float, state: Optional[Tensor] = None):
    """S_t = decay S_(t-1) + k_t v_t^T ; o_t = S_t^T q_t for one head -> (outputs, last state)."""
    s = torch.zeros(k.shape[1], v.shape[1], dtype=k.dtype) if state is None else state.clone()
    out = []
    for t in range(q.shape[0]):
        s = decay * s + torch.outer(k[t], v[t])
        out.append(s.T @ q[t])
    return torch.stack(out), s


def lightning(h: Tensor, p: Dict[str, Tensor], cfg: dict, eps: float) -> Tensor:
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (silu(linear(h, p[n])) for n in ("q", "k", "v"))
    heads = [decayed_recurrence(q[:, a * dim:(a + 1) * dim], k[:, a * dim:(a + 1) * dim],
                                v[:, a * vdim:(a + 1) * vdim], cfg["decay"][a])[0] for a in range(H)]
    return linear(rms_norm(torch.cat(heads, -1), p["norm"], eps) * sigmoid(linear(h, p["g"])), p["o"])


def gated_mlp(h: Tensor, p: Dict[str, Tensor]) -> Tensor:
    return linear(silu(linear(h, p["gate"])) * linear(h, p["up"]), p["down"])


MIXERS = {"latent_attention": latent_attention, "lightning": lightning}


def below(weights: Dict[str, Tensor], prefix: str) -> Dict[str, Tensor]:
    return {n[len(prefix):]: t for n, t in weights.items() if n.startswith(prefix)}


def forward(weights: Dict[str, Tensor], config: dict, tokens, layers_out: Optional[List[Tensor]] = None,
            dtype: torch.dtype = torch.float64) -> Tensor:
    """Logits (T, vocab) of one sequence.  layers_out, if given, receives the residual stream after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(config["layers"]):
        lw = below(w, f"l{i}.")
        y = MIXERS[layer["type"]](layer_norm(x, lw["norm1"], eps), below(lw, "mix."), layer["mixer"], eps)
        x = x + layer_norm(y, lw["norm1b"], eps)
        if layer["mlp"] is not None:
            y = gated_mlp(layer_norm(x, lw["norm2"], eps), below(lw, "mlp."))
            x = x + layer_norm(y, lw["norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return linear(layer_norm(x, w["final.norm"], eps), w["head"])


def greedy(weights: Dict[str, Tensor], config: dict, prompt, new_tokens: int) -> List[int]:
    ids = [int(t) for t in prompt]
    for _ in range(new_tokens):
        ids.append(int(forward(weights, config, ids)[-1].argmax()))
    return ids
