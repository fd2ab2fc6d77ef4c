"""Biruvik: a small decoder-only language model that mixes gated linear attention (HGRN2), differential attention without positions
and windowed latent attention, with norms of one number on both sides of every sublayer, plain squared-ReLU feed-forwards and capped
logits.  Sizes, constants and the order of layers come from its configuration; the machinery is models/hybrid.py."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

import torch.nn as nn

from ..layers.differential_attention import DifferentialAttention
from ..layers.ffn import PlainFeedForward
from ..layers.gated_linear_attention import GatedLinearAttention
from ..layers.latent_attention import LatentAttention
from .hybrid import HybridDecoderModel, HybridLayer
from .registry import register_model


@dataclass
class BiruvikConfig:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]       # {"type", "mixer": {...}, "mlp": {"kind", "ff"} | None}
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    logit_softcap: Optional[float] = None
    eos_token_id: Optional[Any] = None
    pad_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "BiruvikConfig":
        cap = d.get("logit_softcap")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]),
                   embedding_scale=float(d["embedding"]["scale"]), norm_eps=float(d["norm"]["eps"]),
                   logit_softcap=float(cap) if cap else None, eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def _differential(cfg: BiruvikConfig, m: Dict[str, Any]) -> nn.Module:
    t = m.get("q_temp") or {"coef": 0.0, "every": 0}
    return DifferentialAttention(cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["diff"], cfg.norm_eps,
                                 t["coef"], t["every"])


def _latent(cfg: BiruvikConfig, m: Dict[str, Any]) -> nn.Module:
    mask = m.get("mask") or {}
    return LatentAttention(cfg.width, m["heads"], m["dim"], m["vdim"], None, m["kv_rank"], m["scale"], cfg.norm_eps,
                           window=mask.get("size"), head_gate=True)


def _hgrn2(cfg: BiruvikConfig, m: Dict[str, Any]) -> nn.Module:
    return GatedLinearAttention(cfg.width, m["heads"], m["dim"], m["vdim"], cfg.norm_eps)


MIXERS = {"attention": _differential, "latent_attention": _latent, "hgrn2": _hgrn2}

# module path below a layer -> checkpoint name below 'l<i>.'
_NAMES = {
    "norm1.weight": "norm1", "norm1b.weight": "norm1b", "norm2.weight": "norm2", "norm2b.weight": "norm2b",
    "mlp.up.weight": "mlp.up", "mlp.down.weight": "mlp.down",
    "mixer.query.weight": "mix.q", "mixer.query.bias": "mix.q.b", "mixer.key.weight": "mix.k", "mixer.key.bias": "mix.k.b",
    "mixer.value.weight": "mix.v", "mixer.value.bias": "mix.v.b", "mixer.q_norm.weight": "mix.q.norm", "mixer.k_norm.weight": "mix.k.norm",
    "mixer.lq1": "mix.lq1", "mixer.lk1": "mix.lk1", "mixer.lq2": "mix.lq2", "mixer.lk2": "mix.lk2",
    "mixer.kv_down.weight": "mix.dkv", "mixer.kv_norm.weight": "mix.dkv.norm", "mixer.k_up.weight": "mix.uk", "mixer.v_up.weight": "mix.uv",
    "mixer.gate.weight": "mix.g",
    "mixer.forget.weight": "mix.f", "mixer.forget.bias": "mix.f.b", "mixer.lower": "mix.lower", "mixer.norm.weight": "mix.norm",
    "mixer.out.weight": "mix.o",
}
_TOP = {"word_embeddings.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}


@register_model("Biruvik")
class BiruvikModel(HybridDecoderModel):
    config_class = BiruvikConfig

    def __init__(self, config: BiruvikConfig) -> None:
        layers = []
        for i, spec in enumerate(config.layers):
            if spec["type"] not in MIXERS:
                raise ValueError(f"layer {i}: mixer {spec['type']!r} is not one of {sorted(MIXERS)}")
            mlp = spec.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r} (only 'dense')")
            layers.append(HybridLayer(config.width, MIXERS[spec["type"]](config, spec["mixer"]),
                                      PlainFeedForward(config.width, mlp["ff"]) if mlp is not None else None, config.norm_eps, "rms",
                                      scalar=True))
        super().__init__(config, config.width, config.vocab, layers, config.norm_eps, "rms", embed_scale=config.embedding_scale,
                         softcap=config.logit_softcap, scalar=True)

    @classmethod
    def from_config(cls, config: BiruvikConfig) -> "BiruvikModel":
        return cls(config)

    @staticmethod
    def checkpoint_name(name: str) -> str:
        """The checkpoint's name of one of this module's parameters."""
        if name in _TOP:
            return _TOP[name]
        _, i, rest = name.split(".", 2)
        return f"l{i}.{_NAMES[rest]}"
