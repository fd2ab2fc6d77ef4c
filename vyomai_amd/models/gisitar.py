"""Gisitar: a small decoder-only language model that mixes latent attention (without positions) and lightning attention,
with norms on both sides of every sublayer.  Sizes, constants and the order of layers come from its configuration; the
machinery is models/hybrid.py."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

import torch.nn as nn

from ..layers.ffn import GatedFeedForward
from ..layers.latent_attention import LatentAttention
from ..layers.lightning_attention import LightningAttention
from .hybrid import HybridDecoderModel, HybridLayer
from .registry import register_model


@dataclass
class GisitarConfig:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]       # {"type", "mixer": {...}, "mlp": {"kind", "ff"} | None}
    norm_eps: float = 1e-5
    eos_token_id: Optional[Any] = None
    pad_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "GisitarConfig":
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]), norm_eps=float(d["norm"]["eps"]),
                   eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def _latent(cfg: GisitarConfig, m: Dict[str, Any]) -> nn.Module:
    return LatentAttention(cfg.width, m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["scale"], cfg.norm_eps)


def _lightning(cfg: GisitarConfig, m: Dict[str, Any]) -> nn.Module:
    return LightningAttention(cfg.width, m["heads"], m["dim"], m["vdim"], m["decay"], cfg.norm_eps)


MIXERS = {"latent_attention": _latent, "lightning": _lightning}

# module path below a layer -> checkpoint name below 'l<i>.'
_NAMES = {
    "norm1.weight": "norm1", "norm1b.weight": "norm1b", "norm2.weight": "norm2", "norm2b.weight": "norm2b",
    "mlp.gate.weight": "mlp.gate", "mlp.up.weight": "mlp.up", "mlp.down.weight": "mlp.down",
    "mixer.gate.weight": "mix.g", "mixer.out.weight": "mix.o",
    "mixer.q_down.weight": "mix.dq", "mixer.q_norm.weight": "mix.dq.norm", "mixer.q_up.weight": "mix.uq",
    "mixer.kv_down.weight": "mix.dkv", "mixer.kv_norm.weight": "mix.dkv.norm", "mixer.k_up.weight": "mix.uk",
    "mixer.v_up.weight": "mix.uv",
    "mixer.query.weight": "mix.q", "mixer.key.weight": "mix.k", "mixer.value.weight": "mix.v", "mixer.norm.weight": "mix.norm",
}
_TOP = {"word_embeddings.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}


@register_model("Gisitar")
class GisitarModel(HybridDecoderModel):
    config_class = GisitarConfig

    def __init__(self, config: GisitarConfig) -> None:
        layers = []
        for i, spec in enumerate(config.layers):
            if spec["type"] not in MIXERS:
                raise ValueError(f"layer {i}: mixer {spec['type']!r} is not one of {sorted(MIXERS)}")
            mlp = spec.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r} (only 'dense')")
            layers.append(HybridLayer(config.width, MIXERS[spec["type"]](config, spec["mixer"]),
                                      GatedFeedForward(config.width, mlp["ff"]) if mlp is not None else None, config.norm_eps))
        super().__init__(config, config.width, config.vocab, layers, config.norm_eps)

    @classmethod
    def from_config(cls, config: GisitarConfig) -> "GisitarModel":
        return cls(config)

    @staticmethod
    def checkpoint_name(name: str) -> str:
        """The checkpoint's name of one of this module's parameters."""
        if name in _TOP:
            return _TOP[name]
        _, i, rest = name.split(".", 2)
        return f"l{i}.{_NAMES[rest]}"
