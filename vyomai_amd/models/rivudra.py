"""Rivudra: a small decoder-only language model of parallel layers: windowed attention (grouped heads, rotary positions on
neighbouring columns, a sink, an output gate) beside a mixture of experts with a shared one, both reading one norm.  Sizes,
constants and the order of layers come from its configuration; the machinery is models/hybrid.py."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Union

import torch.nn as nn

from ..layers.ffn import GatedFeedForward, MixtureFeedForward
from ..layers.window_attention import WindowAttention
from .hybrid import HybridDecoderModel, ParallelLayer
from .registry import register_model

SWISH_ALPHA = 1.702   # the experts' gate: g sigmoid(SWISH_ALPHA g)


@dataclass
class RivudraConfig:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]       # {"type", "mixer": {...}, "mlp": {"kind", "router", "expert", "shared"} | None}
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    eos_token_id: Optional[Any] = None
    pad_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "RivudraConfig":
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]),
                   embedding_scale=float(d["embedding"]["scale"]), norm_eps=float(d["norm"]["eps"]),
                   eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def _attention(cfg: RivudraConfig, m: Dict[str, Any]) -> nn.Module:
    return WindowAttention(cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["mask"]["size"],
                           m["rot"]["base"], m["rot"]["dims"], sink=True)


def _mixture(cfg: RivudraConfig, m: Dict[str, Any]) -> nn.Module:
    r, e, s = m["router"], m["expert"], m.get("shared")
    groups = r.get("groups") or {"count": 1, "keep": 1}
    shared = None if s is None else GatedFeedForward(cfg.width, s["ff"], "clamped", s["limit"], SWISH_ALPHA)
    return MixtureFeedForward(cfg.width, r["experts"], r["top"], e["ff"], e["limit"], groups["count"], groups["keep"], r["scale"],
                              SWISH_ALPHA, shared)


MIXERS = {"attention": _attention}
FEED_FORWARDS = {"moe": _mixture}

# module path below a layer -> checkpoint name below 'l<i>.'
_NAMES = {
    "norm1.weight": "norm1",
    "mixer.query.weight": "mix.q", "mixer.key.weight": "mix.k", "mixer.value.weight": "mix.v", "mixer.gate.weight": "mix.g",
    "mixer.out.weight": "mix.o",
    "mlp.router.weight": "mlp.router", "mlp.shared.gate.weight": "mlp.shared.gate", "mlp.shared.up.weight": "mlp.shared.up",
    "mlp.shared.down.weight": "mlp.shared.down",
}
_EXPERTS = {"mlp.gate": "gate", "mlp.up": "up", "mlp.down": "down"}
_TOP = {"word_embeddings.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}


@register_model("Rivudra")
class RivudraModel(HybridDecoderModel):
    config_class = RivudraConfig

    def __init__(self, config: RivudraConfig) -> None:
        layers = []
        for i, spec in enumerate(config.layers):
            if spec["type"] not in MIXERS:
                raise ValueError(f"layer {i}: mixer {spec['type']!r} is not one of {sorted(MIXERS)}")
            mlp = spec.get("mlp")
            if mlp is not None and mlp["kind"] not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r} is not one of {sorted(FEED_FORWARDS)}")
            layers.append(ParallelLayer(config.width, MIXERS[spec["type"]](config, spec["mixer"]),
                                        FEED_FORWARDS[mlp["kind"]](config, mlp) if mlp is not None else None,
                                        config.norm_eps, "rms", offset=1.0))
        super().__init__(config, config.width, config.vocab, layers, config.norm_eps, "rms", offset=1.0,
                         embed_scale=config.embedding_scale)

    @classmethod
    def from_config(cls, config: RivudraConfig) -> "RivudraModel":
        return cls(config)

    def checkpoint_name(self, name: str) -> Union[str, List[str]]:
        """The checkpoint's name (the experts': names) of one of this module's parameters."""
        if name in _TOP:
            return _TOP[name]
        _, i, rest = name.split(".", 2)
        if rest in _EXPERTS:
            return [f"l{i}.mlp.e{e}.{_EXPERTS[rest]}" for e in range(self.layers[int(i)].mlp.experts)]
        return f"l{i}.{_NAMES[rest]}"
