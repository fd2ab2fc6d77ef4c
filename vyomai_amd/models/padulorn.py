"""Padulorn: a small decoder-only language model that mixes retention and windowed attention (kept first tokens, norms over the whole
query and key projection, YaRN-scaled rotary positions, values mixed with those of the first such layer), each followed by an
optional mixture of plain experts with a sigmoid router; one norm per sublayer, on its output.  Sizes, constants and the order of
layers come from its configuration; the machinery is models/hybrid.py."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Union

import torch.nn as nn

from ..layers.ffn import MixtureFeedForward
from ..layers.retention import Retention
from ..layers.window_attention import VALUES_FIRST, VALUES_MIX, VALUES_OWN, WindowAttention
from .hybrid import HybridDecoderModel, HybridLayer
from .registry import register_model


@dataclass
class PadulornConfig:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]       # {"type", "mixer": {...}, "mlp": {"kind", "router", "expert"} | None}
    embedding_scale: float = 1.0
    norm_eps: float = 1e-5
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    eos_token_id: Optional[Any] = None
    pad_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "PadulornConfig":
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=list(d["layers"]),
                   embedding_scale=float(d["embedding"]["scale"]), norm_eps=float(d["norm"]["eps"]),
                   residual_mult=float(d["residual_mult"]), logit_scale=float(d["logit_scale"]),
                   eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def _attention(cfg: PadulornConfig, m: Dict[str, Any], values: int) -> nn.Module:
    rot, mask = m["rot"], m["mask"]
    return WindowAttention(cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], mask["size"], rot["base"], rot["dims"],
                           sink=False, gate=False, keep_first=mask.get("keep_first") or 0, rot_scaling=rot.get("scaling"),
                           qk_norm_eps=cfg.norm_eps, values=values)


def _retention(cfg: PadulornConfig, m: Dict[str, Any], values: int) -> nn.Module:
    rot = m["rot"]
    return Retention(cfg.width, m["heads"], m["dim"], m["vdim"], m["decay"], cfg.norm_eps, rot["base"], rot["dims"], rot.get("scaling"))


def _mixture(cfg: PadulornConfig, m: Dict[str, Any]) -> nn.Module:
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    return MixtureFeedForward(cfg.width, r["experts"], r["top"], m["expert"]["ff"], groups=groups["count"], keep=groups["keep"],
                              act="gelu", score="sigmoid", group_best=2, normalize=False)


MIXERS = {"attention": _attention, "retention": _retention}
FEED_FORWARDS = {"moe": _mixture}

# module path below a layer -> checkpoint name below 'l<i>.'
_NAMES = {
    "norm1b.weight": "norm1", "norm2b.weight": "norm2",
    "mixer.query.weight": "mix.q", "mixer.key.weight": "mix.k", "mixer.value.weight": "mix.v", "mixer.gate.weight": "mix.g",
    "mixer.out.weight": "mix.o", "mixer.q_norm.weight": "mix.q.norm", "mixer.k_norm.weight": "mix.k.norm", "mixer.value_mix": "mix.vmix",
    "mlp.router.weight": "mlp.router",
}
_EXPERTS = {"mlp.up": "up", "mlp.down": "down"}
_TOP = {"word_embeddings.weight": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}


@register_model("Padulorn")
class PadulornModel(HybridDecoderModel):
    config_class = PadulornConfig

    def __init__(self, config: PadulornConfig) -> None:
        layers, mixes = [], 0      # mixes: columns of the values that later layers mix in
        for i, spec in enumerate(config.layers):
            kind, mlp = spec["type"], spec.get("mlp")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: mixer {kind!r} is not one of {sorted(MIXERS)}")
            if mlp is not None and mlp["kind"] not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r} is not one of {sorted(FEED_FORWARDS)}")
            values = VALUES_OWN
            if spec["mixer"].get("v_mix"):
                values, columns = VALUES_MIX if mixes else VALUES_FIRST, spec["mixer"]["kv_heads"] * spec["mixer"]["vdim"]
                if mixes not in (0, columns):
                    raise ValueError(f"layer {i}: values of {columns} columns cannot be mixed with {mixes}")
                mixes = columns
            layers.append(HybridLayer(config.width, MIXERS[kind](config, spec["mixer"], values),
                                      FEED_FORWARDS[mlp["kind"]](config, mlp) if mlp is not None else None, config.norm_eps, "rms",
                                      pre=False, mult=config.residual_mult))
        super().__init__(config, config.width, config.vocab, layers, config.norm_eps, "rms", embed_scale=config.embedding_scale,
                         logit_scale=config.logit_scale)

    @classmethod
    def from_config(cls, config: PadulornConfig) -> "PadulornModel":
        return cls(config)

    def checkpoint_name(self, name: str) -> Union[str, List[str]]:
        """The checkpoint's name (the experts': names) of one of this module's parameters."""
        if name in _TOP:
            return _TOP[name]
        _, i, rest = name.split(".", 2)
        if rest in _EXPERTS:
            return [f"l{i}.mlp.e{e}.{_EXPERTS[rest]}" for e in range(self.layers[int(i)].mlp.experts)]
        return f"l{i}.{_NAMES[rest]}"
