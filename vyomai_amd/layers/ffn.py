"""FeedForward with the reference's signature and parameter names (VyomAI/layers/ffn.py:18-40):
LN(dropout(out(act(intermediate(x)))) + input_tensor), width multiplier*hidden (NOT
config.intermediate_size, like the reference :19-23).

MI355X: two MFMA GEMM launches -- bias+GELU in the first epilogue, bias+dropout+residual in the
second -- and one LayerNorm launch."""
from __future__ import annotations

from typing import Optional, Union

import torch
import torch.nn as nn

from .. import ops
from .._lib import (ACT_GELU_ERF, ACT_GELU_TANH, ACT_RELU2, ACT_SILU, MOE_CLAMPED, MOE_GELU, SCORE_SIGMOID, SCORE_SOFTMAX, VyMoe)
from ..ops import up8
from .packing import Packed, pad2

# activations with a fused HIP epilogue; the reference's table (:7-15) also lists leaky_relu,
# relu6, sigmoid, silu/swish, tanh, which no shipped model or test selects.
_FUSED_ACT = {"gelu": ACT_GELU_ERF, "gelu_tanh": ACT_GELU_TANH, "gelu_pytorch_tanh": ACT_GELU_TANH}
_REFERENCE_ACTS = {"gelu", "leaky_relu", "relu6", "sigmoid", "silu", "swish", "tanh"}


class FeedForward(nn.Module):
    def __init__(self, config, multiplier: Union[int, float] = 4) -> None:
        super().__init__()
        inner = int(multiplier) * config.hidden_size
        self.intermediate = nn.Linear(config.hidden_size, inner)
        self.dropout = nn.Dropout(config.hidden_dropout_prob)
        self.layernorm = nn.LayerNorm(config.hidden_size, eps=config.layer_norm_eps)
        name = getattr(config, "hidden_act", None)
        if name in _FUSED_ACT:
            self.act = _FUSED_ACT[name]
        elif name in _REFERENCE_ACTS:
            raise NotImplementedError(f"hidden_act={name!r} has no fused MI355X epilogue yet (gelu only)")
        else:
            self.act = ACT_GELU_ERF  # unknown names fall back to GELU like the reference (:26-29)
        self.out = nn.Linear(inner, config.hidden_size)

    def forward(self, hidden_state: torch.Tensor, input_tensor: torch.Tensor) -> torch.Tensor:
        from ..autograd import ffn_block
        return ffn_block(hidden_state, input_tensor, self.intermediate.weight, self.intermediate.bias,
                         self.out.weight, self.out.bias, self.layernorm.weight, self.layernorm.bias,
                         self.layernorm.eps, self.act, self.dropout.p, self.training)


_GATED_ACT = {"silu": ACT_SILU, "gelu_tanh": ACT_GELU_TANH, "gelu": ACT_GELU_ERF}


class GatedFeedForward(nn.Module):
    """down(act(gate(x)) * up(x)), no biases: one packed [gate; up] product, the gated activation, one product.
    act "clamped": with g = min(gate, limit), u = clamp(up, -limit, limit): down(g sigmoid(alpha g) (u + 1))."""

    def __init__(self, width: int, inner: int, act: str = "silu", limit: float = 0.0, alpha: float = 1.702) -> None:
        super().__init__()
        self.width, self.inner, self.limit, self.alpha = width, inner, float(limit), float(alpha)
        self.clamped = act == "clamped"
        self.act = None if self.clamped else _GATED_ACT[act]
        self.gate = nn.Linear(width, inner, bias=False)
        self.up = nn.Linear(width, inner, bias=False)
        self.down = nn.Linear(inner, width, bias=False)

    def matrices(self):
        """Padded [gate; up] and down matrices."""
        dp, ip = up8(self.width), up8(self.inner)
        return torch.cat([pad2(self.gate.weight, ip, dp), pad2(self.up.weight, ip, dp)]), pad2(self.down.weight, dp, ip)

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            p.w_gu, p.w_down = (w.contiguous() for w in self.matrices())
        return Packed.of(self, list(self.parameters()), build)

    def activation(self, gate_up: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        if self.clamped:
            return ops.clamped_act(gate_up, self.limit, self.alpha, out)
        return ops.gated_act(gate_up, self.act, out)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        p = self.packed()
        return ops.linear(self.activation(ops.linear(h, p.w_gu)), p.w_down)

    # what a layer asks of its feed-forward: the part that runs on every token, and the routed rows beside it
    @property
    def dense(self) -> Optional["GatedFeedForward"]:
        return self

    def routed(self, h: torch.Tensor, L: int = 1, count: Optional[torch.Tensor] = None) -> Optional["ops.Routed"]:
        return None


_PLAIN_ACT = {"relu2": ACT_RELU2, "gelu_tanh": ACT_GELU_TANH, "gelu": ACT_GELU_ERF}


class PlainFeedForward(nn.Module):
    """down(act(up(x))), no gate and no biases: the activation is the first product's epilogue.  act "relu2": max(z, 0)^2."""
    clamped, limit, alpha = False, 0.0, 0.0

    def __init__(self, width: int, inner: int, act: str = "relu2") -> None:
        super().__init__()
        self.width, self.inner, self.act = width, inner, _PLAIN_ACT[act]
        self.up = nn.Linear(width, inner, bias=False)
        self.down = nn.Linear(inner, width, bias=False)

    def matrices(self):
        raise ValueError("a feed-forward without a gate does not share its products with a mixer's (no parallel layers)")

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            dp, ip = up8(self.width), up8(self.inner)
            p.w_up, p.w_down = pad2(self.up.weight, ip, dp).contiguous(), pad2(self.down.weight, dp, ip).contiguous()
        return Packed.of(self, list(self.parameters()), build)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        p = self.packed()
        return ops.linear(ops.linear(h, p.w_up, act=self.act), p.w_down)

    @property
    def dense(self) -> Optional["PlainFeedForward"]:
        return self

    def routed(self, h: torch.Tensor, L: int = 1, count: Optional[torch.Tensor] = None) -> Optional["ops.Routed"]:
        return None


_EXPERT_ACT = {"clamped": MOE_CLAMPED, "gelu": MOE_GELU}
_SCORE = {"softmax": SCORE_SOFTMAX, "sigmoid": SCORE_SIGMOID}


class MixtureFeedForward(nn.Module):
    """`top` of `experts` small feed-forwards per token and (shared may be None) one dense one for every token.  act "clamped":
    the clamped gated one of GatedFeedForward; "gelu": down(gelu(up(x))), the exact GELU, no gate.

    Router scores are softmax(router(x)) or sigmoid(router(x)) (`score`) in fp32; experts form `groups` equal groups of neighbours
    and only those of the `keep` best groups can be chosen (a group's score: the sum of its `group_best` largest scores, 1 or 2);
    the chosen scores are normalised to sum 1 (if `normalize`) and multiplied by `scale`.  The experts' weights are one tensor each (experts first); once packed, they are views of the packed storage, so there is one
    copy of them in memory."""

    def __init__(self, width: int, experts: int, top: int, inner: int, limit: float = 0.0, groups: int = 1, keep: int = 1,
                 scale: float = 1.0, alpha: float = 1.702, shared: Optional[GatedFeedForward] = None, act: str = "clamped",
                 score: str = "softmax", group_best: int = 1, normalize: bool = True) -> None:
        super().__init__()
        if experts < 1 or groups < 1 or experts % groups or not 1 <= keep <= groups or not 1 <= top <= keep * (experts // groups):
            raise ValueError(f"{top} of {experts} experts, {keep} of {groups} groups")
        if act not in _EXPERT_ACT or score not in _SCORE or group_best not in (1, 2):
            raise ValueError(f"experts' activation {act!r}, scores {score!r}, groups by {group_best} scores")
        self.width, self.experts, self.top, self.inner, self.limit, self.alpha = width, experts, top, inner, float(limit), float(alpha)
        self.groups, self.keep, self.scale = groups, keep, float(scale)
        self.act, self.score, self.group_best, self.normalize = _EXPERT_ACT[act], _SCORE[score], int(group_best), bool(normalize)
        self.router = nn.Linear(width, experts, bias=False)
        self.gate = nn.Parameter(torch.empty(experts, inner, width)) if self.act == MOE_CLAMPED else None
        self.up = nn.Parameter(torch.empty(experts, inner, width))
        self.down = nn.Parameter(torch.empty(experts, width, inner))
        self.shared = shared

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            dp, ip, n, w = up8(self.width), up8(self.inner), self.inner, self.width
            dt, dev = self.up.dtype, self.up.device
            p.w_router = pad2(self.router.weight, self.experts, dp).contiguous()
            rows = 1 if self.gate is None else 2      # rows interleaved: gate 0, up 0, gate 1, ...
            p.w_gu = torch.zeros(self.experts, rows * ip, dp, dtype=dt, device=dev)
            p.w_down = torch.zeros(self.experts, dp, ip, dtype=dt, device=dev)
            for param, place in ((self.gate, p.w_gu[:, 0:2 * n:2, :w]), (self.up, p.w_gu[:, rows - 1:rows * n:rows, :w]),
                                 (self.down, p.w_down[:, :w, :n])):
                if param is not None:
                    place.copy_(param)
                    param.data = place
            p.desc = VyMoe(self.experts, self.top, self.groups, self.keep, dp, ip, self.act, self.score, self.group_best,
                           int(self.normalize), self.scale, self.limit, self.alpha, p.w_router.data_ptr(), p.w_gu.data_ptr(),
                           p.w_down.data_ptr())
        return Packed.of(self, [p for p in (self.router.weight, self.gate, self.up, self.down) if p is not None], build)

    @property
    def dense(self) -> Optional[GatedFeedForward]:
        return self.shared

    def routed(self, h: torch.Tensor, L: int = 1, count: Optional[torch.Tensor] = None) -> "ops.Routed":
        return ops.moe(h, self.packed().desc, L, count)
