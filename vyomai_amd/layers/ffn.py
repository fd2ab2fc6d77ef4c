"""FeedForward with the reference's signature and parameter names (VyomAI/layers/ffn.py:18-40):
LN(dropout(out(act(intermediate(x)))) + input_tensor), width multiplier*hidden (NOT
config.intermediate_size, like the reference :19-23).

MI355X: two MFMA GEMM launches -- bias+GELU in the first epilogue, bias+dropout+residual in the
second -- and one LayerNorm launch."""
from __future__ import annotations

from typing import Union

import torch
import torch.nn as nn

from .. import ops
from .._lib import ACT_GELU_ERF, ACT_GELU_TANH, ACT_SILU
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
    """down(act(gate(x)) * up(x)), no biases: one packed [gate; up] product, the gated activation, one product."""

    def __init__(self, width: int, inner: int, act: str = "silu") -> None:
        super().__init__()
        self.width, self.inner, self.act = width, inner, _GATED_ACT[act]
        self.gate = nn.Linear(width, inner, bias=False)
        self.up = nn.Linear(width, inner, bias=False)
        self.down = nn.Linear(inner, width, bias=False)

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            dp, ip = up8(self.width), up8(self.inner)
            p.w_gu = torch.cat([pad2(self.gate.weight, ip, dp), pad2(self.up.weight, ip, dp)]).contiguous()
            p.w_down = pad2(self.down.weight, dp, ip).contiguous()
        return Packed.of(self, list(self.parameters()), build)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        p = self.packed()
        return ops.linear(ops.gated_act(ops.linear(h, p.w_gu), self.act), p.w_down)
