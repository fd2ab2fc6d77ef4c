"""Gated linear attention with a forget gate per key channel, tied to the input gate 1 - f (HGRN2),

    f = lower + (1 - lower) sigmoid(W_f h + b) ,   S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T ,   o_t = S_t^T q_t ,

q = silu of its projection; every head's o is RMS-normed with a weight that the heads share, then projected.  The memory of the
past is the fp32 state S, as in lightning attention (layers/lightning_attention.py), whose recurrence and scan it shares."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops import up8
from .norms import WeightNorm
from .packing import Packed, head_cols, head_rows, head_vec, pad_vec


class GatedLinearAttention(nn.Module):
    kind = "gated"
    silu = True                 # of q

    def __init__(self, width: int, heads: int, dim: int, vdim: int, eps: float) -> None:
        super().__init__()
        self.width, self.heads, self.dim, self.vdim, self.eps = width, heads, dim, vdim, float(eps)
        self.query = nn.Linear(width, heads * dim, bias=False)
        self.forget = nn.Linear(width, heads * dim)
        self.lower = nn.Parameter(torch.zeros(heads * dim))      # least value of every gate
        self.value = nn.Linear(width, heads * vdim, bias=False)
        self.norm = WeightNorm(vdim, eps, "rms")
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("state", (self.heads, up8(self.dim), up8(self.vdim)))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            H, dp = self.heads, up8(self.width)
            p.w_in = torch.cat([head_rows(m.weight, H, dp) for m in (self.query, self.forget, self.value)]).contiguous()
            p.f_bias = head_vec(self.forget.bias, H)             # (added in fp32, with the gate)
            p.f_lower = 1.0 - head_vec(1.0 - self.lower.float(), H)   # 1 in padded channels: nothing is written there
            p.norm = pad_vec(self.norm.weight, up8(self.vdim))
            p.w_o = head_cols(self.out.weight, H, dp)
        return Packed.of(self, list(self.parameters()), build)

    def matrices(self):
        """Padded input (see packed) and output matrices."""
        p = self.packed()
        return p.w_in, p.w_o

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | gate | v]) -> normed heads (B*L, heads * padded vdim); the state advances."""
        p = self.packed()
        o = ops.gated_attention(rows, self.heads, up8(self.dim), up8(self.vdim), batch.states(layer), p.f_lower, p.f_bias, B, L,
                                start=batch.start, slots=batch.slots, count=batch.count, silu=self.silu)
        return ops.head_norm_gate(o, self.heads, self.vdim, None, self.eps, out, p.norm)

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
