"""Lightning attention: linear attention with a constant decay per head,

    S_t = decay S_(t-1) + k_t v_t^T ,   o_t = S_t^T q_t ,   q, k, v = silu of the projections,

the concatenated heads RMS-normed together, multiplied by a sigmoid gate and projected.  The only memory of the past is
the fp32 state S (one dk x dv matrix per head and sequence)."""
from __future__ import annotations

from typing import Optional, Sequence

import torch
import torch.nn as nn

from .. import ops
from .._lib import DECAY_CHUNK
from ..ops import up8
from .norms import WeightNorm
from .packing import Packed, head_cols, head_rows, head_vec


def decay_powers(decay: Sequence[float], device) -> torch.Tensor:
    """(heads, DECAY_CHUNK + 1) fp32: powers of the decays, made in double precision and rounded once."""
    t = torch.tensor([[d ** i for i in range(DECAY_CHUNK + 1)] for d in decay], dtype=torch.float64)
    return t.float().to(device)


class LightningAttention(nn.Module):
    kind = "decay"
    silu, rotary, k_scale = True, None, 1.0     # of q, k, v; rotary positions and factor on the keys: none

    def __init__(self, width: int, heads: int, dim: int, vdim: int, decay: Sequence[float], eps: float) -> None:
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        self.width, self.heads, self.dim, self.vdim, self.eps = width, heads, dim, vdim, float(eps)
        self.decay = tuple(float(d) for d in decay)
        self.query = nn.Linear(width, heads * dim, bias=False)
        self.key = nn.Linear(width, heads * dim, bias=False)
        self.value = nn.Linear(width, heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads * vdim, bias=False)
        self.norm = WeightNorm(heads * vdim, eps, "rms")
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("state", (self.heads, up8(self.dim), up8(self.vdim)))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            H, dp = self.heads, up8(self.width)
            p.w_in = torch.cat([head_rows(m.weight, H, dp)
                                for m in (self.query, self.key, self.value, self.gate)]).contiguous()
            p.norm = head_vec(self.norm.weight, H)
            p.w_o = head_cols(self.out.weight, H, dp)
            p.decay_pow = decay_powers(self.decay, p.w_in.device)
        return Packed.of(self, list(self.parameters()), build)

    def matrices(self):
        """Padded input (see packed) and output matrices."""
        p = self.packed()
        return p.w_in, p.w_o

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | k | v | gate]) -> gated heads (B*L, heads * padded vdim); the state advances."""
        p = self.packed()
        H, dim, vdim = self.heads, up8(self.dim), up8(self.vdim)
        o = ops.decay_attention(rows, H, dim, vdim, batch.states(layer), p.decay_pow, B, L, start=batch.start,
                                slots=batch.slots, count=batch.count)
        g0 = H * (2 * dim + vdim)
        return ops.rmsnorm_gate(o, p.norm, H * self.vdim, rows[:, g0: g0 + H * vdim], self.eps, out)

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
