"""Retention: linear attention with a constant decay per head and rotary positions on queries and keys,

    S_t = decay S_(t-1) + k_t v_t^T ,   o_t = S_t^T q_t ,

every head's o divided by its own root mean square, multiplied by the silu of a gate and projected.  The memory of the past is the
fp32 state S, as in lightning attention (layers/lightning_attention.py), whose kernels it shares.

The rotary pairs are halves of a head apart (columns i and i + dims / 2): the packed query and key rows are put in an order in
which they are neighbours, the state's rows with them."""
from __future__ import annotations

from typing import Dict, Optional, Sequence

import torch
import torch.nn as nn

from .. import ops
from ..ops import up8
from .lightning_attention import decay_powers
from .packing import Packed, halves_to_pairs, head_cols, head_rows
from .positional_embeddings import PairRotary


class Retention(nn.Module):
    kind = "decay"
    silu = False                # of q, k, v

    def __init__(self, width: int, heads: int, dim: int, vdim: int, decay: Sequence[float], eps: float, rot_base: float = 10000.0,
                 rot_dims: int = 0, rot_scaling: Optional[Dict[str, float]] = None) -> None:
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        if rot_dims > dim:
            raise ValueError(f"{rot_dims} rotated columns of {dim}")
        self.width, self.heads, self.dim, self.vdim, self.eps = width, heads, dim, vdim, float(eps)
        self.decay = tuple(float(d) for d in decay)
        self.rotary, self.k_scale = PairRotary(rot_base, rot_dims, rot_scaling), dim ** -0.5
        self.query = nn.Linear(width, heads * dim, bias=False)
        self.key = nn.Linear(width, heads * dim, bias=False)
        self.value = nn.Linear(width, heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads * vdim, bias=False)
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("state", (self.heads, up8(self.dim), up8(self.vdim)))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            H, dp = self.heads, up8(self.width)
            q, k = (halves_to_pairs(m.weight, H, self.rotary.dims) for m in (self.query, self.key))
            p.w_in = torch.cat([head_rows(w, H, dp) for w in (q, k, self.value.weight, self.gate.weight)]).contiguous()
            p.w_o = head_cols(self.out.weight, H, dp)
            p.decay_pow = decay_powers(self.decay, p.w_in.device)
            p.norm = None           # no weight: every head is normed by itself
        return Packed.of(self, list(self.parameters()), build)

    def matrices(self):
        """Padded input (see packed) and output matrices."""
        p = self.packed()
        return p.w_in, p.w_o

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | k | v | gate]) -> normed, gated heads (B*L, heads * padded vdim); the state advances."""
        p = self.packed()
        H, dim, vdim = self.heads, up8(self.dim), up8(self.vdim)
        o = ops.decay_attention(rows, H, dim, vdim, batch.states(layer), p.decay_pow, B, L, start=batch.start, slots=batch.slots,
                                count=batch.count, silu=False, rotary=self.rotary.table(batch.max_keys, rows.device),
                                k_scale=self.k_scale)
        g0 = H * (2 * dim + vdim)
        return ops.head_norm_gate(o, H, self.vdim, rows[:, g0: g0 + H * vdim], self.eps, out)

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
