"""Latent attention: queries through a low-rank latent, keys and values expanded per head from ONE normalised latent per
token, which is all that is cached; softmax over every earlier token; sigmoid gate on the output.

Prefill expands keys and values of the whole context with one product and runs the flash kernel (values have a width of
their own, the gate is its epilogue).  Decode never expands them: vy_latent_decode takes the query into the latent space.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops import up8
from .norms import WeightNorm
from .packing import Packed, head_cols, head_rows, pad2, pad_vec


class LatentAttention(nn.Module):
    kind = "latent"

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: int, kv_rank: int, scale: float,
                 eps: float) -> None:
        super().__init__()
        self.width, self.heads, self.dim, self.vdim = width, heads, dim, vdim
        self.q_rank, self.kv_rank, self.scale, self.eps = q_rank, kv_rank, float(scale), float(eps)
        self.q_down = nn.Linear(width, q_rank, bias=False)
        self.q_norm = WeightNorm(q_rank, eps, "rms")
        self.q_up = nn.Linear(q_rank, heads * dim, bias=False)
        self.kv_down = nn.Linear(width, kv_rank, bias=False)
        self.kv_norm = WeightNorm(kv_rank, eps, "rms")
        self.k_up = nn.Linear(kv_rank, heads * dim, bias=False)
        self.v_up = nn.Linear(kv_rank, heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads * vdim, bias=False)
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("latent", up8(self.kv_rank))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            H, dp, qr, kr = self.heads, up8(self.width), up8(self.q_rank), up8(self.kv_rank)
            p.w_in = torch.cat([pad2(self.q_down.weight, qr, dp), pad2(self.kv_down.weight, kr, dp),
                                head_rows(self.gate.weight, H, dp)]).contiguous()
            p.q_norm, p.c_norm = pad_vec(self.q_norm.weight, qr), pad_vec(self.kv_norm.weight, kr)
            p.w_uq = head_rows(self.q_up.weight, H, qr)
            w_uk, p.w_uv = head_rows(self.k_up.weight, H, kr), head_rows(self.v_up.weight, H, kr)
            p.w_ukv = torch.cat([w_uk, p.w_uv]).contiguous()                               # prefill: one product
            p.w_uv = p.w_ukv[w_uk.shape[0]:]                                               # decode, (H * vdim, kr)
            p.w_ukt = w_uk.view(H, -1, kr).transpose(1, 2).contiguous()                    # decode, (H, kr, dim)
            p.w_o = head_cols(self.out.weight, H, dp)
        return Packed.of(self, list(self.parameters()), build)

    def matrices(self):
        """Padded input (see packed) and output matrices."""
        p = self.packed()
        return p.w_in, p.w_o

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q latent | kv latent | gate]) -> gated heads (B*L, heads * padded vdim).  The latents of
        the new tokens go to the cache."""
        p = self.packed()
        H, dim, vdim = self.heads, up8(self.dim), up8(self.vdim)
        cache = batch.latents(layer)
        cq, c = ops.latent_norm(rows, p.q_norm, self.q_rank, p.c_norm, self.kv_rank, B, L, self.eps, cache=cache,
                                slots=batch.slots, start=batch.start, count=batch.count, want_c=batch.fresh)
        q = ops.linear(cq, p.w_uq).view(B, L, H, dim).transpose(1, 2)
        S = L if batch.fresh else batch.max_keys
        if not batch.fresh:
            c = cache.index_select(0, batch.slots)[:, :S].reshape(B * S, -1)
        kv = ops.linear(c, p.w_ukv).view(B, S, -1)
        k = kv[..., : H * dim].unflatten(-1, (H, dim)).transpose(1, 2)
        v = kv[..., H * dim:].unflatten(-1, (H, vdim)).transpose(1, 2)
        g0 = cq.shape[1] + p.c_norm.numel()
        gate = rows[:, g0: g0 + H * vdim].unflatten(0, (B, L))
        o = ops.attention_ex(q, k, v, self.scale, gate=gate, start=None if batch.fresh else batch.start,
                             slots=None if batch.fresh else batch.slots, out=None if out is None else out.unflatten(0, (B, L)))
        return o.view(B * L, -1) if out is None else out

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        """h (B*L, padded width) of the new tokens -> mixer output (B*L, padded width)."""
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
