"""Latent attention: queries through a low-rank latent (or projected directly), keys and values expanded per head from ONE
normalised latent per token, which is all that is cached; softmax over every earlier token, or over the last `window` ones (then
the cache is a ring of so many latents); sigmoid gate on the output, one number per column or per head.

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

    def __init__(self, width: int, heads: int, dim: int, vdim: int, q_rank: Optional[int], kv_rank: int, scale: float,
                 eps: float, window: Optional[int] = None, head_gate: bool = False) -> None:
        """q_rank None: no latent in front of the queries.  window None: every earlier token.  head_gate: a gate per head."""
        super().__init__()
        if window is not None and window < 1:
            raise ValueError(f"window {window}")
        self.width, self.heads, self.dim, self.vdim = width, heads, dim, vdim
        self.q_rank, self.kv_rank, self.scale, self.eps = q_rank, kv_rank, float(scale), float(eps)
        self.window, self.head_gate = window, bool(head_gate)
        if q_rank is None:
            self.query = nn.Linear(width, heads * dim, bias=False)
        else:
            self.q_down = nn.Linear(width, q_rank, bias=False)
            self.q_norm = WeightNorm(q_rank, eps, "rms")
            self.q_up = nn.Linear(q_rank, heads * dim, bias=False)
        self.kv_down = nn.Linear(width, kv_rank, bias=False)
        self.kv_norm = WeightNorm(kv_rank, eps, "rms")
        self.k_up = nn.Linear(kv_rank, heads * dim, bias=False)
        self.v_up = nn.Linear(kv_rank, heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads if head_gate else heads * vdim, bias=False)
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        if self.window is not None:
            return ("window", (1, up8(self.kv_rank), self.window))
        return ("latent", up8(self.kv_rank))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            H, dp, kr = self.heads, up8(self.width), up8(self.kv_rank)
            if self.q_rank is None:
                first = head_rows(self.query.weight, H, dp)
            else:
                qr = up8(self.q_rank)
                first = pad2(self.q_down.weight, qr, dp)
                p.q_norm, p.w_uq = pad_vec(self.q_norm.weight, qr), head_rows(self.q_up.weight, H, qr)
            gate = pad2(self.gate.weight, up8(H), dp) if self.head_gate else head_rows(self.gate.weight, H, dp)
            p.w_in = torch.cat([first, pad2(self.kv_down.weight, kr, dp), gate]).contiguous()
            p.n_first, p.c_norm = first.shape[0], pad_vec(self.kv_norm.weight, kr)
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
        """Packed projections (B*L, [q latent or q | kv latent | gate]) -> gated heads (B*L, heads * padded vdim).  The latents
        of the new tokens go to the cache."""
        p = self.packed()
        H, dim, vdim, kr = self.heads, up8(self.dim), up8(self.vdim), p.c_norm.numel()
        cache, at = batch.latents(layer), dict(slots=batch.slots, start=batch.start)
        past = 0 if batch.fresh else batch.past if self.window is None else min(self.window - 1, batch.past)
        behind = self.window is not None and past > 0       # the ring's old rows are read before new ones take their places
        norm_q, n_q = (p.q_norm, self.q_rank) if self.q_rank is not None else (None, p.n_first)
        cq, c = ops.latent_norm(rows, norm_q, n_q, p.c_norm, self.kv_rank, B, L, self.eps, cache=None if behind else cache, **at,
                                count=batch.count, want_c=batch.fresh or self.window is not None)
        q = ops.linear(cq, p.w_uq) if cq is not None else rows[:, : p.n_first]
        S = L
        if behind:
            S, new = past + L, (c, B, L, 1, kr, 0, 0, kr)
            c = ops.window_context(*new, cache, past, **at).view(B * S, kr)
            ops.window_rows(*new, ring=cache, count=batch.count, **at)
        elif past:
            S = batch.max_keys
            c = cache.index_select(0, batch.slots)[:, :S].reshape(B * S, -1)
        kv = ops.linear(c, p.w_ukv).view(B, S, -1)
        q = q.unflatten(0, (B, L)).unflatten(2, (H, dim)).transpose(1, 2)
        k = kv[..., : H * dim].unflatten(-1, (H, dim)).transpose(1, 2)
        v = kv[..., H * dim:].unflatten(-1, (H, vdim)).transpose(1, 2)
        g0 = p.n_first + kr
        gate = rows[:, g0: g0 + (up8(H) if self.head_gate else H * vdim)].unflatten(0, (B, L))
        win = {} if self.window is None else dict(window=self.window, start_cap=past)
        o = ops.attention_ex(q, k, v, self.scale, gate=gate, gate_heads=self.head_gate, out=None if out is None else out.unflatten(0, (B, L)),
                             **win, **({} if past == 0 else at))
        return o.view(B * L, -1) if out is None else out

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        """h (B*L, padded width) of the new tokens -> mixer output (B*L, padded width)."""
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
