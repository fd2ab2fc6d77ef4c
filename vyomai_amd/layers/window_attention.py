"""Sliding-window attention: grouped query heads (values may have a width of their own), rotary positions on neighbouring
columns, an optional sink (one added to every softmax denominator) and a sigmoid gate on the output.  Query i sees the last
`window` tokens up to itself, so a sequence's memory is a ring of `window` rows per key/value head.

Prefill rotates the keys in place in the packed projection rows and runs the flash kernel (the queries' rotation, window, sink
and gate are its own); behind a past the ring's rows and the new ones form the context.  Decode is vy_window_decode.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops import up8
from .packing import Packed, head_cols, head_rows
from .positional_embeddings import PairRotary


class WindowAttention(nn.Module):
    kind = "window"

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, window: int,
                 rot_base: float = 10000.0, rot_dims: int = 0, sink: bool = True) -> None:
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads, {kv_heads} key/value heads")
        if window < 1 or not scale > 0 or rot_dims > dim:
            raise ValueError(f"window {window}, scale {scale}, {rot_dims} rotated columns of {dim}")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.window, self.sink = float(scale), int(window), bool(sink)
        self.rotary = PairRotary(rot_base, rot_dims)
        self.query = nn.Linear(width, heads * dim, bias=False)
        self.key = nn.Linear(width, kv_heads * dim, bias=False)
        self.value = nn.Linear(width, kv_heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads * vdim, bias=False)
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("window", (self.kv_heads, up8(self.dim) + up8(self.vdim), self.window))

    def matrices(self):
        """Padded [q; k; v; gate] and output matrices."""
        H, G, dp = self.heads, self.kv_heads, up8(self.width)
        return (torch.cat([head_rows(m.weight, n, dp) for m, n in ((self.query, H), (self.key, G), (self.value, G), (self.gate, H))]),
                head_cols(self.out.weight, H, dp))

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            p.w_in, p.w_o = self.matrices()
        return Packed.of(self, list(self.parameters()), build)

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | k | v | gate]) -> gated heads (B*L, heads * padded vdim); the keys and values of the
        new tokens go to the ring."""
        H, G, dim, vdim = self.heads, self.kv_heads, up8(self.dim), up8(self.vdim)
        nk, gk, gv, nv = H * dim, G * dim, G * vdim, H * vdim
        ring, at = batch.ring(layer), dict(slots=batch.slots, start=batch.start)
        table = self.rotary.table(batch.max_keys, rows.device)
        q = rows[:, :nk].unflatten(0, (B, L)).unflatten(2, (H, dim)).transpose(1, 2)
        gate = rows[:, nk + gk + gv: nk + gk + gv + nv].unflatten(0, (B, L))
        out = torch.empty((B * L, nv), dtype=rows.dtype, device=rows.device) if out is None else out
        new = (rows, B, L, G, dim, vdim, nk, nk + gk)
        past = min(self.window - 1, batch.past)
        if past == 0:
            ops.window_rows(*new, rotary=table, ring=ring, count=batch.count, **at)
            k = rows[:, nk: nk + gk].unflatten(0, (B, L)).unflatten(2, (G, dim)).transpose(1, 2)
            v = rows[:, nk + gk: nk + gk + gv].unflatten(0, (B, L)).unflatten(2, (G, vdim)).transpose(1, 2)
        else:
            if table is not None:
                ops.window_rows(*new, rotary=table, **at)
            ctx = ops.window_context(*new, ring, past, **at)
            ops.window_rows(*new, ring=ring, count=batch.count, **at)   # (after its old rows were read)
            k, v = ctx[..., :dim], ctx[..., dim:]
        ops.attention_ex(q, k, v, self.scale, gate=gate, window=self.window, sink=self.sink, rotary=table, start_cap=past,
                         out=out.unflatten(0, (B, L)), **at)
        return out

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        """h (B*L, padded width) of the new tokens -> mixer output (B*L, padded width)."""
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
