"""Sliding-window attention: grouped query heads (values may have a width of their own) and rotary positions on neighbouring
columns.  Query i sees the last `window` tokens up to itself and the `keep_first` first ones of its sequence, so a sequence's
memory is a ring of keep_first + window rows per key/value head.  Optional: a sink (one added to every softmax denominator), a
sigmoid gate on the output, RMS norms over the whole query and the whole key projection (before the rotation), and values mixed
with those of the first such layer.

Prefill makes queries, keys and values in place in the packed projection rows (vy_qkv_rows) and runs the flash kernel; without
norms and mixing only the keys are touched (the queries' rotation is the flash kernel's own).  Behind a past the ring's rows and
the new ones form the context.  Decode is vy_window_decode.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops import up8
from .norms import WeightNorm
from .packing import Packed, head_cols, head_rows, head_vec
from .positional_embeddings import PairRotary

VALUES_OWN, VALUES_FIRST, VALUES_MIX = 0, 1, 2   # VY_VALUES_*: a layer's values: its own; its own, kept for later layers; mixed


class WindowAttention(nn.Module):
    kind = "window"

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, window: int,
                 rot_base: float = 10000.0, rot_dims: int = 0, sink: bool = True, gate: bool = True, keep_first: int = 0,
                 rot_scaling: Optional[Dict[str, float]] = None, qk_norm_eps: Optional[float] = None,
                 values: int = VALUES_OWN) -> None:
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads, {kv_heads} key/value heads")
        if window < 1 or keep_first < 0 or not scale > 0 or rot_dims > dim:
            raise ValueError(f"window {window}, {keep_first} kept tokens, scale {scale}, {rot_dims} rotated columns of {dim}")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.window, self.keep_first, self.sink = float(scale), int(window), int(keep_first), bool(sink)
        self.values = values
        self.rotary = PairRotary(rot_base, rot_dims, rot_scaling)
        self.query = nn.Linear(width, heads * dim, bias=False)
        self.key = nn.Linear(width, kv_heads * dim, bias=False)
        self.value = nn.Linear(width, kv_heads * vdim, bias=False)
        self.gate = nn.Linear(width, heads * vdim, bias=False) if gate else None
        self.q_norm = WeightNorm(heads * dim, qk_norm_eps, "rms") if qk_norm_eps is not None else None
        self.k_norm = WeightNorm(kv_heads * dim, qk_norm_eps, "rms") if qk_norm_eps is not None else None
        if values != VALUES_OWN:
            self.value_mix = nn.Parameter(torch.zeros(()))   # share of the first layer's values
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("window", (self.kv_heads, up8(self.dim) + up8(self.vdim), self.keep_first + self.window, self.keep_first))

    def matrices(self):
        """Padded [q; k; v; gate] and output matrices."""
        H, G, dp = self.heads, self.kv_heads, up8(self.width)
        parts = [(self.query, H), (self.key, G), (self.value, G)] + ([(self.gate, H)] if self.gate is not None else [])
        return torch.cat([head_rows(m.weight, n, dp) for m, n in parts]), head_cols(self.out.weight, H, dp)

    @property
    def prepares(self) -> bool:
        """Whether queries, keys or values need more than the keys' rotation ahead of attention."""
        return self.q_norm is not None or self.values != VALUES_OWN

    def constants(self) -> Packed:
        """What a decode step or vy_qkv_rows needs besides the matrices: an ops.QkvPrep without its rows (None: nothing)."""
        params = [p for n, p in self.named_parameters() if n in ("q_norm.weight", "k_norm.weight", "value_mix")]

        def build(p: Packed) -> None:
            p.prep = None
            if self.prepares:
                n = self.q_norm is not None
                p.prep = ops.QkvPrep(head_vec(self.q_norm.weight, self.heads) if n else None,
                                     head_vec(self.k_norm.weight, self.kv_heads) if n else None, self.heads * self.dim,
                                     self.kv_heads * self.dim, self.q_norm.eps if n else 0.0,
                                     float(self.value_mix) if self.values == VALUES_MIX else 0.0, self.vdim)
        return Packed.of(self, params, build, "_constants")

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            p.w_in, p.w_o = (w.contiguous() for w in self.matrices())
        return Packed.of(self, list(self.parameters()), build)

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | k | v | gate]) -> (gated) heads (B*L, heads * padded vdim); the keys and values of the
        new tokens go to the ring."""
        H, G, dim, vdim = self.heads, self.kv_heads, up8(self.dim), up8(self.vdim)
        nk, gk, gv, nv = H * dim, G * dim, G * vdim, H * vdim
        ring, at, keep = batch.ring(layer), dict(slots=batch.slots, start=batch.start), self.keep_first
        table = self.rotary.table(batch.max_keys, rows.device)
        prep = self.constants().prep
        if self.values == VALUES_FIRST:
            batch.shared_values = rows[:, nk + gk: nk + gk + gv], self.vdim
        elif self.values == VALUES_MIX:
            prep = prep._replace(values=batch.shared_values[0], values_dim=batch.shared_values[1])
        q = rows[:, :nk].unflatten(0, (B, L)).unflatten(2, (H, dim)).transpose(1, 2)
        gate = rows[:, nk + gk + gv: nk + gk + gv + nv].unflatten(0, (B, L)) if self.gate is not None else None
        out = torch.empty((B * L, nv), dtype=rows.dtype, device=rows.device) if out is None else out
        new = (rows, B, L, G, dim, vdim, nk, nk + gk)
        past = min(keep + self.window - 1, batch.past)
        to_ring = dict(ring=ring, keep=keep, count=batch.count)
        if prep is not None:
            ops.qkv_rows(rows, B, L, H, G, dim, vdim, 0, nk, nk + gk, prep, rotary=table, **at, **(to_ring if past == 0 else {}))
        elif past == 0:
            ops.window_rows(*new, rotary=table, **to_ring, **at)
        elif table is not None:
            ops.window_rows(*new, rotary=table, **at)
        if past == 0:
            k = rows[:, nk: nk + gk].unflatten(0, (B, L)).unflatten(2, (G, dim)).transpose(1, 2)
            v = rows[:, nk + gk: nk + gk + gv].unflatten(0, (B, L)).unflatten(2, (G, vdim)).transpose(1, 2)
        else:
            ctx = ops.window_context(*new, ring, past, keep=keep, **at)
            ops.window_rows(*new, **to_ring, **at)   # (after its old rows were read)
            k, v = ctx[..., :dim], ctx[..., dim:]
        ops.attention_ex(q, k, v, self.scale, gate=gate, window=self.window, keep=keep, sink=self.sink,
                         rotary=table if prep is None else None, start_cap=past, out=out.unflatten(0, (B, L)), **at)
        return out

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        """h (B*L, padded width) of the new tokens -> mixer output (B*L, padded width)."""
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in), B, L, batch, layer), p.w_o)
