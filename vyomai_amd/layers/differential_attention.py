"""Differential attention: every head attends twice, with two maps of queries and keys over the same values, and hands on the
difference of the two outputs, a1 - lambda a2, divided by its root mean square and multiplied by 1 - diff.  lambda is one number
of the layer, made from four vectors and `diff`.  Grouped query heads, biases on the projections, RMS norms over the columns of
every head and map, no positions but a temperature on the queries that grows with the logarithm of their position; every earlier
token is seen.

Prefill norms queries and keys in place in the packed projection rows and puts keys and values where they stay (vy_qkv_rows);
vy_diff_attn_fwd reads them there.  Decode is vy_window_decode over the same rows.
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from .._lib import VyDiff
from ..ops import up8
from .kv_cache import EVERY_TOKEN
from .norms import WeightNorm
from .packing import Packed, head_bias, head_cols, head_rows, pad_vec


class DifferentialAttention(nn.Module):
    kind = "differential"

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, diff: float, eps: float,
                 temp_coef: float = 0.0, temp_every: int = 0) -> None:
        """dim: columns of one map's query or key.  temp_every 0: no temperature."""
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads, {kv_heads} key/value heads")
        if not scale > 0 or temp_every < 0 or int(temp_every) != temp_every:
            raise ValueError(f"scale {scale}, a temperature that grows every {temp_every} tokens")
        self.width, self.heads, self.kv_heads, self.dim, self.vdim = width, heads, kv_heads, dim, vdim
        self.scale, self.diff, self.eps = float(scale), float(diff), float(eps)
        self.temp_coef, self.temp_every = float(temp_coef), int(temp_every)
        self.query = nn.Linear(width, heads * 2 * dim)
        self.key = nn.Linear(width, kv_heads * 2 * dim)
        self.value = nn.Linear(width, kv_heads * vdim)
        self.q_norm, self.k_norm = WeightNorm(dim, eps, "rms"), WeightNorm(dim, eps, "rms")
        for n in ("lq1", "lk1", "lq2", "lk2"):
            setattr(self, n, nn.Parameter(torch.zeros(dim)))
        self.out = nn.Linear(heads * vdim, width, bias=False)

    def cache_spec(self):
        return ("window", (self.kv_heads, 2 * up8(self.dim) + up8(self.vdim), EVERY_TOKEN))

    def constants(self) -> Packed:
        """prep: what vy_qkv_rows and a decode step do to queries and keys; diff: the difference and the norm behind it."""
        def build(p: Packed) -> None:
            w = [pad_vec(n.weight, up8(self.dim)) for n in (self.q_norm, self.k_norm)]
            p.prep = ops.QkvPrep(w[0].repeat(2 * self.heads), w[1].repeat(2 * self.kv_heads), self.dim, self.dim, self.eps,
                                 n_v=self.vdim, group=up8(self.dim), temp_every=self.temp_every, temp_coef=self.temp_coef)
            dots = [float((a.double() * b.double()).sum().exp()) for a, b in ((self.lq1, self.lk1), (self.lq2, self.lk2))]
            p.diff = VyDiff(dots[0] - dots[1] + self.diff, 1.0 - self.diff, self.eps, self.vdim)
        return Packed.of(self, [self.q_norm.weight, self.k_norm.weight, self.lq1, self.lk1, self.lq2, self.lk2], build, "_constants")

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            dp, parts = up8(self.width), ((self.query, 2 * self.heads), (self.key, 2 * self.kv_heads), (self.value, self.kv_heads))
            p.w_in = torch.cat([head_rows(m.weight, n, dp) for m, n in parts]).contiguous()
            p.b_in = torch.cat([head_bias(m.bias, n) for m, n in parts]).contiguous()
            p.w_o = head_cols(self.out.weight, self.heads, dp)
        return Packed.of(self, [p for n, p in self.named_parameters() if n.split(".")[0] in ("query", "key", "value", "out")], build)

    def mix(self, rows: torch.Tensor, B: int, L: int, batch, layer: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Packed projections (B*L, [q | k | v]) -> heads (B*L, heads * padded vdim); keys and values go to the cache."""
        c, ring = self.constants(), batch.ring(layer)
        H, G, dim, vdim = self.heads, self.kv_heads, 2 * up8(self.dim), up8(self.vdim)
        at = dict(slots=batch.slots, start=batch.start, count=batch.count)
        ops.qkv_rows(rows, B, L, H, G, dim, vdim, 0, H * dim, (H + G) * dim, c.prep, ring=ring, **at)
        return ops.diff_attention(rows, B, L, H, G, dim, vdim, ring, self.scale, c.diff, out=out, **at)

    def forward(self, h: torch.Tensor, B: int, L: int, batch, layer: int) -> torch.Tensor:
        """h (B*L, padded width) of the new tokens -> mixer output (B*L, padded width)."""
        p = self.packed()
        return ops.linear(self.mix(ops.linear(h, p.w_in, p.b_in), B, L, batch, layer), p.w_o)
