"""Norms with a weight and no bias, applied in fp32 by vy_residual_norm / vy_latent_norm / vy_rmsnorm_gate.  The module
holds the weight; the kernels fuse the norm with what surrounds it (the residual sum, a projection's split, a gate)."""
from __future__ import annotations

import torch
import torch.nn as nn


class WeightNorm(nn.Module):
    """kind 'layer': (x - mean) / sqrt(var + eps) * w; kind 'rms': x / sqrt(mean(x^2) + eps) * w.  offset: the factor is
    offset + w (1 for weights that are stored around zero).  scalar: one number for all coordinates."""

    def __init__(self, width: int, eps: float, kind: str = "layer", offset: float = 0.0, scalar: bool = False) -> None:
        super().__init__()
        if kind not in ("layer", "rms"):
            raise ValueError(f"norm kind {kind!r}")
        self.weight = nn.Parameter(torch.full(() if scalar else (width,), 1.0 - offset))
        self.width, self.eps, self.kind, self.offset = width, float(eps), kind, float(offset)
