"""Kernel-side copies of weights: padded to multiples of 8 elements (zero padding, so the products are unchanged), sibling
projections stacked into one matrix.  Built once per parameter version and kept beside the module."""
from __future__ import annotations

from typing import Callable, Sequence

import torch
import torch.nn as nn

from ..ops import up8


def pad2(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    """w (r, c) in the upper left corner of a (rows, cols) matrix of zeros."""
    if tuple(w.shape) == (rows, cols):
        return w
    out = torch.zeros(rows, cols, dtype=w.dtype, device=w.device)
    out[: w.shape[0], : w.shape[1]] = w
    return out


def pad_vec(w: torch.Tensor, n: int) -> torch.Tensor:
    """fp32 copy of a norm weight, zero-padded to n."""
    out = torch.zeros(n, dtype=torch.float32, device=w.device)
    out[: w.numel()] = w.float()
    return out


def norm_vec(norm, n: int, mult: float = 1.0) -> torch.Tensor:
    """fp32 factors of a WeightNorm (times mult), zero-padded to n."""
    return pad_vec(((norm.weight.float() + norm.offset) * mult).expand(norm.width), n)


def head_rows(w: torch.Tensor, heads: int, cols: int) -> torch.Tensor:
    """(heads * dim, k <= cols) -> (heads * up8(dim), cols): every head's rows padded by themselves."""
    dim = w.shape[0] // heads
    out = torch.zeros(heads, up8(dim), cols, dtype=w.dtype, device=w.device)
    out[:, :dim, : w.shape[1]] = w.view(heads, dim, w.shape[1])
    return out.view(heads * up8(dim), cols)


def head_cols(w: torch.Tensor, heads: int, rows: int) -> torch.Tensor:
    """(n, heads * dim) -> (rows, heads * up8(dim))."""
    dim = w.shape[1] // heads
    out = torch.zeros(rows, heads, up8(dim), dtype=w.dtype, device=w.device)
    out[: w.shape[0], :, :dim] = w.view(w.shape[0], heads, dim)
    return out.view(rows, heads * up8(dim))


def halves_to_pairs(w: torch.Tensor, heads: int, dims: int) -> torch.Tensor:
    """Rows of every head put in another order: row i and row i + dims / 2 of its first `dims` become neighbours (2i, 2i + 1).
    Queries and keys whose rotary pairs are halves apart run on kernels that rotate neighbours: dot products do not see it."""
    dim, half = w.shape[0] // heads, dims // 2
    order = [c for i in range(half) for c in (i, i + half)] + list(range(dims, dim))
    return w.view(heads, dim, *w.shape[1:])[:, order].reshape(w.shape)


def head_vec(w: torch.Tensor, heads: int) -> torch.Tensor:
    """fp32 copy of a norm weight over concatenated heads, every head padded by itself."""
    dim = w.numel() // heads
    out = torch.zeros(heads, up8(dim), dtype=torch.float32, device=w.device)
    out[:, :dim] = w.float().view(heads, dim)
    return out.view(-1)


def head_bias(b: torch.Tensor, heads: int) -> torch.Tensor:
    """A bias over concatenated heads in its own type, every head padded by itself (as head_rows pads the weights)."""
    return head_rows(b[:, None], heads, 1)[:, 0]


class Packed:
    """Attribute bag of a module's kernel-side tensors, rebuilt when one of its parameters changed.  (A build may turn a
    parameter into a view of its packed copy: the parameters' state is noted after it.)"""

    @staticmethod
    def of(owner: nn.Module, params: Sequence[torch.Tensor], build: Callable[["Packed"], None], name: str = "_packed_cache") -> "Packed":
        def state():
            return tuple((p.data_ptr(), p._version, p.dtype) for p in params)
        key = state()
        hit = owner.__dict__.get(name)
        if hit is None or hit.key != key:
            hit = Packed()
            with torch.no_grad():
                build(hit)
            hit.key = state()
            owner.__dict__[name] = hit
        return hit
