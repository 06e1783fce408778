"""Zero padding of weights to the sizes the kernels step in."""
from __future__ import annotations

import torch


def round_up(n: int, multiple: int) -> int:
    return -(-n // multiple) * multiple


def pad_to(t: torch.Tensor, rows: int | None, columns: int | None) -> torch.Tensor:
    """A matrix with zero rows and columns behind its own (None: as many as it has)."""
    rows, columns = t.shape[0] if rows is None else rows, t.shape[1] if columns is None else columns
    if (rows, columns) == tuple(t.shape):
        return t.contiguous()
    out = t.new_zeros(rows, columns)
    out[:t.shape[0], :t.shape[1]] = t
    return out


def pad_heads(t: torch.Tensor, heads: int, size: int, columns: int | None = None) -> torch.Tensor:
    """(heads * n, K) -> (heads * size, columns): zero rows behind every head's own, zero columns behind all."""
    n, k = t.shape[0] // heads, t.shape[1]
    columns = k if columns is None else columns
    out = t.new_zeros(heads, size, columns)
    out[:, :n, :k] = t.view(heads, n, k)
    return out.view(heads * size, columns)
