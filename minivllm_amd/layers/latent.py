"""Operators of attention over latents: one cached row per token that every head's keys and values are made of.

All of it calls libminivllm_amd.so on the current torch stream."""
from __future__ import annotations

import torch

from minivllm_amd import _C

__all__ = ["latent_width", "latent_norm_store", "head_linear", "latent_decode", "latent_decode_workspace_bytes"]

_TILED = (32, 64, 96, 128, 192, 256, 384, 512)      # widths the bf16 decode kernel is built for


def _ptr(t):
    return 0 if t is None else t.data_ptr()


def latent_width(rank: int) -> int:
    """Width of a cached row: the rank, filled up with zeros to the next width with a tiled kernel (or multiple of 32)."""
    if rank > 2048:
        raise ValueError(f"latents of {rank} numbers: at most 2048")
    return next((w for w in _TILED if w >= rank), -(-rank // 32) * 32)


def latent_norm_store(rows: torch.Tensor, weight: torch.Tensor, eps: float, cache: torch.Tensor | None = None,
                      slots: torch.Tensor | None = None, need_rows: bool = True) -> torch.Tensor | None:
    """c = rms(row) * weight for ``rows`` (T, padded; the first ``weight.numel()`` columns count), into ``cache``
    (blocks, block_size, padded) at ``slots`` int64 (T,) (-1: not) and, with ``need_rows``, as a packed (T, padded) tensor."""
    _C.require_cuda(rows, weight, cache, slots)
    t, padded = rows.shape
    rank = weight.numel()
    if rows.stride(1) != 1 or weight.dtype != torch.float32 or not weight.is_contiguous() or rank > padded:
        raise ValueError("rows must be dense and the weight contiguous float32 of at most their width")
    if cache is not None:
        if cache.dtype != rows.dtype or cache.dim() != 3 or cache.shape[2] != padded or not cache.is_contiguous():
            raise ValueError(f"cache must be contiguous (blocks, block_size, {padded}) in the rows' dtype")
        if slots is None or slots.dtype != torch.int64 or slots.numel() != t or not slots.is_contiguous():
            raise ValueError("slots must be contiguous int64, one per row")
    out = torch.empty((t, padded), dtype=rows.dtype, device=rows.device) if need_rows else None
    st = _C.load().mvllm_latent_norm_store(
        _ptr(out), _ptr(rows), rows.stride(0) if t > 1 else padded, _ptr(weight), float(eps), _ptr(cache),
        0 if cache is None else cache.shape[0] * cache.shape[1], _ptr(slots if cache is not None else None), t, rank, padded,
        _C.dtype_code(rows.dtype), _C.current_stream_ptr(rows.device))
    _C.check(st, "latent_norm_store")
    return out


def head_linear(x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """out[t, h] = W_h x[t, h]: x (T, H, K) and out (T, H, N) with dense last dimensions, weight (H, N, K) contiguous."""
    _C.require_cuda(x, weight, out)
    t, heads, k = x.shape
    if weight.dim() != 3 or weight.shape[0] != heads or weight.shape[2] != k or weight.dtype != x.dtype or not weight.is_contiguous():
        raise ValueError(f"weight must be contiguous ({heads}, N, {k}) in x's dtype, got {tuple(weight.shape)}")
    n = weight.shape[1]
    if out is None:
        out = torch.empty((t, heads, n), dtype=x.dtype, device=x.device)
    if tuple(out.shape) != (t, heads, n) or out.dtype != x.dtype or out.stride(2) != 1 or x.stride(2) != 1:
        raise ValueError("x and out must have dense rows and out the product's shape")
    st = _C.load().mvllm_head_linear(
        _ptr(out), out.stride(0), out.stride(1) if heads > 1 else n, _ptr(x), x.stride(0) if t > 1 else heads * k,
        x.stride(1) if heads > 1 else k, _ptr(weight), t, heads, n, k, _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "head_linear")
    return out


def latent_decode_workspace_bytes(rows: int, num_heads: int, padded: int, max_keys: int, dtype: torch.dtype) -> int:
    return int(_C.load().mvllm_latent_decode_workspace_bytes(rows, num_heads, padded, max_keys, _C.dtype_code(dtype)))


def latent_decode(q: torch.Tensor, cache: torch.Tensor, block_tables: torch.Tensor, row_entry: torch.Tensor, lens: torch.Tensor,
                  scale: float, workspace: torch.Tensor | None = None) -> torch.Tensor:
    """softmax(scale q . c) c per (row, head) over the first ``lens[row]`` latents of entry ``row_entry[row]``.

    q (rows, H, padded), cache (blocks, block_size, padded), block_tables int32 (entries, width), row_entry int32 (>= rows,),
    lens int64 (rows,).  ``workspace``: a caller-owned uint8 tensor, used if it is large enough."""
    _C.require_cuda(q, cache, block_tables, row_entry, lens, workspace)
    rows, heads, padded = q.shape
    if not q.is_contiguous() or cache.dim() != 3 or cache.shape[2] != padded or cache.dtype != q.dtype or not cache.is_contiguous():
        raise ValueError(f"q must be contiguous and the cache contiguous (blocks, block_size, {padded}) in its dtype")
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or not block_tables.is_contiguous():
        raise ValueError("block_tables must be contiguous int32 (entries, width)")
    if row_entry.dtype != torch.int32 or row_entry.numel() < rows or lens.dtype != torch.int64 or lens.numel() != rows \
            or not row_entry.is_contiguous() or not lens.is_contiguous():
        raise ValueError("row_entry must be int32 and lens int64, one per row")
    out = torch.empty_like(q)
    width, block_size = block_tables.shape[1], cache.shape[1]
    need = latent_decode_workspace_bytes(rows, heads, padded, width * block_size, q.dtype)
    if need and (workspace is None or workspace.numel() < need):
        workspace = torch.empty(need, dtype=torch.uint8, device=q.device)
    st = _C.load().mvllm_latent_decode(
        _ptr(out), _ptr(q), _ptr(cache), _ptr(block_tables), width, _ptr(row_entry), _ptr(lens), rows, heads, padded,
        block_size, cache.shape[0], float(scale), _C.dtype_code(q.dtype), _ptr(workspace),
        0 if workspace is None else workspace.numel(), _C.current_stream_ptr(q.device))
    _C.check(st, "latent_decode")
    return out
