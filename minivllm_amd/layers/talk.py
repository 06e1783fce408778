"""Operators of attention whose heads' scores are mixed before the softmax.

Queries carry the score scale and log2 e; everything else is in natural units.  All of it calls libminivllm_amd.so on the
current torch stream."""
from __future__ import annotations

import torch

from minivllm_amd import _C
from minivllm_amd.layers.fused import _check, _ptr
from minivllm_amd.layers.window import _floats, _heads

__all__ = ["talk_head_size", "talk_prefill", "talk_decode", "talk_decode_workspace_bytes"]


def talk_head_size(*sizes: int) -> int:
    """Head size the kernels run at for keys and values of these sizes (zeros fill them up)."""
    need = max(sizes)
    return next((d for d in (32, 64, 96, 128) if d >= need), -(-need // 8) * 8)


def _common(out, q, k, v, talk, sinks):
    rows, heads, dim = q.shape
    _check(q, q.dtype, (rows, heads, dim), "q")
    for name, t in (("k", k), ("v", v)):
        _check(t, q.dtype, (*k.shape[:-1], dim), name)
    _check(talk, torch.float32, (heads, heads), "talk")
    _floats("sinks", sinks, heads)
    return rows, heads, dim, k.shape[-2], _heads("out", out, q, 1 if rows else 0, heads, dim)


def talk_prefill(out: torch.Tensor, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, talk: torch.Tensor, cu_q: torch.Tensor,
                 cu_k: torch.Tensor | None = None, block_tables: torch.Tensor | None = None, sinks: torch.Tensor | None = None,
                 out_rows: torch.Tensor | None = None) -> None:
    """Pieces of packed queries q (T, H, dim) over keys and values: packed (K, G, dim), or with ``block_tables`` int32 (pieces,
    width) caches (blocks, block_size, G, dim).  A piece has cu_k keys, its queries are the last of them (``cu_k`` None: as many
    as queries, packed).  ``talk`` float32 (H, H): row h holds what every head's scores count in head h's; ``sinks`` float32
    (H,); row t of the result goes to row ``out_rows[t]`` int32 of out (*, H, >= dim)."""
    _C.require_cuda(out, q, k, v, talk, cu_q, cu_k, block_tables, sinks, out_rows)
    rows, heads, dim, groups, strides = _common(out, q, k, v, talk, sinks)
    paged = block_tables is not None
    if k.dim() != (4 if paged else 3) or (paged and cu_k is None):
        raise ValueError("packed keys (K, G, dim), or block_tables, cu_k and caches (blocks, block_size, G, dim)")
    for name, t in (("cu_q", cu_q), ("cu_k", cu_k)):
        if t is not None and (t.dtype != torch.int32 or t.numel() != cu_q.numel() or not t.is_contiguous()):
            raise ValueError(f"{name} must be contiguous int32, all of one length")
    if paged and (block_tables.dtype != torch.int32 or block_tables.dim() != 2 or block_tables.shape[0] < cu_q.numel() - 1 or not block_tables.is_contiguous()):
        raise ValueError("block_tables must be contiguous int32 (pieces, width)")
    if out_rows is not None:
        _check(out_rows, torch.int32, (rows,), "out_rows")
    elif out.shape[0] < rows:
        raise ValueError("out has fewer rows than q")
    st = _C.load().mvllm_talk_prefill(
        _ptr(out), *strides, _ptr(out_rows), _ptr(q), _ptr(k), _ptr(v), _ptr(cu_q), _ptr(cu_k), _ptr(block_tables),
        block_tables.shape[1] if paged else 0, k.shape[1] if paged else 0, k.shape[0] if paged else 0, _ptr(talk), _ptr(sinks),
        cu_q.numel() - 1, rows, heads, groups, dim, _C.dtype_code(q.dtype), _C.current_stream_ptr(q.device))
    _C.check(st, "talk_prefill")


def talk_decode_workspace_bytes(rows: int, num_heads: int, num_kv_heads: int, dim: int, max_keys: int, dtype: torch.dtype) -> int:
    return int(_C.load().mvllm_talk_decode_workspace_bytes(rows, num_heads, num_kv_heads, dim, max_keys, _C.dtype_code(dtype)))


def talk_decode(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor,
                lens: torch.Tensor, talk: torch.Tensor, sinks: torch.Tensor | None = None,
                workspace: torch.Tensor | None = None) -> None:
    """Single query rows q (rows, H, dim) over the first ``lens`` int64 (rows,) tokens of a row's ``block_tables`` int32
    (rows, width); everything else as in ``talk_prefill``."""
    _C.require_cuda(out, q, k_cache, v_cache, block_tables, lens, talk, sinks, workspace)
    rows, heads, dim, groups, strides = _common(out, q, k_cache, v_cache, talk, sinks)
    if k_cache.dim() != 4 or out.shape[0] < rows:
        raise ValueError("caches must be (blocks, block_size, G, dim), out must have a row per query")
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or block_tables.shape[0] < rows or not block_tables.is_contiguous():
        raise ValueError("block_tables must be contiguous int32 (rows, width)")
    _check(lens, torch.int64, (rows,), "lens")
    need = talk_decode_workspace_bytes(rows, heads, groups, dim, block_tables.shape[1] * k_cache.shape[1], q.dtype)
    if need and (workspace is None or workspace.numel() < need):
        workspace = torch.empty(need, dtype=torch.uint8, device=q.device)
    st = _C.load().mvllm_talk_decode(
        _ptr(out), *strides, _ptr(q), _ptr(k_cache), _ptr(v_cache), _ptr(block_tables), block_tables.shape[1], _ptr(lens), _ptr(talk),
        _ptr(sinks), rows, heads, groups, dim, k_cache.shape[1], k_cache.shape[0], _C.dtype_code(q.dtype), _ptr(workspace),
        0 if workspace is None else workspace.numel(), _C.current_stream_ptr(q.device))
    _C.check(st, "talk_decode")
