"""Operators of windowed attention whose cached rows are keys and values at once, make both, or hold both side by side.

All of it calls libminivllm_amd.so on the current torch stream; tensors are read and written where projections leave and take
them (dense rows, any row stride)."""
from __future__ import annotations

import torch

from minivllm_amd import _C

__all__ = ["head_size", "shared_part_size", "latent_layout", "copy_rows", "head_rope", "latent_rope_store", "window_prefill",
           "window_decode", "window_decode_workspace_bytes"]

_HEADS = (32, 64, 96, 128, 192, 256)                     # head sizes of the tiled prefill kernels
_WIDTHS = (32, 64, 96, 128, 192, 256, 384, 512)          # widths of a cached row with a tiled decode kernel


def head_size(*sizes: int) -> int:
    """Head size the kernels run at for keys and values of these sizes (zeros fill them up)."""
    need = max(sizes)
    if need > 512:
        raise ValueError(f"heads of {need}: at most 512")
    return next((d for d in _HEADS if d >= need), -(-need // 32) * 32)


def shared_part_size(rot: int) -> int:
    """The same for the part of the keys that all heads share."""
    return 32 if rot <= 32 else 64 if rot <= 64 else -(-rot // 32) * 32


def latent_layout(rank: int, rot: int) -> tuple[int, int, int]:
    """(column of the rotated part, width of a cached row, its columns that count as values) for a latent and its rotated part."""
    at = -(-rank // 16) * 16
    need = at + shared_part_size(rot)
    if need > 2048:
        raise ValueError(f"latents of {rank} + {rot} numbers: at most 2048 together")
    width = next((w for w in _WIDTHS if w >= need), None)
    if width is None and need <= 576 and at <= 512:
        return at, 576, 512
    width = width or -(-need // 32) * 32
    return at, width, width


def _ptr(t):
    return 0 if t is None else t.data_ptr()


def _stride(t, dim, dense):
    """Stride of a dimension, as if it were dense where it has one element."""
    return t.stride(dim) if t.shape[dim] > 1 else dense


def _index(t, rows, name):
    if t is not None and (t.dtype != torch.int64 or t.numel() < rows or not t.is_contiguous()):
        raise ValueError(f"{name} must be contiguous int64, one per row")


def copy_rows(src: torch.Tensor, dst: torch.Tensor | None, dst_rows: torch.Tensor | None = None,
              src_rows: torch.Tensor | None = None, dst2: torch.Tensor | None = None, dst2_rows: torch.Tensor | None = None) -> None:
    """dst[dst_rows[t]] = src[src_rows[t]], and the same into dst2; negative indices are skipped, no indices: row t."""
    _C.require_cuda(src, dst, dst_rows, src_rows, dst2, dst2_rows)
    width = src.shape[1]
    rows = src.shape[0] if src_rows is None else src_rows.numel()
    for name, t, index in (("dst", dst, dst_rows), ("dst2", dst2, dst2_rows)):
        if t is None:
            continue
        if t.dtype != src.dtype or t.dim() != 2 or t.shape[1] != width or t.stride(1) != 1:
            raise ValueError(f"{name} must be (*, {width}) in src's dtype with dense rows")
        if index is None and t.shape[0] < rows:
            raise ValueError(f"{name} has fewer rows than are copied")
        _index(index, rows, name + "_rows")
    if src.stride(1) != 1:
        raise ValueError("src must have dense rows")
    of = lambda t: (0, 0, 0) if t is None else (_ptr(t), _stride(t, 0, width), t.shape[0])
    st = _C.load().mvllm_copy_rows(*of(dst), _ptr(dst_rows), *of(dst2), _ptr(dst2_rows), *of(src), _ptr(src_rows), rows, width,
                                   _C.dtype_code(src.dtype), _C.current_stream_ptr(src.device))
    _C.check(st, "copy_rows")


def head_rope(x: torch.Tensor, column: int, rot: int, table: torch.Tensor, positions: torch.Tensor, interleaved: bool,
              first_out: torch.Tensor | None = None, out_column: int = 0, first_rows: int = 0) -> None:
    """Turns columns ``column`` .. + ``rot`` of every head of x (T, H, d) by ``table`` float32 (max_position, dims / 2, 2), in place;
    the first ``first_rows`` rows go to ``first_out`` (>= first_rows, H, w) from ``out_column`` on, with zeros up to w."""
    _C.require_cuda(x, table, positions, first_out)
    t, heads, d = x.shape
    if x.stride(2) != 1 or table.dtype != torch.float32 or table.dim() != 3 or not table.is_contiguous() or table.shape[2] != 2 \
            or column + rot > d or 2 * table.shape[1] > rot:
        raise ValueError("x must have dense heads with the part inside, table float32 (max_position, <= rot / 2, 2)")
    _index(positions, t, "positions")
    out_row = out_head = width = 0
    if first_rows:
        if first_out.shape[0] < first_rows or first_out.shape[1] != heads or first_out.dtype != x.dtype or first_out.stride(2) != 1:
            raise ValueError("first_out must have the first rows' heads in x's dtype")
        out_head = _stride(first_out, 1, first_out.shape[2])
        out_row, width = _stride(first_out, 0, heads * first_out.shape[2]), first_out.shape[2] - out_column
    st = _C.load().mvllm_head_rope(_ptr(x), _stride(x, 0, heads * d), _stride(x, 1, d), column, _ptr(first_out), out_row, out_head,
                                   out_column, width, first_rows, _ptr(table), rot, 2 * table.shape[1], int(interleaved),
                                   table.shape[0], _ptr(positions), t, heads, _C.dtype_code(x.dtype), _C.current_stream_ptr(x.device))
    _C.check(st, "head_rope")


def latent_rope_store(rows: torch.Tensor, weight: torch.Tensor, eps: float, rot_column: int, rot: int, table: torch.Tensor,
                      positions: torch.Tensor, interleaved: bool, cache: torch.Tensor | None, slots: torch.Tensor | None,
                      out: torch.Tensor | None = None, out_rows: torch.Tensor | None = None, rows2: torch.Tensor | None = None,
                      weight2: torch.Tensor | None = None) -> torch.Tensor | None:
    """[rms(latent) * weight | rotated part] of ``rows`` (T, width: latent at 0, rotated part at ``rot_column``) into ``cache``
    (blocks, block_size, width) at ``slots`` and into rows ``out_rows`` of ``out`` (*, width).  ``rows2`` (T, width2): returns
    rms(rows2[:, :weight2.numel()]) * weight2 from the same launch."""
    _C.require_cuda(rows, weight, table, positions, cache, slots, out, out_rows, rows2, weight2)
    t, width = rows.shape
    for name, r, w in (("rows", rows, weight), ("rows2", rows2, weight2)):
        if r is not None and (r.shape[0] != t or r.stride(1) != 1 or r.dtype != rows.dtype or w.dtype != torch.float32
                              or not w.is_contiguous() or w.numel() > r.shape[1]):
            raise ValueError(f"{name} must be dense rows of one dtype, its weight contiguous float32 of at most their width")
    if table.dtype != torch.float32 or table.dim() != 3 or table.shape[2] != 2 or not table.is_contiguous():
        raise ValueError("table must be contiguous float32 (max_position, dims / 2, 2)")
    _index(positions, t, "positions")
    _index(slots, t, "slots")
    _index(out_rows, t, "out_rows")
    if cache is not None and (cache.dtype != rows.dtype or cache.dim() != 3 or cache.shape[2] != width or not cache.is_contiguous() or slots is None):
        raise ValueError(f"cache must be contiguous (blocks, block_size, {width}) in the rows' dtype, with slots")
    if out is not None and (out.dtype != rows.dtype or out.shape[1] != width or not out.is_contiguous() or (out_rows is None and out.shape[0] < t)):
        raise ValueError(f"out must be contiguous (*, {width}) in the rows' dtype")
    out2 = None if rows2 is None else torch.empty((t, rows2.shape[1]), dtype=rows.dtype, device=rows.device)
    st = _C.load().mvllm_latent_rope_store(
        _ptr(out), _ptr(out_rows), _ptr(rows), _stride(rows, 0, width), _ptr(weight), float(eps), _ptr(table), rot_column, rot,
        2 * table.shape[1], int(interleaved), table.shape[0], _ptr(positions), _ptr(cache),
        0 if cache is None else cache.shape[0] * cache.shape[1], _ptr(slots), _ptr(out2), _ptr(rows2),
        0 if rows2 is None else _stride(rows2, 0, rows2.shape[1]), _ptr(weight2), 0 if weight2 is None else weight2.numel(),
        0 if rows2 is None else rows2.shape[1], t, weight.numel(), width, _C.dtype_code(rows.dtype), _C.current_stream_ptr(rows.device))
    _C.check(st, "latent_rope_store")
    return out2


def _heads(name, t, like, rows, heads, least):
    """(row stride, head stride) of a (rows, heads, >= least) tensor with dense heads; zeros for None."""
    if t is None:
        return 0, 0
    if t.dim() != 3 or t.shape[0] < rows or t.shape[1] != heads or t.shape[2] < least or t.stride(2) != 1 or t.dtype != like.dtype:
        raise ValueError(f"{name} must be ({rows}, {heads}, >= {least}) in {like.dtype} with dense heads, got {t.dtype} {tuple(t.shape)}")
    return _stride(t, 0, heads * t.shape[2]), _stride(t, 1, t.shape[2])


def _gate(t, like, rows, heads, least):
    """Strides of a gate: one number per column, or (rows, heads) one per head (head stride 1)."""
    if t is None or t.dim() == 3:
        return _heads("gate", t, like, rows, heads, least)
    if t.dim() != 2 or t.shape[0] < rows or t.shape[1] != heads or t.dtype != like.dtype or (heads > 1 and t.stride(1) != 1):
        raise ValueError(f"gate must be ({rows}, {heads}) in {like.dtype} with dense rows, got {t.dtype} {tuple(t.shape)}")
    return _stride(t, 0, heads), 1


def _floats(name, t, n):
    if t is not None and (t.dtype != torch.float32 or t.numel() != n or not t.is_contiguous()):
        raise ValueError(f"{name} must be contiguous float32 ({n},)")


def window_prefill(out: torch.Tensor, q: torch.Tensor, k: torch.Tensor, cu_q: torch.Tensor, cu_k: torch.Tensor, scale: float,
                   window: int, k2: torch.Tensor | None = None, v: torch.Tensor | None = None, gate: torch.Tensor | None = None,
                   slopes: torch.Tensor | None = None, positions: torch.Tensor | None = None, temperature: tuple = (0.0, 0)) -> None:
    """Entries of packed queries q (T, H, dim + rot) over packed keys k (K, G, dim), k2 (K, rot) shared by all heads, values v like k
    (None: the keys), into out (T, H, dim).  Query i of an entry stands at key (keys - queries) + i and sees ``window`` keys up to it
    (0: all); ``slopes`` times the distance is taken off a score, ``temperature`` = (coef, every) makes scores grow with
    ``positions``, ``gate`` (T, H, dim), or (T, H) for one number per head, multiplies the result with its sigmoid."""
    _C.require_cuda(out, q, k, cu_q, cu_k, k2, v, gate, slopes, positions)
    t, heads = q.shape[:2]
    keys, groups, dim = k.shape
    rot = 0 if k2 is None else k2.shape[1]
    if cu_q.dtype != torch.int32 or cu_k.dtype != torch.int32 or cu_q.numel() != cu_k.numel() or not cu_q.is_contiguous() or not cu_k.is_contiguous():
        raise ValueError("cu_q and cu_k must be contiguous int32 of one length")
    if k2 is not None and (k2.dim() != 2 or k2.shape[0] < keys or k2.stride(1) != 1 or k2.dtype != q.dtype):
        raise ValueError("k2 must be (keys, rot) in q's dtype with dense rows")
    _floats("slopes", slopes, heads)
    if temperature[1]:
        _index(positions, t, "positions")
    st = _C.load().mvllm_window_prefill(
        _ptr(out), *_heads("out", out, q, t, heads, dim), _ptr(q), *_heads("q", q, q, t, heads, dim + rot), _ptr(k),
        *_heads("k", k, q, keys, groups, dim), _ptr(k2), 0 if k2 is None else _stride(k2, 0, rot), _ptr(v),
        *_heads("v", v, q, keys, groups, dim), _ptr(gate), *_gate(gate, q, t, heads, dim), _ptr(cu_q), _ptr(cu_k),
        _ptr(positions), _ptr(slopes), cu_q.numel() - 1, t, heads, groups, dim, rot, int(window), float(scale),
        float(temperature[0]), float(temperature[1]), _C.dtype_code(q.dtype), _C.current_stream_ptr(q.device))
    _C.check(st, "window_prefill")


def window_decode_workspace_bytes(rows: int, num_heads: int, num_kv_heads: int, width: int, values: int, max_keys: int,
                                  dtype: torch.dtype) -> int:
    return int(_C.load().mvllm_window_decode_workspace_bytes(rows, num_heads, num_kv_heads, width, values, max_keys, _C.dtype_code(dtype)))


def window_decode(out: torch.Tensor, q: torch.Tensor, cache: torch.Tensor, block_tables: torch.Tensor, row_entry: torch.Tensor,
                  lens: torch.Tensor, scale: float, window: int, ring: int, gate: torch.Tensor | None = None,
                  slopes: torch.Tensor | None = None, temperature: tuple = (0.0, 0), workspace: torch.Tensor | None = None) -> None:
    """Single query rows q (rows, H, width) over ``cache`` (blocks, block_size, G, width), whose rows are keys and, in their first
    columns, values: out (rows, H, width, or 512 of 576).  Cached rows wider than q hold a value of out's width behind the key.
    ``lens`` int64 (rows,): position + 1; ``ring``: token p lies at place
    p mod ring of row ``row_entry[row]`` of ``block_tables`` (0: at place p).  Everything else as in ``window_prefill``."""
    _C.require_cuda(out, q, cache, block_tables, row_entry, lens, gate, slopes, workspace)
    rows, heads, width = q.shape
    split = cache.dim() == 4 and cache.shape[3] > width
    if cache.dim() != 4 or cache.shape[3] != width + split * out.shape[2] or cache.dtype != q.dtype or not cache.is_contiguous():
        raise ValueError(f"cache must be contiguous (blocks, block_size, kv heads, {width} or that and the values' width) in q's dtype")
    if block_tables.dtype != torch.int32 or block_tables.dim() != 2 or not block_tables.is_contiguous():
        raise ValueError("block_tables must be contiguous int32 (entries, width)")
    if row_entry.dtype != torch.int32 or row_entry.numel() < rows or not row_entry.is_contiguous():
        raise ValueError("row_entry must be contiguous int32, one per row")
    _index(lens, rows, "lens")
    _floats("slopes", slopes, heads)
    groups, block_size, values, most = cache.shape[2], cache.shape[1], out.shape[2], block_tables.shape[1]
    need = window_decode_workspace_bytes(rows, heads, groups, cache.shape[3], values, most * block_size, q.dtype)
    if need and (workspace is None or workspace.numel() < need):
        workspace = torch.empty(need, dtype=torch.uint8, device=q.device)
    lib = _C.load()
    st = (lib.mvllm_window_decode_split if split else lib.mvllm_window_decode)(
        _ptr(out), *_heads("out", out, q, rows, heads, 1), _ptr(q), *_heads("q", q, q, rows, heads, width), _ptr(cache),
        _ptr(block_tables), most, _ptr(row_entry), _ptr(lens), _ptr(slopes), _ptr(gate), *_gate(gate, q, rows, heads, values),
        rows, heads, groups, width, values, block_size, cache.shape[0], int(window), int(ring), float(scale), float(temperature[0]),
        float(temperature[1]), _C.dtype_code(q.dtype), _ptr(workspace), 0 if workspace is None else workspace.numel(),
        _C.current_stream_ptr(q.device))
    _C.check(st, "window_decode")
