"""Token mixers of models that run ragged steps (engine/ragged.py): attention over a window cache and the matrix memory.

``RaggedAttention`` runs a step's pieces through the framework's decode, paged-prefill and packed-prefill kernels;
``MatrixMemory`` runs it through the mLSTM recurrence.  Both take the packed projection of the step's rows and return what
the output projection reads.  Caches and states are assigned from outside, as for ``layers.attention.Attention``."""
from __future__ import annotations

import math

import torch
import torch.nn as nn

from minivllm_amd.layers.attention import (flash_attention_prefill, flash_attention_prefill_paged, paged_attention_decode,
                                           store_kvcache)
from minivllm_amd.layers.fused import head_rope_store, head_unrotate_gate
from minivllm_amd.layers.recurrent import MlstmState, gate_linear, mlstm

LOG2E = math.log2(math.e)


def attention_head_dim(dim: int, vdim: int, dtype: torch.dtype) -> int:
    """Head size the attention kernels run at for keys of ``dim`` and values of ``vdim``: the next one with a tiled kernel
    (zeros fill it up), or the next multiple of 8 for the generic kernels."""
    need = max(dim, vdim)
    sizes = (64, 128) if dtype == torch.float32 else (32, 48, 64, 80, 96, 112, 128, 256)
    return next((d for d in sizes if d >= need), -(-need // 8) * 8)


class RaggedAttention(nn.Module):
    """softmax(scale q k + window mask, with an optional sink) over per-head-normed, rotated q and k, optionally with
    rotated values that are turned back on the way out and a sigmoid gate per head.

    The step's projection rows hold q | k | v at their start and, with ``gate_col`` >= 0, one gate pre-activation per head
    from that column on.  ``window``: index into the step's windows."""

    def __init__(self, num_heads, num_kv_heads, dim, vdim, scale, window, block_size, dtype, eps, interleaved=True,
                 gate_col=-1):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.dim, self.vdim = num_heads, num_kv_heads, dim, vdim
        self.head_dim = attention_head_dim(dim, vdim, dtype)
        self.scale, self.window, self.block_size, self.eps = scale, window, block_size, eps
        self.interleaved, self.gate_col = interleaved, gate_col
        self.k_cache = self.v_cache = torch.tensor([])
        self.decode_workspace = None

    def forward(self, proj, step, gain_q=None, gain_k=None, rot_table=None, v_table=None, sink=None):
        w = step.windows[self.window]
        packed = w.num_fresh > 0 or w.late_slots is not None
        # log2 e goes into q with the scale, in fp32: the attention kernels, which multiply q by scale * log2 e and round
        # it, then find a factor of one
        q, k, v = head_rope_store(proj, step.positions, self.num_heads, self.num_kv_heads, self.dim, self.vdim,
                                  self.head_dim, gain_q, gain_k, self.eps, self.scale * LOG2E, rot_table, v_table,
                                  self.interleaved, w.dst_row, w.slots, self.k_cache, self.v_cache, need_kv=packed)
        o = torch.empty_like(q)
        shape = (1.0 / LOG2E, self.num_heads, self.num_kv_heads, self.head_dim)
        a, b = w.num_decode, w.num_decode + w.num_prefixed
        if a:
            paged_attention_decode(q[:a], self.k_cache, self.v_cache, w.decode_tables, w.chunk_lens, *shape, self.block_size,
                                   workspace=self.decode_workspace, sink=sink, out=o[:a])
        if b > a:
            flash_attention_prefill_paged(q[a:b], self.k_cache, self.v_cache, w.prefixed_tables, w.prefixed_cu_q,
                                          w.prefixed_cu_k, *shape, self.block_size, w.prefixed_max_k, sink=sink, out=o[a:b])
        if w.num_fresh:
            flash_attention_prefill(q[b:], k[b:], v[b:], w.fresh_cu, *shape, sink=sink, out=o[b:])
        if w.late_slots is not None:
            store_kvcache(k, v, self.k_cache, self.v_cache, w.late_slots, self.block_size)
        gate = proj[:, self.gate_col:self.gate_col + self.num_heads] if self.gate_col >= 0 else None
        return head_unrotate_gate(o, step.positions, self.vdim, gate, v_table, self.interleaved, w.dst_row)


class MatrixMemory(nn.Module):
    """The mLSTM: projection rows hold q | k | v | output gate; the input and forget gates are projections of their own
    (``gate_weight`` (2 H, width), ``gate_bias`` float32), computed and kept in fp32."""

    def __init__(self, num_heads, dim, vdim, gate_cap, eps):
        super().__init__()
        self.num_heads, self.dim, self.vdim, self.gate_cap, self.eps = num_heads, dim, vdim, gate_cap, eps
        self.gate_col = num_heads * (2 * dim + vdim)
        self.state: MlstmState | None = None

    def forward(self, h, proj, step, gate_weight, gate_bias, norm_weight):
        gates = gate_linear(h, gate_weight, gate_bias, self.num_heads, self.gate_cap)
        return mlstm(step, proj, gates, self.gate_col, norm_weight, self.state, self.eps)
