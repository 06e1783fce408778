"""Token mixers of models that run ragged steps (engine/ragged.py): attention over a window cache or over latents, and matrix
memories.

``RaggedAttention`` runs a step's pieces through the framework's decode, paged-prefill and packed-prefill kernels,
``LatentAttention`` through the latent decode and the same prefill kernels; ``MatrixMemory`` runs it through the mLSTM
recurrence, ``DecayMemory`` through the one with constant decays.  ``RaggedAttention`` and the memories take the packed
projection of the step's rows and return what the output projection reads.  Caches and states are assigned from outside, as
for ``layers.attention.Attention``."""
from __future__ import annotations

import math

import torch
import torch.nn as nn
import torch.nn.functional as F

from minivllm_amd.layers.attention import (decode_workspace_bytes, flash_attention_prefill, flash_attention_prefill_paged,
                                           paged_attention_decode, store_kvcache)
from minivllm_amd.layers.fused import head_rope_store, head_unrotate_gate
from minivllm_amd.layers.basic import Linear
from minivllm_amd.layers.latent import (head_linear, latent_decode, latent_decode_workspace_bytes, latent_norm_store,
                                        latent_width)
from minivllm_amd.layers.recurrent import DecayMemoryState, MlstmState, decay_memory, gate_linear, gated_row_norm, mlstm
from minivllm_amd.utils.padding import pad_heads, pad_to, round_up

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

    def workspace_bytes(self, batch, table_width):
        """Scratch of a decode step of ``batch`` rows."""
        return decode_workspace_bytes(batch, self.num_heads, self.head_dim, table_width, self.block_size)

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


class DecayMemory(nn.Module):
    """Lightning attention: q, k and v through silu, a matrix memory with a constant decay per head, one norm over all heads
    of a row and a sigmoid gate per channel.  Projection rows hold q | k | v | gate."""

    def __init__(self, num_heads, dim, vdim, eps):
        super().__init__()
        self.num_heads, self.dim, self.vdim, self.eps = num_heads, dim, vdim, eps
        self.gate_col = num_heads * (2 * dim + vdim)
        self.state: DecayMemoryState | None = None

    def forward(self, proj, step, norm_weight):
        o = decay_memory(step, proj, self.state)
        return gated_row_norm(o, norm_weight, proj[:, self.gate_col:self.gate_col + self.num_heads * self.vdim], self.eps)


class LatentAttention(nn.Module):
    """Causal softmax attention without positions whose keys and values are linear in one cached latent per token.

    Single tokens and short portions are answered from the latents (queries through the heads' key matrices, results through
    their value matrices); for long portions keys and values are made of the latents and the prefill kernels run.  With
    ``source`` the latents, their cache and the slots are another module's.  Heads are ``head_dim`` wide everywhere, zeros past
    ``dim`` / ``vdim``; weights come from ``load``."""

    def __init__(self, width, num_heads, dim, vdim, rank, scale, window, block_size, dtype, eps, source=None, small_rows=0):
        super().__init__()
        self.num_heads, self.dim, self.vdim, self.rank, self.scale, self.eps = num_heads, dim, vdim, rank, scale, eps
        self.head_dim = round_up(attention_head_dim(dim, vdim, dtype), 16)
        self.latent_width = latent_width(rank)
        self.window, self.block_size, self.dtype = window, block_size, dtype
        self._source = (source,) if source is not None else ()           # not a submodule
        self.q_size = num_heads * self.head_dim
        with torch.device("meta"):
            self.proj = Linear(width, self.q_size + (0 if source is not None else self.latent_width), bias=False, small_rows=small_rows)
            self.out = Linear(self.q_size, width, bias=False, small_rows=small_rows)
        self.cache = torch.tensor([])                                     # (blocks, block_size, latent_width), the owner's
        self.rows = None                                                  # the step's latents, packed, the owner's
        self.decode_workspace = None

    @property
    def owner(self):
        return self._source[0] if self._source else self

    @torch.no_grad()
    def load(self, get, matrix, inputs):
        """``get(name)``: checkpoint tensor, ``matrix(t)``: on the device in the model's type; ``inputs``: columns of h."""
        h, d, w, p = self.num_heads, self.head_dim, self.latent_width, lambda t: nn.Parameter(t.contiguous(), requires_grad=False)
        rows = [pad_heads(matrix(get("q")), h, d, inputs)]
        if not self._source:
            rows.append(pad_to(matrix(get("dkv")), w, inputs))
            self.norm_weight = get("dkv.norm").to(device=rows[0].device, dtype=torch.float32).contiguous()
        self.proj.weight = p(torch.cat(rows))
        uk, uv = (pad_heads(matrix(get(n)), h, d, w) for n in ("uk", "uv"))           # (H * D, width)
        self.up_k, self.up_v = uk, uv
        self.absorb_k = uk.view(h, d, w).transpose(1, 2).contiguous()
        self.absorb_v = uv.view(h, d, w)
        self.out.weight = p(pad_heads(matrix(get("o")).t().contiguous(), h, d).t())

    def workspace_bytes(self, batch, table_width):
        return latent_decode_workspace_bytes(batch, self.num_heads, self.latent_width, table_width * self.block_size, self.dtype)

    def forward(self, h, step):
        view, own = step.windows[self.window], not self._source
        t, heads, d = h.shape[0], self.num_heads, self.head_dim
        a, b = view.absorbed, view.absorbed + view.num_prefixed
        if t <= self.proj.small_rows:
            both = self.proj(h)
            q, c = both[:, :self.q_size], both[:, self.q_size:] if own else None
        else:                                                             # separate products: packed queries for the prefill
            q = F.linear(h, self.proj.weight[:self.q_size])
            c = F.linear(h, self.proj.weight[self.q_size:]) if own else None
        if own:
            self.rows = latent_norm_store(c, self.norm_weight, self.eps, self.cache, view.slots, need_rows=b < t)
        cache, rows = self.owner.cache, self.owner.rows
        o = torch.empty((t, heads, d), dtype=h.dtype, device=h.device)
        q = q.unflatten(-1, (heads, d))
        if a:
            x = head_linear(q[:a], self.absorb_k)
            x = latent_decode(x, cache, view.tables, step.row_entry, view.lens, self.scale, self.decode_workspace)
            head_linear(x, self.absorb_v, out=o[:a])
        shape = (self.scale, heads, heads, d)
        if b > a:
            # the cached latents of these entries, block by block, and the keys and values made of them: a cache of its own
            key = id(self.owner)
            if key not in step.scratch:
                step.scratch[key] = cache[view.gather].view(-1, self.latent_width)
            blocks = (-1, self.block_size, heads, d)
            k, v = (F.linear(step.scratch[key], w).view(blocks) for w in (self.up_k, self.up_v))
            flash_attention_prefill_paged(q[a:b], k, v, view.scratch_tables, view.prefixed_cu_q, view.prefixed_cu_k, *shape,
                                          self.block_size, view.prefixed_max_k, out=o[a:b])
        if b < t:
            k, v = (F.linear(rows[b:], w).view(-1, heads, d) for w in (self.up_k, self.up_v))
            flash_attention_prefill(q[b:], k, v, view.fresh_cu, *shape, out=o[b:])
        return self.out(o.view(t, heads * d))
