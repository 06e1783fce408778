"""Token mixers of models that run ragged steps (engine/ragged.py): attention over a window cache or over latents, and matrix
memories.

``RaggedAttention`` runs a step's pieces through the framework's decode, paged-prefill and packed-prefill kernels,
``LatentAttention`` through the latent decode and the same prefill kernels, ``SharedKeyAttention``, ``RotaryLatentAttention`` and
``UnitHeadAttention`` through the windowed kernels, ``TalkingAttention`` through the ones that mix heads' scores;
``MatrixMemory`` runs it through the mLSTM recurrence, ``DecayMemory`` through the one with constant decays.  ``RaggedAttention``
and the memories take the packed projection of the step's rows and return what the output projection reads.  Caches and states
are assigned from outside, as for ``layers.attention.Attention``."""
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
from minivllm_amd.layers.talk import talk_decode, talk_decode_workspace_bytes, talk_head_size, talk_prefill
from minivllm_amd.layers.window import (copy_rows, head_rope, head_size, latent_layout, latent_rope_store, shared_part_size,
                                        window_decode, window_decode_workspace_bytes, window_prefill)
from minivllm_amd.layers.recurrent import DecayMemoryState, MlstmState, decay_memory, gate_linear, gated_row_norm, mlstm
from minivllm_amd.engine.windows import SlidingWindow
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


def distance_slopes(heads: int) -> torch.Tensor:
    """2^(-8 (h + 1) / heads) of head h, float32."""
    return (2.0 ** (-8.0 * torch.arange(1, heads + 1, dtype=torch.float64) / heads)).float()


class SharedKeyAttention(nn.Module):
    """Grouped softmax attention in a sliding window whose values are the keys, without a rotation: ``slopes`` times the distance is
    taken off a score, ``temperature`` = (coef, every) makes scores grow with the query's position, a gate per channel follows.

    It works between two projections that it may share with other sublayers: ``forward`` reads columns q | k | gate of ``proj`` and
    writes ``out`` (T, H * head_dim).  ``sizes``: columns it needs of both; ``window``: index into the step's windows."""

    def __init__(self, num_heads, num_kv_heads, dim, scale, window, view: SlidingWindow, block_size, dtype, temperature=(0.0, 0),
                 slopes=None, gated=True):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.dim, self.scale = num_heads, num_kv_heads, dim, scale
        self.window, self.view, self.block_size, self.dtype = window, view, block_size, dtype
        self.temperature, self.slopes, self.gated = temperature, slopes, gated
        d = self.head_dim = head_size(dim)
        self.q_size, self.k_size = num_heads * d, num_kv_heads * d
        self.sizes = (self.q_size + self.k_size + (self.q_size if gated else 0), self.q_size)
        self.cache = torch.tensor([])                                     # (blocks, block_size, G, head_dim)
        self.decode_workspace = None

    def load(self, get, matrix, inputs):
        """``get(name)``: checkpoint tensor, ``matrix(t)``: on the device in the model's type.  Returns this sublayer's rows of the
        projection in front of it and its columns of the one behind."""
        d, rows = self.head_dim, [("q", self.num_heads), ("k", self.num_kv_heads)] + [("g", self.num_heads)] * self.gated
        front = torch.cat([pad_heads(matrix(get(n)), h, d, inputs) for n, h in rows])
        if self.slopes is not None:
            self.slopes = self.slopes.to(front.device)
        return front, pad_heads(matrix(get("o")).t().contiguous(), self.num_heads, d).t()

    def allocate(self, num_blocks, device):
        self.cache = torch.zeros(num_blocks, self.block_size, self.num_kv_heads, self.head_dim, dtype=self.dtype, device=device)

    def workspace_bytes(self, batch, table_width):
        return window_decode_workspace_bytes(batch, self.num_heads, self.num_kv_heads, self.head_dim, self.head_dim,
                                             table_width * self.block_size, self.dtype)

    def forward(self, h, proj, out, step):
        view, heads, groups, d = step.windows[self.window], self.num_heads, self.num_kv_heads, self.head_dim
        a = view.absorbed
        q, k, o = proj[:, :self.q_size].unflatten(-1, (heads, d)), proj[:, self.q_size:self.q_size + self.k_size], out.unflatten(-1, (heads, d))
        gate = proj[:, self.q_size + self.k_size:self.sizes[0]].unflatten(-1, (heads, d)) if self.gated else None
        cut = lambda t, *rows: None if t is None else t[slice(*rows)]
        places, keys, key_rows, cu_k = self.cache.view(-1, self.k_size), None, None, view.cu_q
        if view.past_slots is not None:                                   # the past comes out of the ring before the new keys go in
            keys, key_rows, cu_k = torch.empty((view.num_keys, self.k_size), dtype=k.dtype, device=k.device), view.key_rows, view.cu_k
            copy_rows(places, keys, view.past_rows, view.past_slots)
        copy_rows(k, places, view.slots, None, keys, key_rows)
        how = dict(slopes=self.slopes, temperature=self.temperature)
        if a:
            window_decode(o[:a], q[:a], self.cache, view.tables, step.row_entry, view.lens, self.scale, self.view.size, self.view.places,
                          gate=cut(gate, 0, a), workspace=self.decode_workspace, **how)
        if view.num_long:
            keys = k[a:] if keys is None else keys
            window_prefill(o[a:], q[a:], keys.unflatten(-1, (groups, d)), view.cu_q, cu_k, self.scale, self.view.size,
                           gate=cut(gate, a, None), positions=step.positions[a:], **how)


class RotaryLatentAttention(nn.Module):
    """Softmax attention in a sliding window over keys and values made of one cached latent per token, with a rotated part of the
    keys beside it that all heads share.  Queries come from the input, or from a normed latent of their own (``q_rank``).

    Single rows and short entries are answered from the latents (queries through the heads' key matrices, results through their
    value matrices), for long entries keys and values are made of them.  It works between two projections like
    ``SharedKeyAttention``: columns q (or the queries' latent) | latent | rotated part.  ``table``: float32
    (max_position, dims / 2, 2), assigned from outside."""

    def __init__(self, num_heads, dim, rot_dim, vdim, rank, scale, window, view: SlidingWindow, block_size, dtype, eps, interleaved,
                 q_rank=0, small_rows=0):
        super().__init__()
        self.num_heads, self.dim, self.rot_dim, self.vdim, self.rank, self.scale = num_heads, dim, rot_dim, vdim, rank, scale
        self.window, self.view, self.block_size, self.dtype, self.eps = window, view, block_size, dtype, eps
        self.interleaved, self.q_rank = interleaved, q_rank
        d, self.rot_size = head_size(dim, vdim), shared_part_size(rot_dim)
        self.head_dim, self.q_dim = d, d + self.rot_size
        self.rot_column, self.latent_width, self.values = latent_layout(rank, rot_dim)
        self.q_size = num_heads * self.q_dim
        self.q_columns = round_up(q_rank, 64) if q_rank else self.q_size
        self.sizes = (self.q_columns + self.latent_width, num_heads * d)
        if q_rank:
            with torch.device("meta"):
                self.up_q = Linear(self.q_columns, self.q_size, bias=False, small_rows=small_rows)
        self.table = None
        self.cache = torch.tensor([])                                     # (blocks, block_size, 1, latent_width)
        self.decode_workspace = None

    @torch.no_grad()
    def load(self, get, matrix, inputs):
        """As ``SharedKeyAttention.load``."""
        heads, d, r = self.num_heads, self.head_dim, self.rot_dim

        def query_rows(t, columns):                                       # (H * (dim + rot_dim), n): both parts filled up
            t = matrix(t)
            w = t.new_zeros(heads, self.q_dim, columns)
            of = t.view(heads, self.dim + r, -1)
            w[:, :self.dim, :t.shape[1]], w[:, d:d + r, :t.shape[1]] = of[:, :self.dim], of[:, self.dim:]
            return w.view(heads * self.q_dim, columns)

        down = matrix(get("dkv"))
        latent = down.new_zeros(self.latent_width, inputs)
        latent[:self.rank, :down.shape[1]], latent[self.rot_column:self.rot_column + r, :down.shape[1]] = down[:self.rank], down[self.rank:]
        f32 = lambda name: get(name).to(device=down.device, dtype=torch.float32).contiguous()
        self.norm_weight, self.q_norm_weight = f32("dkv.norm"), None
        if self.q_rank:
            self.q_norm_weight = f32("dq.norm")
            self.up_q.weight = nn.Parameter(query_rows(get("uq"), self.q_columns), requires_grad=False)
            first = pad_to(matrix(get("dq")), self.q_columns, inputs)
        else:
            first = query_rows(get("q"), inputs)
        uk, uv = (pad_heads(matrix(get(n)), heads, d, self.rot_column) for n in ("uk", "uv"))       # (H * D, latent columns)
        self.up_kv = torch.cat([uk, uv])
        self.absorb_k = uk.view(heads, d, -1).transpose(1, 2).contiguous()
        self.absorb_v = pad_to(uv, None, self.values)[:, :self.values].contiguous().view(heads, d, self.values)
        return torch.cat([first, latent]), pad_heads(matrix(get("o")).t().contiguous(), heads, d).t()

    def allocate(self, num_blocks, device):
        self.cache = torch.zeros(num_blocks, self.block_size, 1, self.latent_width, dtype=self.dtype, device=device)

    def workspace_bytes(self, batch, table_width):
        return window_decode_workspace_bytes(batch, self.num_heads, 1, self.latent_width, self.values, table_width * self.block_size, self.dtype)

    def forward(self, h, proj, out, step):
        view, heads, d, w, rot = step.windows[self.window], self.num_heads, self.head_dim, self.latent_width, self.rot_column
        t, a, new = proj.shape[0], view.absorbed, lambda *shape: torch.empty(shape, dtype=proj.dtype, device=proj.device)
        cache, rows, key_rows = self.cache.view(-1, self.block_size, w), None, None
        if view.num_long:
            rows, key_rows = new(view.num_keys, w), view.key_rows
            if view.past_slots is not None:                               # out of the ring before the new latents go in
                copy_rows(cache.view(-1, w), rows, view.past_rows, view.past_slots)
        first, latents = proj[:, :self.q_columns], proj[:, self.q_columns:self.sizes[0]]
        c_q = latent_rope_store(latents, self.norm_weight, self.eps, rot, self.rot_dim, self.table, step.positions, self.interleaved,
                                cache, view.slots, rows, key_rows, first if self.q_rank else None, self.q_norm_weight)
        q = (self.up_q(c_q) if self.q_rank else first).unflatten(-1, (heads, self.q_dim))
        x = new(a, heads, w) if a else None
        head_rope(q, d, self.rot_dim, self.table, step.positions, self.interleaved, x, rot, a)
        o = out.unflatten(-1, (heads, d))
        if a:
            y = new(a, heads, self.values)
            head_linear(q[:a, :, :d], self.absorb_k, out=x[:, :, :rot])
            window_decode(y, x, self.cache, view.tables, step.row_entry, view.lens, self.scale, self.view.size, self.view.places,
                          workspace=self.decode_workspace)
            head_linear(y, self.absorb_v, out=o[:a])
        if view.num_long:
            k, v = F.linear(rows[:, :rot], self.up_kv).unflatten(-1, (2, heads, d)).unbind(1)
            window_prefill(o[a:], q[a:], k, view.cu_q, view.cu_k, self.scale, self.view.size, k2=rows[:, rot:rot + self.rot_size], v=v)


class _HeadsAttention(nn.Module):
    """Grouped heads between projections of their own: rows q | k | v | (a gate per head) in front, heads side by side behind.
    Heads are ``head_dim`` wide behind the front projection, zeros past ``dim`` / ``vdim``.  ``table``: float32 (max_position,
    dims / 2, 2) or None, assigned from outside; ``window``: index into the step's windows."""

    def __init__(self, width, num_heads, num_kv_heads, dim, vdim, head_dim, scale, window, block_size, dtype, eps, interleaved, bias,
                 gated, small_rows):
        super().__init__()
        self.num_heads, self.num_kv_heads, self.dim, self.vdim, self.head_dim = num_heads, num_kv_heads, dim, vdim, head_dim
        self.window, self.block_size, self.dtype, self.eps, self.interleaved = window, block_size, dtype, eps, interleaved
        self.scale, self.gated = scale, gated
        self.gate_col = num_heads * dim + num_kv_heads * (dim + vdim)
        self.out_size = num_heads * head_dim
        with torch.device("meta"):
            self.proj = Linear(width, round_up(self.gate_col + (num_heads if gated else 0), 16), bias=bias, small_rows=small_rows)
            self.out = Linear(self.out_size, width, bias=False, small_rows=small_rows)
        self.table = None
        self.decode_workspace = None

    @torch.no_grad()
    def load(self, get, matrix, inputs):
        """``get(name)``: checkpoint tensor, ``matrix(t)``: on the device in the model's type; ``inputs``: columns of h."""
        p, total = lambda t: nn.Parameter(t.contiguous(), requires_grad=False), self.proj.out_features
        self.proj.weight = p(pad_to(torch.cat([matrix(get(n)) for n in ("q", "k", "v") + ("g",) * self.gated]), total, inputs))
        if self.proj.bias is not None:
            self.proj.bias = p(F.pad(torch.cat([matrix(get(n + ".b")) for n in ("q", "k", "v")]), (0, total - self.gate_col)))
        self.out.weight = p(pad_heads(matrix(get("o")).t().contiguous(), self.num_heads, self.head_dim).t())
        self.f32 = lambda name: get(name).to(device=self.out.weight.device, dtype=torch.float32).contiguous()

    def heads(self, proj, step, **how):
        # log2 e goes into q with the scale, in fp32, as in RaggedAttention
        return head_rope_store(proj, step.positions, self.num_heads, self.num_kv_heads, self.dim, self.vdim, self.head_dim,
                               eps=self.eps, q_scale=self.scale * LOG2E, rot_table=self.table, interleaved=self.interleaved, **how)


class UnitHeadAttention(_HeadsAttention):
    """Softmax attention in a sliding window over heads of unit root mean square: rotated queries and keys (``unit_qk``), values
    (``unit_v``), with a learned factor per head on the scores and a sigmoid gate per head on the results.  A cached row holds a
    key and behind it its value."""

    def __init__(self, width, num_heads, num_kv_heads, dim, vdim, scale, window, view: SlidingWindow, block_size, dtype, eps,
                 interleaved=True, unit_qk=True, unit_v=True, bias=True, gated=True, small_rows=0):
        super().__init__(width, num_heads, num_kv_heads, dim, vdim, head_size(dim, vdim), scale, window, block_size, dtype, eps,
                         interleaved, bias, gated, small_rows)
        self.view, self.unit_qk, self.unit_v = view, unit_qk, unit_v
        self.cache = torch.tensor([])                                     # (blocks, block_size, G, 2 * head_dim)
        self.head_scale = None

    def load(self, get, matrix, inputs):
        super().load(get, matrix, inputs)
        self.head_scale = self.f32("temp")

    def allocate(self, num_blocks, device):
        self.cache = torch.zeros(num_blocks, self.block_size, self.num_kv_heads, 2 * self.head_dim, dtype=self.dtype, device=device)

    def workspace_bytes(self, batch, table_width):
        return window_decode_workspace_bytes(batch, self.num_heads, self.num_kv_heads, 2 * self.head_dim, self.head_dim,
                                             table_width * self.block_size, self.dtype)

    def forward(self, h, step):
        view, d, a = step.windows[self.window], self.head_dim, step.windows[self.window].absorbed
        proj = self.proj(h)
        keys = None
        if view.num_long:
            keys = torch.empty((view.num_keys, self.num_kv_heads, 2 * d), dtype=proj.dtype, device=proj.device)
            if view.past_slots is not None:                               # out of the ring before the new ones go in
                copy_rows(self.cache.view(-1, keys[0].numel()), keys.flatten(1), view.past_rows, view.past_slots)
        q = self.heads(proj, step, unit_qk=self.unit_qk, unit_v=self.unit_v, head_scale=self.head_scale, kv_cache=self.cache,
                       slots=view.slots, kv_out=keys, kv_rows=view.key_rows)
        gate = proj[:, self.gate_col:self.gate_col + self.num_heads] if self.gated else None
        cut = lambda *rows: None if gate is None else gate[slice(*rows)]
        o = torch.empty_like(q)
        if a:
            window_decode(o[:a], q[:a], self.cache, view.tables, step.row_entry, view.lens, 1.0 / LOG2E, self.view.size, self.view.places,
                          gate=cut(0, a), workspace=self.decode_workspace)
        if view.num_long:
            window_prefill(o[a:], q[a:], keys[..., :d], view.cu_q, view.cu_k, 1.0 / LOG2E, self.view.size, v=keys[..., d:], gate=cut(a, None))
        return self.out(o.flatten(1))


class TalkingAttention(_HeadsAttention):
    """Chunked attention whose heads' scores are mixed before the softmax (``talk``), with a sink; queries and keys are normed over
    all heads of a row at once, then rotated."""

    def __init__(self, width, num_heads, num_kv_heads, dim, vdim, scale, window, block_size, dtype, eps, interleaved=True, sink=None,
                 small_rows=0):
        super().__init__(width, num_heads, num_kv_heads, dim, vdim, talk_head_size(dim, vdim), scale, window, block_size, dtype, eps,
                         interleaved, False, False, small_rows)
        if num_heads > 64 or self.out_size > 16384:
            raise ValueError(f"{num_heads} heads of {self.head_dim}: at most 64 and 16384 columns together")
        self.sink = sink                                                  # one number for all heads, or None
        self.k_cache = self.v_cache = torch.tensor([])                    # (blocks, block_size, G, head_dim)

    def load(self, get, matrix, inputs):
        super().load(get, matrix, inputs)
        self.gain_q, self.gain_k, self.talk = (self.f32(n) for n in ("q.norm", "k.norm", "talk"))
        self.sinks = None if self.sink is None else torch.full((self.num_heads,), float(self.sink), device=self.talk.device)

    def allocate(self, num_blocks, device):
        shape = (num_blocks, self.block_size, self.num_kv_heads, self.head_dim)
        self.k_cache, self.v_cache = (torch.zeros(shape, dtype=self.dtype, device=device) for _ in range(2))

    def workspace_bytes(self, batch, table_width):
        return talk_decode_workspace_bytes(batch, self.num_heads, self.num_kv_heads, self.head_dim, table_width * self.block_size, self.dtype)

    def forward(self, h, step):
        w = step.windows[self.window]
        a, b = w.num_decode, w.num_decode + w.num_prefixed
        q, k, v = self.heads(self.proj(h), step, gain_q=self.gain_q, gain_k=self.gain_k, row_norm=True, dst_row=w.dst_row, slots=w.slots,
                             k_cache=self.k_cache, v_cache=self.v_cache, need_kv=w.num_fresh > 0 or w.late_slots is not None)
        o = torch.empty_like(q)
        if a:
            talk_decode(o[:a], q[:a], self.k_cache, self.v_cache, w.decode_tables, w.chunk_lens, self.talk, self.sinks, self.decode_workspace)

        def prefill(lo, hi, *keys, **how):                                # results go back to where the rows came from
            where = dict(out=o, out_rows=w.src_row[lo:hi]) if w.src_row is not None else dict(out=o[lo:hi])
            talk_prefill(q=q[lo:hi], k=keys[0], v=keys[1], talk=self.talk, sinks=self.sinks, **where, **how)

        if b > a:
            prefill(a, b, self.k_cache, self.v_cache, cu_q=w.prefixed_cu_q, cu_k=w.prefixed_cu_k, block_tables=w.prefixed_tables)
        if w.num_fresh:
            prefill(b, q.shape[0], k[b:], v[b:], cu_q=w.fresh_cu)
        if w.late_slots is not None:
            store_kvcache(k, v, self.k_cache, self.v_cache, w.late_slots, self.block_size)
        return self.out(o.flatten(1))
