"""Metadata of a ragged step: entries of any length (portions of prompts beside single decoded tokens) in one packed batch.

Rows are packed entry by entry: entries of one token first, then short ones, then long ones.  Attention sees a row's entry
cut at chunk borders: the piece that goes on in a chunk whose earlier tokens are cached reads the cache (``prefixed``),
pieces that start a chunk read the packed keys and values of the step (``fresh``), single tokens take the decode kernel.
Pieces are sorted in that order (``dst_row``), so that each kernel runs over consecutive rows.  Only the tokens of an entry's
last chunk stay cached; where the entry also reads the chunk before, whose blocks they go to, they are stored after
attention (``late_slots``).
Layers that cache one latent per token (``LatentStep``) answer single and short entries row by row from the cache; long
entries with a cached prefix come before those without.
Layers with a sliding window (``RingStep``) answer single and short entries row by row from their ring; long entries bring the
last tokens of their past with them, taken out of the ring before the new ones go in.
A recurrence takes single and short entries row by row and long ones in blocks of rows, cut into ``segments`` that run side
by side where there are too few of them to fill the GPU."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

import numpy as np
import torch

from minivllm_amd.engine.windows import LONG_ROWS, SlidingWindow


@dataclass
class WindowStep:
    """One attention window's view of the step."""
    num_decode: int = 0
    num_prefixed: int = 0                             # rows of pieces with a cached prefix
    num_fresh: int = 0
    dst_row: Optional[torch.Tensor] = None            # int32 [T], None: rows stay in order
    src_row: Optional[torch.Tensor] = None            # int32 [T], the way back, None: rows stay in order
    slots: Optional[torch.Tensor] = None              # int64 [T], stored before attention (-1: not)
    late_slots: Optional[torch.Tensor] = None         # int64 [T] in dst_row order, stored after attention, or None
    chunk_lens: Optional[torch.Tensor] = None         # int64 [num_decode]
    decode_tables: Optional[torch.Tensor] = None      # int32 [num_decode, width]
    prefixed_cu_q: Optional[torch.Tensor] = None      # int32 [pieces + 1]
    prefixed_cu_k: Optional[torch.Tensor] = None
    prefixed_tables: Optional[torch.Tensor] = None
    prefixed_max_k: int = 0
    fresh_cu: Optional[torch.Tensor] = None


@dataclass
class LatentStep:
    """The step as layers see it that cache one latent per token and attend to the whole sequence."""
    absorbed: int = 0                                 # rows of single and short entries (the first ones)
    num_prefixed: int = 0                             # rows of long entries behind a cached prefix, next
    num_fresh: int = 0                                # rows of long entries that start a sequence
    slots: Optional[torch.Tensor] = None              # int64 [T]
    lens: Optional[torch.Tensor] = None               # int64 [absorbed]: keys a row sees
    tables: Optional[torch.Tensor] = None             # int32 [entries, width]
    prefixed_cu_q: Optional[torch.Tensor] = None      # int32 [entries + 1]
    prefixed_cu_k: Optional[torch.Tensor] = None
    prefixed_max_k: int = 0
    gather: Optional[torch.Tensor] = None             # int64 [blocks]: the prefixed entries' blocks, one after the other
    scratch_tables: Optional[torch.Tensor] = None     # int32 [entries, width]: their places in that order
    fresh_cu: Optional[torch.Tensor] = None


@dataclass
class RingStep:
    """The step as layers with a sliding window see it: new tokens go to ``slots`` of the ring; rows of long entries find their
    keys in a packed order, every entry's past in front of its own."""
    absorbed: int = 0                                 # rows of single and short entries (the first ones)
    num_long: int = 0                                 # rows of long entries, next
    num_keys: int = 0                                 # packed keys of the long entries
    slots: Optional[torch.Tensor] = None              # int64 [T], -1: overwritten by a later row of the step
    lens: Optional[torch.Tensor] = None               # int64 [absorbed]: position + 1
    tables: Optional[torch.Tensor] = None             # int32 [entries, width]
    cu_q: Optional[torch.Tensor] = None               # int32 [long entries + 1]
    cu_k: Optional[torch.Tensor] = None
    key_rows: Optional[torch.Tensor] = None           # int64 [T]: packed place of a row's own key, -1 for absorbed rows
    past_slots: Optional[torch.Tensor] = None         # int64 [n]: where the past of the long entries lies (None: no past) ...
    past_rows: Optional[torch.Tensor] = None          # ... and its packed places


@dataclass
class RaggedStep:
    num_tokens: int
    num_entries: int
    num_single: int                                   # entries of one token, packed first
    input_ids: torch.Tensor                           # int64 [T]
    positions: torch.Tensor                           # int64 [T]
    cu_seqlens: torch.Tensor                          # int32 [entries + 1]
    row_entry: torch.Tensor                           # int32 [T]
    bank_in: torch.Tensor                             # int32 [entries]: banks of the short-convolution state
    bank_out: torch.Tensor
    state_slots: torch.Tensor                         # int32 [entries]
    windows: list = field(default_factory=list)       # WindowStep (LatentStep, RingStep) per window
    multi_rows: int = 0                               # rows of entries with more than one token
    num_short: int = 0                                # entries below LONG_ROWS (the first ones)
    segments: Optional[torch.Tensor] = None           # int32 [n, 4] of long entries: entry, first row, rows, flags
    split: bool = False                               # some long entry has more than one segment
    order: list = field(default_factory=list)         # entry e of the packing is sequence order[e] of the caller
    starts: list = field(default_factory=list)        # first packed row of the caller's sequence i
    scratch: dict = field(default_factory=dict)       # what layers of one step share


BLOCK_ROWS = 64                # rows per block of a recurrence's block form: segments are whole blocks
FILL_WORKGROUPS = 512          # segments are made shorter until there are this many workgroups ...
MIN_SEGMENT_ROWS = 256         # ... but not shorter than this


def _segments(lens, cu, units):
    """[entry, first row, rows, flags (1 first, 2 last, 4 only)] of every long entry."""
    long_entries = [e for e, n in enumerate(lens) if n >= LONG_ROWS]
    total = int(sum(lens[e] for e in long_entries))
    length = total
    if long_entries and units and len(long_entries) * units < FILL_WORKGROUPS // 2:
        length = max(-(-total * units // (FILL_WORKGROUPS * BLOCK_ROWS)) * BLOCK_ROWS, MIN_SEGMENT_ROWS)
    out = []
    for e in long_entries:
        n, at = int(lens[e]), int(cu[e])
        pieces = max(-(-n // length), 1)
        size = -(-n // (pieces * BLOCK_ROWS)) * BLOCK_ROWS
        cuts = list(range(0, n, size)) + [n]
        for i, (lo, hi) in enumerate(zip(cuts, cuts[1:])):
            first, last = i == 0, hi == n
            out.append([e, at + lo, hi - lo, int(first) | 2 * int(last) | 4 * int(first and last)])
    return out


def _pad_tables(tables):
    width = max((len(t) for t in tables), default=1) or 1
    out = np.full((len(tables), width), -1, dtype=np.int32)
    for i, t in enumerate(tables):
        out[i, :len(t)] = t
    return out


def _window_arrays(items, window, index, block_size, cu):
    """Host arrays of one window; items: (tokens before, new tokens, sequence) in packing order."""
    total = int(cu[-1])
    slots = np.full(total, -1, dtype=np.int64)
    late = np.full(total, -1, dtype=np.int64)
    any_late = False
    chunk_lens, decode_tables = [], []
    pre_rows, pre_q, pre_k, pre_tables = [], [0], [0], []
    fresh_rows, fresh_q = [], [0]
    single = 0
    for e, (p0, n, seq) in enumerate(items):
        table = np.asarray(seq.group_tables[index], dtype=np.int64)
        at = int(cu[e])
        local = np.arange(p0, p0 + n)
        size = window or p0 + n
        place = local % size
        where = table[place // block_size] * block_size + place % block_size
        if n == 1:
            chunk_lens.append(int(place[0]) + 1)
            decode_tables.append(seq.group_tables[index])
            slots[at] = where[0]
            single += 1
            continue
        head = 0
        if p0 % size:
            head = min(size - p0 % size, n)
            pre_rows.append(np.arange(at, at + head))
            pre_q.append(pre_q[-1] + head)
            pre_k.append(pre_k[-1] + p0 % size + head)
            pre_tables.append(seq.group_tables[index])
            slots[at:at + head] = where[:head]
        if head < n:
            fresh_rows.append(np.arange(at + head, at + n))
            cuts = list(range(head + size, n, size)) + [n]
            base = fresh_q[-1] - head
            fresh_q.extend(base + c for c in cuts)
            last = cuts[-2] if len(cuts) > 1 else head
            if head:
                late[at + last:at + n] = where[last:]
                any_late = True
            else:
                slots[at + last:at + n] = where[last:]
    order = np.concatenate([np.arange(single), *pre_rows, *fresh_rows]).astype(np.int64)     # packed row of each sorted row
    sorted_as_packed = bool((order == np.arange(total)).all())
    dst = np.empty(total, dtype=np.int32)
    dst[order] = np.arange(total, dtype=np.int32)
    out = dict(slots=slots)
    if not sorted_as_packed:
        out["dst_row"] = dst
        out["src_row"] = order.astype(np.int32)
    if any_late:
        out["late_slots"] = late[order]
    if single:
        out["chunk_lens"] = np.asarray(chunk_lens, dtype=np.int64)
        out["decode_tables"] = _pad_tables(decode_tables)
    if pre_rows:
        out["prefixed_cu_q"] = np.asarray(pre_q, dtype=np.int32)
        out["prefixed_cu_k"] = np.asarray(pre_k, dtype=np.int32)
        out["prefixed_tables"] = _pad_tables(pre_tables)
    if fresh_rows:
        out["fresh_cu"] = np.asarray(fresh_q, dtype=np.int32)
    counts = dict(num_decode=single, num_prefixed=pre_q[-1], num_fresh=fresh_q[-1],
                  prefixed_max_k=int(np.diff(pre_k).max()) if pre_rows else 0)
    return out, counts


def _latent_arrays(items, index, block_size, cu, num_short):
    """Host arrays of a LatentStep; items as for ``_window_arrays``."""
    slots = np.empty(int(cu[-1]), dtype=np.int64)
    pre_q, pre_k, gather, scratch, fresh = [0], [0], [], [], [0]
    tables = [seq.group_tables[index] for _, _, seq in items]
    for e, (p0, n, _) in enumerate(items):
        place = np.arange(p0, p0 + n)
        slots[cu[e]:cu[e + 1]] = np.asarray(tables[e], dtype=np.int64)[place // block_size] * block_size + place % block_size
        if e < num_short:
            continue
        if p0:
            pre_q.append(pre_q[-1] + n)
            pre_k.append(pre_k[-1] + p0 + n)
            used = -(-(p0 + n) // block_size)
            scratch.append(list(range(len(gather), len(gather) + used)))
            gather += tables[e][:used]
        else:
            fresh.append(fresh[-1] + n)
    absorbed = int(cu[num_short])
    out = dict(slots=slots, tables=_pad_tables(tables))
    if absorbed:
        out["lens"] = np.concatenate([np.arange(p, p + n, dtype=np.int64) + 1 for p, n, _ in items[:num_short]])
    if scratch:
        out.update(prefixed_cu_q=np.asarray(pre_q, dtype=np.int32), prefixed_cu_k=np.asarray(pre_k, dtype=np.int32),
                   gather=np.asarray(gather, dtype=np.int64), scratch_tables=_pad_tables(scratch))
    if len(fresh) > 1:
        out["fresh_cu"] = np.asarray(fresh, dtype=np.int32)
    counts = dict(absorbed=absorbed, num_prefixed=pre_q[-1], num_fresh=fresh[-1],
                  prefixed_max_k=int(np.diff(pre_k).max()) if scratch else 0)
    return out, counts


def _ring_arrays(items, window, index, block_size, cu, num_short):
    """Host arrays of a RingStep; items as for ``_window_arrays``."""
    total = int(cu[-1])
    slots, key_rows = np.full(total, -1, dtype=np.int64), np.full(total, -1, dtype=np.int64)
    cu_q, cu_k, past_slots, past_rows = [0], [0], [], []
    for e, (p0, n, seq) in enumerate(items):
        table = np.asarray(seq.group_tables[index], dtype=np.int64)

        def slots_of(positions):
            place = positions % window.places if window.places else positions
            return table[place // block_size] * block_size + place % block_size

        stay = min(n, window.places) if window.places else n
        slots[cu[e + 1] - stay:cu[e + 1]] = slots_of(np.arange(p0 + n - stay, p0 + n))
        if e < num_short:
            continue
        past = min(p0, window.size - 1) if window.size else p0
        if past:
            past_slots.append(slots_of(np.arange(p0 - past, p0)))
            past_rows.append(cu_k[-1] + np.arange(past))
        key_rows[cu[e]:cu[e + 1]] = cu_k[-1] + past + np.arange(n)
        cu_q.append(cu_q[-1] + n)
        cu_k.append(cu_k[-1] + past + n)
    absorbed = int(cu[num_short])
    out = dict(slots=slots, tables=_pad_tables([seq.group_tables[index] for _, _, seq in items]))
    if absorbed:
        out["lens"] = np.concatenate([np.arange(p, p + n, dtype=np.int64) + 1 for p, n, _ in items[:num_short]])
    if len(cu_q) > 1:
        out.update(cu_q=np.asarray(cu_q, dtype=np.int32), cu_k=np.asarray(cu_k, dtype=np.int32), key_rows=key_rows)
    if past_slots:
        out.update(past_slots=np.concatenate(past_slots), past_rows=np.concatenate(past_rows).astype(np.int64))
    return out, dict(absorbed=absorbed, num_long=cu_q[-1], num_keys=cu_k[-1])


def ragged_arrays(seqs, windows, block_size, memory_units=0, latent=False):
    """Host side of a step over ``seqs``: each runs its tokens [num_computed_tokens, + num_scheduled_tokens).  Returns
    (arrays, window arrays, window counts, facts), everything in numpy; the sequences' convolution banks flip for entries
    of more than one token."""
    kind = [((n > 1) + (n >= LONG_ROWS), s.num_computed_tokens == 0) for n, s in ((s.num_scheduled_tokens, s) for s in seqs)]
    order = sorted(range(len(seqs)), key=lambda i: kind[i])                                  # stable
    items = [(seqs[i].num_computed_tokens, seqs[i].num_scheduled_tokens, seqs[i]) for i in order]
    lens = np.asarray([n for _, n, _ in items], dtype=np.int64)
    cu = np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)
    ids = np.concatenate([np.asarray(s.token_ids[p:p + n], dtype=np.int64) for p, n, s in items])
    positions = np.concatenate([np.arange(p, p + n, dtype=np.int64) for p, n, _ in items])
    bank_in, bank_out = [], []
    for _, n, s in items:
        bank_in.append(2 * s.state_slot + s.state_bank)
        if n > 1:
            s.state_bank ^= 1
        bank_out.append(2 * s.state_slot + s.state_bank)
    arrays = dict(input_ids=ids, positions=positions, cu_seqlens=cu,
                  row_entry=np.repeat(np.arange(len(items), dtype=np.int32), lens),
                  bank_in=np.asarray(bank_in, dtype=np.int32), bank_out=np.asarray(bank_out, dtype=np.int32),
                  state_slots=np.asarray([s.state_slot for _, _, s in items], dtype=np.int32))
    num_short = int((lens < LONG_ROWS).sum())
    per_window = [_ring_arrays(items, w, g, block_size, cu, num_short) if isinstance(w, SlidingWindow) else
                  _latent_arrays(items, g, block_size, cu, num_short) if latent else _window_arrays(items, w, g, block_size, cu)
                  for g, w in enumerate(windows)]
    starts = [0] * len(seqs)
    for e, i in enumerate(order):
        starts[i] = int(cu[e])
    singles = int((lens == 1).sum())
    segments = _segments(lens, cu, memory_units) if memory_units else []
    if segments:
        arrays["segments"] = np.asarray(segments, dtype=np.int32)
    facts = dict(num_tokens=int(cu[-1]), num_entries=len(items), num_single=singles, multi_rows=int(cu[-1]) - singles,
                 num_short=num_short, split=any(not s[3] & 4 for s in segments), order=order, starts=starts)
    return arrays, [a for a, _ in per_window], [c for _, c in per_window], facts


def ragged_step(seqs, windows, block_size, device, memory_units=0, latent=False) -> RaggedStep:
    """The step's device tensors: one copy per integer type, every tensor a 16-byte aligned slice of it.  ``latent``: the
    views of windows that are plain numbers are LatentSteps."""
    arrays, window_arrays, counts, facts = ragged_arrays(seqs, windows, block_size, memory_units, latent)
    named = [((None, k), a) for k, a in arrays.items()]
    for g, wa in enumerate(window_arrays):
        named += [((g, k), a) for k, a in wa.items()]
    placed = {}
    for np_dtype, torch_dtype in ((np.int32, torch.int32), (np.int64, torch.int64)):
        mine = [(key, a) for key, a in named if a.dtype == np_dtype]
        offsets, total = [], 0
        for _, a in mine:
            offsets.append(total)
            total += -(-a.size // 4) * 4
        host = torch.empty(max(total, 1), dtype=torch_dtype, pin_memory=device.type == "cuda")
        view = host.numpy()
        for (_, a), at in zip(mine, offsets):
            view[at:at + a.size] = a.reshape(-1)
        dev = host.to(device, non_blocking=True)
        for (key, a), at in zip(mine, offsets):
            placed[key] = dev[at:at + a.size].view(a.shape)
    views = [RingStep if isinstance(w, SlidingWindow) else LatentStep if latent else WindowStep for w in windows]
    ws = [views[g](**counts[g], **{k: placed[(g, k)] for k in wa}) for g, wa in enumerate(window_arrays)]
    return RaggedStep(windows=ws, **{k: placed[(None, k)] for k in arrays}, **facts)
