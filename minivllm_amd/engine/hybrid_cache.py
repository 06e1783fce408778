"""Cache manager of models whose layers keep different things per sequence: blocks of keys and values for attention layers
(one block table per attention window, shared by all layers with that window) and one slot of recurrent state.

A window of ``size`` is chunked attention: a token sees the earlier tokens of its own chunk only, so a sequence needs the
blocks of one chunk, and the next chunk overwrites them; token ``p`` lies at place ``p mod size`` of the table.  Window 0
keeps everything.  A sliding window (engine/windows.py) is a ring of places in the same way.  Blocks come from the block pools of ``BlockManager``; prefixes are not shared (a recurrent state
cannot be entered in the middle), so the pools are used without hashes.

Same interface towards the scheduler as ``BlockManager``."""
from __future__ import annotations

from collections import deque

from minivllm_amd.engine.block_manager import BlockManager
from minivllm_amd.engine.sequence import Sequence
from minivllm_amd.engine.windows import places


class HybridCacheManager:
    def __init__(self, windows: list, num_blocks: int, block_size: int, num_slots: int):
        self.windows = list(windows)
        self.block_size = block_size
        self.num_slots = num_slots
        self.pools = [BlockManager(num_blocks, block_size) for _ in self.windows]
        self.free_slots: deque[int] = deque(range(num_slots))

    def blocks_for(self, window, tokens: int) -> int:
        most = places(window)
        return -(-(min(tokens, most) if most else tokens) // self.block_size)

    def _missing(self, seq: Sequence) -> list[int]:
        held = seq.group_tables or [[] for _ in self.windows]
        return [max(self.blocks_for(w, len(seq)) - len(t), 0) for w, t in zip(self.windows, held)]

    def holds(self, tokens: int) -> bool:
        """Whether a sequence of that many tokens fits an empty cache."""
        return all(self.blocks_for(w, tokens) <= len(pool.blocks) for w, pool in zip(self.windows, self.pools))

    def can_append(self, seq: Sequence) -> bool:
        return all(n <= len(pool.free_block_ids) for n, pool in zip(self._missing(seq), self.pools))

    def can_allocate(self, seq: Sequence) -> bool:
        return bool(self.free_slots) and self.can_append(seq)

    def append(self, seq: Sequence) -> None:
        """Blocks for all of the sequence's tokens."""
        for table, pool, n in zip(seq.group_tables, self.pools, self._missing(seq)):
            table.extend(pool.take_block() for _ in range(n))

    def allocate(self, seq: Sequence) -> None:
        assert seq.state_slot < 0
        seq.state_slot = self.free_slots.popleft()
        seq.state_bank = 0
        seq.group_tables = [[] for _ in self.windows]
        self.append(seq)

    def deallocate(self, seq: Sequence) -> None:
        for table, pool in zip(seq.group_tables, self.pools):
            for block_id in reversed(table):
                pool.give_back(block_id)
        seq.group_tables = []
        if seq.state_slot >= 0:
            self.free_slots.append(seq.state_slot)
        seq.state_slot = -1
        seq.num_computed_tokens = 0

    def hash_deferred_blocks(self) -> None:
        """Nothing is shared, so nothing is hashed."""
