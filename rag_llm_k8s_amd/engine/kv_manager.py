"""Paged KV-cache block manager (64-token blocks).

Uses the native C++ allocator from ``_ragk_rt`` when built (O(1) free-list ops in C++,
called once per scheduled sequence per step); the Python class below has the identical
interface and is the fallback / test oracle.

Block 0 is reserved as a scratch block: padded (dummy) rows of a captured decode graph
write their K/V there, so graph replay never touches a live sequence's cache.
"""
from __future__ import annotations

BLOCK = 64


class PyBlockManager:
    def __init__(self, num_blocks: int, reserve_scratch: bool = True):
        if num_blocks < 2:
            raise ValueError("need at least 2 KV blocks")
        self.num_blocks = num_blocks
        self.scratch = 0 if reserve_scratch else -1
        first = 1 if reserve_scratch else 0
        self._free = list(range(num_blocks - 1, first - 1, -1))
        self.tables = {}

    def free_blocks(self) -> int:
        return len(self._free)

    def blocks_needed(self, seq_id, n_tokens) -> int:
        have = len(self.tables.get(seq_id, ()))
        need = -(-n_tokens // BLOCK)
        return max(0, need - have)

    def can_allocate(self, seq_id, n_tokens) -> bool:
        return self.blocks_needed(seq_id, n_tokens) <= len(self._free)

    def ensure(self, seq_id, n_tokens):
        """Make sure the sequence owns blocks for positions [0, n_tokens). Returns the table."""
        t = self.tables.setdefault(seq_id, [])
        need = -(-n_tokens // BLOCK)
        if need - len(t) > len(self._free):
            raise MemoryError("KV cache exhausted")
        while len(t) < need:
            t.append(self._free.pop())
        return t

    def table(self, seq_id):
        return self.tables.get(seq_id, [])

    def slot(self, seq_id, pos) -> int:
        return self.tables[seq_id][pos // BLOCK] * BLOCK + pos % BLOCK

    def free(self, seq_id):
        t = self.tables.pop(seq_id, None)
        if t:
            self._free.extend(reversed(t))


class StateSlots:
    """Recurrent-state slots: one per live sequence, whatever its length. Slot 0 is scratch (padded rows of a
    captured decode graph). A slot is not cleared when it changes hands: a sequence's first tokens start
    from zero state inside the kernels, which know them by their position."""

    def __init__(self, num_slots: int):
        if num_slots < 2:
            raise ValueError("need at least 2 state slots")
        self.num_slots = num_slots
        self._free = list(range(num_slots - 1, 0, -1))
        self.owner = {}

    def available(self) -> int:
        return len(self._free)

    def ensure(self, seq_id) -> int:
        if seq_id not in self.owner:
            if not self._free:
                raise MemoryError("recurrent-state slots exhausted")
            self.owner[seq_id] = self._free.pop()
        return self.owner[seq_id]

    def slot(self, seq_id) -> int:
        return self.owner[seq_id]

    def free(self, seq_id):
        s = self.owner.pop(seq_id, None)
        if s is not None:
            self._free.append(s)


class SequenceCache:
    """What one live sequence holds: its K/V blocks and, for recurrent models, its state slot."""

    def __init__(self, blocks, slots=None):
        self.blocks, self.slots = blocks, slots

    def can_allocate(self, seq_id, n_tokens) -> bool:
        if self.slots is not None and seq_id not in self.slots.owner and not self.slots.available():
            return False
        return self.blocks.can_allocate(seq_id, n_tokens)

    def ensure(self, seq_id, n_tokens):
        if self.slots is not None:
            self.slots.ensure(seq_id)
        return self.blocks.ensure(seq_id, n_tokens)

    def state(self, seq_id) -> int:
        return 0 if self.slots is None else self.slots.slot(seq_id)

    def table(self, seq_id):
        return self.blocks.table(seq_id)

    def slot(self, seq_id, pos) -> int:
        return self.blocks.slot(seq_id, pos)

    def free_blocks(self) -> int:
        return self.blocks.free_blocks()

    def free(self, seq_id):
        if self.slots is not None:
            self.slots.free(seq_id)
        self.blocks.free(seq_id)


def make_block_manager(num_blocks: int):
    try:
        from ..runtime import native_rt

        rt = native_rt()
        if rt is not None:
            return rt.BlockManager(num_blocks, True)
    except Exception:
        pass
    return PyBlockManager(num_blocks)
