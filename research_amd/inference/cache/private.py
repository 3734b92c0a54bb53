"""Block allocator without sharing, with a slot for recurrent state per sequence.

Behind the same protocol as the prefix-sharing allocators (cache/protocol.py).
A layer with recurrent state has one state per sequence, the one after its last
token; blocks shared by prefix would bring keys without the state that goes
with them, so sequences of such models own all their blocks.  A sequence holds
its blocks and its slot from ``allocate`` to ``deallocate``; both are handed out
again, oldest first, to other sequences.  Owns no device memory.
"""

from __future__ import annotations

from collections import deque
from typing import Deque, Dict, List, Optional, Tuple


class PrivateKVCache:
    def __init__(self, num_blocks: int, block_size: int = 16, num_state_slots: int = 0) -> None:
        assert num_blocks > 0
        assert block_size > 0
        self.block_size = block_size
        self.num_blocks = num_blocks
        self.num_state_slots = num_state_slots
        self.free_block_ids: Deque[int] = deque(range(num_blocks))
        self.free_state_slots: Deque[int] = deque(range(num_state_slots))
        self._blocks: Dict[int, List[int]] = {}
        self._tokens: Dict[int, int] = {}
        self._slots: Dict[int, int] = {}

    # -- queries ---------------------------------------------------------
    def num_free_blocks(self) -> int:
        return len(self.free_block_ids)

    def _blocks_for(self, num_tokens: int) -> int:
        return -(-num_tokens // self.block_size)

    def can_allocate(self, num_tokens: int) -> bool:
        return (self._blocks_for(num_tokens) <= len(self.free_block_ids)
                and (self.num_state_slots == 0 or len(self.free_state_slots) > 0))

    def get_block_ids(self, seq_id: int) -> Tuple[int, ...]:
        return tuple(self._blocks.get(seq_id, ()))

    def get_cached_tokens(self, seq_id: int) -> int:
        return 0

    def num_tokens(self, seq_id: int) -> int:
        """Tokens the sequence's blocks were taken for."""
        return self._tokens.get(seq_id, 0)

    def state_slot(self, seq_id: int) -> int:
        return self._slots.get(seq_id, -1)

    # -- lifecycle -------------------------------------------------------
    def allocate(self, seq_id: int, token_ids: List[int]) -> Tuple[int, ...]:
        """Blocks for ``token_ids`` and a state slot; raises without a trace when either is short."""
        assert seq_id not in self._blocks, f"Sequence {seq_id} already allocated"
        if self.num_state_slots and not self.free_state_slots:
            raise RuntimeError(f"No free state slot for sequence {seq_id}")
        need = self._blocks_for(len(token_ids))
        if need > len(self.free_block_ids):
            raise RuntimeError(f"No free blocks for sequence {seq_id}: needs {need}, {len(self.free_block_ids)} free")
        self._blocks[seq_id] = [self.free_block_ids.popleft() for _ in range(need)]
        self._tokens[seq_id] = len(token_ids)
        if self.num_state_slots:
            self._slots[seq_id] = self.free_state_slots.popleft()
        return self.get_block_ids(seq_id)

    def extend(self, seq_id: int, num_tokens: int) -> None:
        """Room for ``num_tokens`` more tokens; raises without a trace when the pool is short."""
        total = self._tokens[seq_id] + num_tokens
        need = self._blocks_for(total) - len(self._blocks[seq_id])
        if need > len(self.free_block_ids):
            raise RuntimeError("No free blocks for token append")
        for _ in range(need):
            self._blocks[seq_id].append(self.free_block_ids.popleft())
        self._tokens[seq_id] = total

    def append_token(self, seq_id: int, token_id: int) -> Optional[int]:
        """Record one more token; returns the new block id when the token starts a new block, else None."""
        before = len(self._blocks[seq_id])
        self.extend(seq_id, 1)
        return self._blocks[seq_id][-1] if len(self._blocks[seq_id]) > before else None

    def deallocate(self, seq_id: int) -> None:
        blocks = self._blocks.pop(seq_id, None)
        if blocks is None:
            return
        del self._tokens[seq_id]
        self.free_block_ids.extend(reversed(blocks))
        slot = self._slots.pop(seq_id, None)
        if slot is not None:
            self.free_state_slots.append(slot)
