"""What a sequence holds on the device between steps, and who may hold it.

CacheManager owns two pools and the tensors behind them:
  * pages: blocks of `block_size` token rows, listed per sequence in its block table.  Layers with a per-token cache ask
    for their storage with paged(); all of them are addressed by the same block tables.
  * state slots: one per live sequence.  Layers that carry a fixed amount of state from token to token ask for theirs with
    per_slot() and index it by the sequence's slot.
A slot or page is never cleared when it changes hands: a portion that starts at position 0 ignores the slot's state, and
attention reads only rows below the sequence's length.
"""
from __future__ import annotations

from collections import deque

import torch


class CacheManager:
    def __init__(self, num_blocks: int, block_size: int, num_slots: int, device, pages: bool = True, slots: bool = False):
        self.block_size, self.num_blocks, self.num_slots = block_size, num_blocks, num_slots
        self.device = device
        self.uses_pages, self.uses_slots = pages, slots
        self.free_blocks = deque(range(num_blocks))
        self.free_slots = deque(range(num_slots))

    # ------------------------------------------------------------------ storage
    def paged(self, *row_shape, dtype=torch.bfloat16, lead=()):
        """Zeroed storage [*lead, num_blocks, block_size, *row_shape]."""
        return torch.zeros((*lead, self.num_blocks, self.block_size, *row_shape), dtype=dtype, device=self.device)

    def per_slot(self, *shape, dtype=torch.float32):
        """Zeroed storage [num_slots, *shape]."""
        return torch.zeros((self.num_slots, *shape), dtype=dtype, device=self.device)

    # ------------------------------------------------------------------ who holds what
    def blocks_needed(self, n_tokens: int) -> int:
        return (n_tokens + self.block_size - 1) // self.block_size if self.uses_pages else 0

    def can_hold(self, seq, n_tokens: int) -> bool:
        """Whether seq could grow to n_tokens now."""
        if self.uses_slots and seq.state_slot < 0 and not self.free_slots:
            return False
        return self.blocks_needed(n_tokens) - len(seq.block_table) <= len(self.free_blocks)

    def hold(self, seq, n_tokens: int) -> None:
        """Gives seq the pages for n_tokens tokens and, if the model keeps state, a slot."""
        if len(seq.block_table) * self.block_size >= n_tokens and (not self.uses_slots or seq.state_slot >= 0):
            return      # the usual decode step
        if not self.can_hold(seq, n_tokens):
            raise RuntimeError("KV cache exhausted: this engine does not preempt; raise num_blocks or the number of state slots")
        if self.uses_slots and seq.state_slot < 0:
            seq.state_slot = self.free_slots.popleft()
        for _ in range(self.blocks_needed(n_tokens) - len(seq.block_table)):
            seq.block_table.append(self.free_blocks.popleft())

    def release(self, seq) -> None:
        self.free_blocks.extend(seq.block_table)
        seq.block_table = []
        if seq.state_slot >= 0:
            self.free_slots.append(seq.state_slot)
            seq.state_slot = -1
