"""Slots for what a sequence keeps besides its cache blocks: the recurrent state of layers that have one.  A slot holds a
sequence's state in every such layer; it is taken with the sequence's first block and given back with its last.  Nothing is
cleared: a sequence whose first token has position 0 starts from zeros whatever the slot holds (csrc/ssm.hip)."""
from __future__ import annotations

from collections import deque

__all__ = ["StateSlots"]


class StateSlots:
    def __init__(self, num_slots: int) -> None:
        if num_slots <= 0:
            raise ValueError(f"a pool of state slots needs at least one slot (num_slots={num_slots})")
        self.num_slots = num_slots
        self._free: deque[int] = deque(range(num_slots))

    @property
    def num_free(self) -> int:
        return len(self._free)

    def take(self, sequence) -> None:
        """Give the sequence a slot (it keeps the one it has)."""
        if sequence.state_slot >= 0:
            return
        if not self._free:
            raise RuntimeError(f"no free state slots: all {self.num_slots} are held by live sequences")
        sequence.state_slot = self._free.popleft()

    def release(self, sequence) -> None:
        if sequence.state_slot >= 0:
            self._free.append(sequence.state_slot)
            sequence.state_slot = -1
