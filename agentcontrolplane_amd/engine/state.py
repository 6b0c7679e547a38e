"""Slots of recurrent state.

Layers with a recurrence keep a fixed-size state per sequence instead of pages:
a slot in pools that the model allocates once (``allocate_state``).  A sequence
holds one slot from its admission until it finishes or is preempted; every
recurrent layer uses the same slot number, as every attention layer uses the same
block table.  A slot's contents always cover exactly the tokens that the block
manager counts for its sequence; a sequence's first chunk starts from zero, so a
slot is handed on without being cleared.
"""
from __future__ import annotations

from typing import Dict, List


class OutOfStateSlotsError(RuntimeError):
    pass


class StateSlots:
    def __init__(self, num_slots: int):
        self.num_slots = num_slots
        self._free: List[int] = list(range(num_slots - 1, -1, -1))
        self._slots: Dict[int, int] = {}

    @property
    def free(self) -> int:
        return len(self._free)

    def has(self, seq_id: int) -> bool:
        return seq_id in self._slots

    def slot(self, seq_id: int) -> int:
        return self._slots[seq_id]

    def acquire(self, seq_id: int) -> int:
        if seq_id in self._slots:
            raise KeyError(f"seq {seq_id} already holds a state slot")
        if not self._free:
            raise OutOfStateSlotsError(
                f"seq {seq_id}: all {self.num_slots} state slots are in use"
            )
        self._slots[seq_id] = self._free.pop()
        return self._slots[seq_id]

    def release(self, seq_id: int) -> None:
        slot = self._slots.pop(seq_id, None)
        if slot is not None:
            self._free.append(slot)

    def transfer(self, new_seq_id: int, old_seq_id: int) -> None:
        """The new sequence goes on from the old one's state."""
        if new_seq_id in self._slots:
            raise KeyError(f"seq {new_seq_id} already holds a state slot")
        self._slots[new_seq_id] = self._slots.pop(old_seq_id)
