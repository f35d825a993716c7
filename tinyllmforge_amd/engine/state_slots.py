"""Slots of the recurrent state: one per live sequence, taken at admission and given back at the end or at preemption.
A slot is not cleared in between: the kernels start from a zero state at position 0."""
from __future__ import annotations

from collections import deque

from .sequence import Sequence


class StateSlots:
    def __init__(self, num_slots: int):
        assert num_slots > 0
        self.num_slots = num_slots
        self.free: deque[int] = deque(range(num_slots))

    def can_acquire(self) -> bool:
        return bool(self.free)

    def acquire(self, seq: Sequence):
        assert seq.state_slot < 0
        seq.state_slot = self.free.popleft()

    def release(self, seq: Sequence):
        if seq.state_slot >= 0:
            self.free.append(seq.state_slot)
            seq.state_slot = -1
