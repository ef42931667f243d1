"""Slots of per-sequence recurrent state, the constant-size companion of the paged KV cache.

A running sequence owns one slot from admission to release (a swapped-out one keeps it: its blocks move, its state does
not).  A group that will fork (n > 1 sequences from one prompt) reserves the slots of its children when it is admitted, so
that a fork never fails; a fork's state copy is handed to the next step through `take_copies`.  A slot's content is never
cleared: a sequence's first step starts from zeros by its length, whatever the slot held before."""
from typing import Dict, List, Tuple


class StateSlotManager:

    def __init__(self, num_slots: int) -> None:
        if num_slots < 1:
            raise ValueError("at least one state slot is needed")
        self.num_slots = num_slots
        self._free: List[int] = list(range(num_slots - 1, -1, -1))
        self._slot: Dict[int, int] = {}
        self._reserved: Dict[int, List[int]] = {}  # prompt sequence -> slots set aside for its forks
        self._copies: List[Tuple[int, int]] = []

    def num_free(self) -> int:
        return len(self._free)

    def can_allocate(self, n: int = 1) -> bool:
        return n <= len(self._free)

    def allocate(self, seq_id: int, n: int = 1) -> int:
        """A slot for `seq_id`, and n - 1 more set aside for sequences forked from it."""
        if seq_id in self._slot:
            raise ValueError(f"sequence {seq_id} has a state slot already")
        if not self.can_allocate(max(1, n)):
            raise RuntimeError("no free state slot")
        self._slot[seq_id] = self._free.pop()
        if n > 1:
            self._reserved[seq_id] = [self._free.pop() for _ in range(n - 1)]
        return self._slot[seq_id]

    def slot_of(self, seq_id: int) -> int:
        return self._slot[seq_id]

    def fork(self, parent_id: int, child_id: int) -> None:
        reserved = self._reserved.get(parent_id)
        if not reserved and not self._free:
            raise RuntimeError("no free state slot")
        slot = reserved.pop() if reserved else self._free.pop()
        self._slot[child_id] = slot
        self._copies.append((self._slot[parent_id], slot))

    def free(self, seq_id: int) -> None:
        slot = self._slot.pop(seq_id, None)
        if slot is None:
            return
        self._copies = [c for c in self._copies if slot != c[1]]  # (a copy FROM it still finds the state in place)
        self._free.append(slot)
        self._free.extend(self._reserved.pop(seq_id, ()))

    def take_copies(self) -> List[Tuple[int, int]]:
        out, self._copies = self._copies, []
        return out
