"""Sequence slots of a batch model: which request sits in which slot and how many tokens it has there."""
from __future__ import annotations


class SlotMap:
    """Requests by id over `capacity` slots. ``begin`` takes the lowest free slot, ``advance`` returns the position a
    request's next tokens start at, ``end`` gives the slot back (its next owner starts over at position 0)."""

    def __init__(self, capacity: int):
        self.capacity = capacity
        self._free = list(range(capacity))
        self._live: dict = {}  # id -> [slot, length]

    def __len__(self) -> int:
        return len(self._live)

    def __contains__(self, rid) -> bool:
        return rid in self._live

    def begin(self, rid) -> int:
        if rid in self._live:
            raise ValueError(f"request {rid!r} is live already")
        if not self._free:
            raise RuntimeError("no free sequence slot")
        slot = min(self._free)
        self._free.remove(slot)
        self._live[rid] = [slot, 0]
        return slot

    def advance(self, rid, n: int) -> tuple[int, int]:
        """(slot, position of the first of the next n tokens)."""
        e = self._live[rid]
        start = e[1]
        e[1] += n
        return e[0], start

    def end(self, rid) -> None:
        slot, _ = self._live.pop(rid)
        self._free.append(slot)
