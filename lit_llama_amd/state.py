"""Slots of per-sequence state.

A slot is what one live sequence owns in every layer: its ring of cached keys / values, its recurrent state, the last inputs of its
convolutions.  Every such tensor is one device allocation with the slot as its first dimension; the manager below only deals out the
slot numbers and grows the allocations.
"""
from __future__ import annotations

from typing import Callable, List

import torch


class SlotManager:
    """Deals out slots 0 .. n - 1; `grow(n)` of the owner reallocates the tensors when all are taken."""

    def __init__(self, grow: Callable[[int], None]):
        self._grow = grow
        self.capacity = 0
        self._free: List[int] = []
        self.live = 0

    def reserve(self, n: int) -> None:
        """Room for n slots at least (a batch that starts together grows the allocations once)."""
        if n > self.capacity:
            self._grow(n)
            self._free.extend(range(self.capacity, n))
            self.capacity = n

    def acquire(self) -> int:
        if not self._free:
            self.reserve(max(1, 2 * self.capacity))
        self.live += 1
        self._free.sort()
        return self._free.pop(0)

    def release(self, slot: int) -> None:
        if not 0 <= slot < self.capacity or slot in self._free:
            raise ValueError(f"slot {slot} is not live")
        self._free.append(slot)
        self.live -= 1


def grown(old: "torch.Tensor | None", shape, dtype, device) -> torch.Tensor:
    """A zeroed [slots, ...] tensor that keeps the rows of `old`."""
    new = torch.zeros(shape, dtype=dtype, device=device)
    if old is not None:
        new[: old.shape[0]].copy_(old)
    return new
