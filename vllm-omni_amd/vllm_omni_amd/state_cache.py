"""Per-request recurrent state on the device: fixed-size slots beside the paged KV cache.

A layer with a recurrence (or a short convolution) keeps, per request, tensors whose size does not grow with the
sequence.  ``StateCache`` owns one slot per live request — rows of every such tensor — plus one scratch slot that padded
rows of a graph replay and graph warm-ups write to.  Slots are handed out when a request enters the batch and come back
when it finishes or is preempted (its tokens are then recomputed from position 0).  A slot is never cleared: the kernels
start from zeros for a request whose first token is position 0.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Sequence

import torch


@dataclass
class StateSpec:
    """One state tensor of one layer: ``shape`` per request."""

    shape: tuple[int, ...]
    dtype: torch.dtype

    @property
    def slot_bytes(self) -> int:
        n = 1
        for d in self.shape:
            n *= d
        return n * torch.empty(0, dtype=self.dtype).element_size()


class StateCache:
    def __init__(self, num_slots: int, device):
        if num_slots < 1:
            raise ValueError("a state cache needs at least one slot")
        self.num_slots = num_slots
        self.device = device
        self.scratch_slot = num_slots
        self._free = list(range(num_slots - 1, -1, -1))

    def allocate(self, specs: Sequence[StateSpec]) -> list[torch.Tensor]:
        """[num_slots + 1, *shape] per spec"""
        return [torch.zeros(self.num_slots + 1, *s.shape, dtype=s.dtype, device=self.device) for s in specs]

    @property
    def num_free(self) -> int:
        return len(self._free)

    def acquire(self) -> int:
        if not self._free:
            raise RuntimeError(f"all {self.num_slots} state slots are held by live requests")
        return self._free.pop()

    def release(self, slot: int) -> None:
        if not 0 <= slot < self.num_slots or slot in self._free:
            raise ValueError(f"state slot {slot} is not held")
        self._free.append(slot)
