"""Fixed-size states of recurrent mixers, one slot per sequence.

A sequence's recurrent state does not grow with it, so a cache row owns one slot for as long as the
cache lives and there is nothing to page.  Rows reach their slots through a map on the device:
moving a sequence to another row exchanges two entries of the map and no state, like the pages of
its keys.  A slot is not cleared when a sequence ends: the kernels start a sequence at position 0
from zero whatever its slot holds.

Per recurrent layer:
  state[i]  [rows, heads, keys, ld]   float32, ld = value size rounded up to 16 (padding stays zero)
  ring[i]   [rows, taps, channels]    the convolution's latest inputs, position p at p % taps (None: no convolution)
"""

from __future__ import annotations

import torch

StateShape = tuple[int, int, int, int, int]  # heads, keys, values, taps (0: no convolution), channels


class StatePool:
    def __init__(self, shapes: list[StateShape], rows: int, device, dtype):
        self.shapes, self.rows = list(shapes), rows
        self.state = [torch.zeros(rows, h, d, -(-e // 16) * 16, dtype=torch.float32, device=device)
                      for h, d, e, _, _ in shapes]
        self.ring = [torch.zeros(rows, taps, ch, dtype=dtype, device=device) if taps else None
                     for _, _, _, taps, ch in shapes]
        self.map = torch.arange(rows, dtype=torch.int32, device=device)
        self.slot = list(range(rows))

    def __len__(self) -> int:
        return len(self.state)

    def tensors(self) -> list[torch.Tensor]:
        return self.state + [t for t in self.ring if t is not None]

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.tensors())

    def swap(self, a: int, b: int) -> None:
        """The sequences of two rows change places."""
        if a != b and self.state:
            self.slot[a], self.slot[b] = self.slot[b], self.slot[a]
            self.map.copy_(torch.tensor(self.slot, dtype=torch.int32))

    def read(self, rows) -> list[torch.Tensor]:
        """Detached copies of the rows' states."""
        idx = torch.tensor([self.slot[r] for r in rows], dtype=torch.int64, device=self.map.device)
        return [t[idx] for t in self.tensors()]

    def write(self, rows, saved: list[torch.Tensor]) -> None:
        idx = torch.tensor([self.slot[r] for r in rows], dtype=torch.int64, device=self.map.device)
        for t, s in zip(self.tensors(), saved):
            t[idx] = s
