"""What sequences hold on the GPU between steps: pages of the attention layers' keys and values, and one slot of every recurrent
layer's state.

One page number stands for 64 tokens in every attention layer (each layer has its own K and V pool, [pages][kv heads][64][size]);
one slot number for a sequence's state in every recurrent layer ([slots][heads][dk][dv] and rings of convolution inputs, f32).  A slot needs no clearing: a
sequence's first step starts its state from zero."""
from __future__ import annotations

from typing import List, Optional

import numpy as np
import torch


class OutOfPages(RuntimeError):
    pass


class Sequence:
    """One sequence's place in the cache."""

    def __init__(self, slot: int):
        self.slot = slot
        self.length = 0                                  # tokens whose keys, values and state are stored
        self.table = np.full((8,), -1, dtype=np.int32)   # page of every 64 tokens; -1: given back or not yet taken
        self.pages = 0                                   # entries of the table in use
        self.released = 0                                # leading entries given back

    def append(self, page: int) -> None:
        if self.pages == len(self.table):
            self.table = np.concatenate([self.table, np.full_like(self.table, -1)])
        self.table[self.pages] = page
        self.pages += 1


class Cache:
    def __init__(self, model, num_pages: int, num_slots: int, device):
        self.page_size, self.num_pages, self.num_slots = model.page_size, num_pages, num_slots
        self.window: Optional[int] = model.window()
        self.paged = bool(model.kv_shapes())
        if not self.paged:
            num_pages = 0
        self.kv = model.page_pools(num_pages, device)
        self.state = [torch.zeros((num_slots, *shape), dtype=torch.float32, device=device) for shape in model.state_shapes()]
        self._pages: List[int] = list(range(num_pages))[::-1]
        self._slots: List[int] = list(range(num_slots))[::-1]

    # ---- slots ----
    def free_slots(self) -> int:
        return len(self._slots)

    def open(self) -> Sequence:
        if not self._slots:
            raise RuntimeError("no state slot is free (%d sequences are live)" % self.num_slots)
        return Sequence(self._slots.pop())

    def close(self, seq: Sequence) -> None:
        self._give_back(seq, seq.pages)
        seq.pages = 0
        self._slots.append(seq.slot)
        seq.slot = -1

    # ---- pages ----
    def free_pages(self) -> int:
        return len(self._pages)

    def missing_pages(self, seq: Sequence, tokens: int) -> int:
        """Pages to take before `tokens` more can be stored."""
        return max(0, -(-(seq.length + tokens) // self.page_size) - seq.pages) if self.paged else 0

    def reserve(self, seq: Sequence, tokens: int) -> None:
        need = self.missing_pages(seq, tokens)
        if need > len(self._pages):
            raise OutOfPages("%d pages needed, %d free" % (need, len(self._pages)))
        for _ in range(need):
            seq.append(self._pages.pop())

    def advance(self, seq: Sequence, tokens: int) -> None:
        """`tokens` more are stored; pages that no window reaches any more are given back."""
        seq.length += tokens
        if self.window is not None:
            self._give_back(seq, max(0, seq.length - self.window + 1) // self.page_size)

    def _give_back(self, seq: Sequence, upto: int) -> None:
        for i in range(seq.released, min(upto, seq.pages)):
            self._pages.append(int(seq.table[i]))
            seq.table[i] = -1
        seq.released = max(seq.released, min(upto, seq.pages))
