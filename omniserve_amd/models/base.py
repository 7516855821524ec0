"""What the engine asks of a model."""
from __future__ import annotations

from typing import List, Optional, Tuple

import torch


class EngineModel:
    """Subclasses set vocab, dtype and device and implement `from_pretrained` and `forward`; the rest are defaults."""

    page_size = 64                       # tokens per cache page
    attn_rows = 128                      # query rows of one prefill attention tile
    min_segments = 1                     # parts of a portion from which on recurrent layers run them in parallel
    chunk_rows = 0                       # tokens per chunk of recurrent layers that work in chunks (0: there are none)
    expand_pages = 0                     # most context pages a layer expands into keys and values at once (0: none does)
    dtypes: Tuple[torch.dtype, ...] = () # number formats the model runs in, its default first
    capturable = True                    # single-token steps may be captured in HIP graphs (empty places: position < 0)
    vocab: int
    dtype: torch.dtype
    device: torch.device

    @classmethod
    def from_pretrained(cls, model_dir: str, config: dict, dtype=None, device="cuda") -> "EngineModel":
        raise NotImplementedError

    def forward(self, batch, cache) -> Optional[torch.Tensor]:
        """Runs engine.batch.DeviceBatch from the cache and state earlier steps left; returns the logits of the wanted rows,
        f32 [rows, vocab], or None when there are none."""
        raise NotImplementedError

    # ---- what the cache holds for a sequence ----
    def kv_shapes(self) -> List[Tuple[int, int, int]]:
        """(kv heads, key size, value size) of every layer that keeps keys and values (a latent row: 1, its size, 0)"""
        return []

    def state_shapes(self) -> List[Tuple[int, ...]]:
        """One sequence's part of every f32 tensor that recurrent layers keep: a state (heads, key size, value size), a ring of a
        convolution's inputs (rows, channels)"""
        return []

    def page_pools(self, num_pages: int, device):
        """One (K, V) pool pair per layer of kv_shapes.  Zeros: places of a page past its sequence's end are multiplied with a
        probability of zero and must be finite."""
        return [tuple(torch.zeros((num_pages, g, self.page_size, d), dtype=self.dtype, device=device) for d in (dk, dv))
                for g, dk, dv in self.kv_shapes()]

    def window(self) -> Optional[int]:
        """The newest token and how many before it some layer may still read; None: all of them."""
        return None

    def linear_workgroups(self) -> int:
        """Fewest workgroups one segment of a prompt gives to a recurrent layer (0: there is none)."""
        return 0

    def greedy(self, logits: torch.Tensor) -> torch.Tensor:
        return logits.argmax(dim=-1)
