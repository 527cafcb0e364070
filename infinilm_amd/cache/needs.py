"""What a mixer asks of the cache manager for one cache entry: one of the needs below, or a tuple of them (the
mixer's view of the cache is then the tuple of their views)."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

import torch


@dataclass(frozen=True)
class PagedKV:
    """Keys and values of every token, in pages.  window > 0: only the last `window` positions
    before (and including) a query are ever read, so older pages can be given back; keep_first > 0:
    the sequence's first `keep_first` positions are read as well, so the pages that hold them stay.
    chunks: a query at position p is only ever read against positions from p - p % size on, for the sizes listed (every layer
    that reads these keys by its own): pages before the earliest of them can be given back.  A window or chunks, not both."""
    num_kv_heads: int
    head_dim: int
    window: int = 0
    keep_first: int = 0
    chunks: Tuple[int, ...] = ()

    def __post_init__(self):
        if self.chunks and (self.window > 0 or self.keep_first or min(self.chunks) <= 0):
            raise ValueError(f"keys kept by chunks of {self.chunks} positions: positive sizes, and no window or kept first positions beside them")


@dataclass(frozen=True)
class FixedState:
    """State of fixed size per request (one row of a pool per request); row 0 is all zeros and
    is what a request starts from."""
    shape: Tuple[int, ...]
    dtype: Optional[torch.dtype] = None  # None: float32
