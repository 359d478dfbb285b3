"""What a mixer asks of the cache; a model's layers are grouped by equal needs."""
from dataclasses import dataclass
from typing import Optional, Tuple

import torch


@dataclass(frozen=True)
class KVNeed:
    """Keys and values of every position, or of the last `window` positions only; `keep_first` (with a window): and
    of the sequence's first so many. `values` False:
    rows of keys alone (a mixer whose values are a part of its key rows, as an attention over one
    shared latent a token has them); the pool is then half the size and the view's `v` is None."""
    kv_heads: int
    head_dim: int
    window: Optional[int] = None
    values: bool = True
    keep_first: int = 0


@dataclass(frozen=True)
class StateNeed:
    """State of a fixed size for each sequence (zero when the sequence starts)."""
    shape: Tuple[int, ...]
    dtype: torch.dtype = torch.float32
