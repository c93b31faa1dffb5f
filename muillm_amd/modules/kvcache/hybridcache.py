"""Cache of a decoder whose layers keep different things: rows per token (keys and values, or a latent row), a
recurrent state, or nothing of their own (a layer that attends over another layer's rows).

Every mixer makes its own layer state (`new_state`); the cache holds them in layer order and gives the
decode loop what MuiStaticCache gives it: capacity (a power of two, grown on demand), the count of seen
tokens, reset for the next sequence. Rows of a batch advance together; a left-padded row starts at
row_start[b], keys in front of it are never seen and recurrent states pass over it."""
from typing import List, Optional, Sequence

import torch

from .cache_utils import MuiCache, _next_pow2


class MuiRowState:
    """Tensors [B, capacity, width] with one row per token."""

    def __init__(self, batch: int, capacity: int, widths: Sequence[int], device, dtype):
        self.rows = [torch.zeros((batch, capacity, w), dtype=dtype, device=device) for w in widths]

    def tensors(self) -> List[torch.Tensor]:
        return list(self.rows)

    def recurrent(self) -> List[torch.Tensor]:
        return []

    def grow(self, capacity: int) -> None:
        for i, old in enumerate(self.rows):
            self.rows[i] = torch.zeros((old.shape[0], capacity, old.shape[2]), dtype=old.dtype, device=old.device)
            self.rows[i][:, :old.shape[1]] = old

    def reset(self) -> None:
        pass  # rows behind the count of seen tokens are never read before they are written again


class MuiLatentState(MuiRowState):
    """Latent rows c [B, capacity, kv_rank] and rotated key parts r [B, capacity, rot] of one layer."""

    def __init__(self, batch: int, capacity: int, kv_rank: int, rot_dim: int, device, dtype):
        super().__init__(batch, capacity, (kv_rank, rot_dim), device, dtype)

    @property
    def c(self) -> torch.Tensor:
        return self.rows[0]

    @property
    def r(self) -> torch.Tensor:
        return self.rows[1]


class MuiKeyValueState(MuiRowState):
    """Keys [B, capacity, kv_heads * dim] (rotated) and values [B, capacity, kv_heads * vdim] of one layer."""

    def __init__(self, batch: int, capacity: int, kv_heads: int, dim: int, vdim: int, device, dtype):
        super().__init__(batch, capacity, (kv_heads * dim, kv_heads * vdim), device, dtype)

    @property
    def k(self) -> torch.Tensor:
        return self.rows[0]

    @property
    def v(self) -> torch.Tensor:
        return self.rows[1]


class MuiRecurrentState:
    """Tensors of fixed size that every token rewrites (memories in fp32, the last inputs of a short convolution,
    the last token); a fresh sequence starts from zero."""

    def __init__(self, *tensors: torch.Tensor):
        self.values = tuple(tensors)

    def tensors(self) -> List[torch.Tensor]:
        return list(self.values)

    def recurrent(self) -> List[torch.Tensor]:
        return list(self.values)

    def grow(self, capacity: int) -> None:
        pass

    def reset(self) -> None:
        for t in self.values:
            t.zero_()


class MuiHybridCache(MuiCache):
    def __init__(self, engine_config, mixers, max_batch_size: int, max_cache_len: int, device, dtype: torch.dtype, front=None):
        """front: what stands in front of the layers and keeps a state of its own (an embedding that looks back)."""
        self.engine_config = engine_config
        self.max_batch_size = max_batch_size
        self.max_cache_len = _next_pow2(max_cache_len)
        self.device, self.dtype = device, dtype
        self.layers = [m.new_state(max_batch_size, self.max_cache_len, device, dtype) for m in mixers]
        self.front = None if front is None else front.new_state(max_batch_size, self.max_cache_len, device, dtype)
        self.row_start: Optional[torch.Tensor] = None
        self._seen_tokens = 0
        # True while a captured decode step runs: positions are read from device memory only
        self.device_length_mode = False
        self.cpp_module = None

    def __len__(self):
        return len(self.layers)

    def _states(self):
        return [s for s in self.layers + [self.front] if s is not None]

    def tensors(self) -> List[torch.Tensor]:
        out = [t for s in self._states() for t in s.tensors()]
        return out if self.row_start is None else out + [self.row_start]

    def step_state(self) -> List[torch.Tensor]:
        return [t for s in self._states() for t in s.recurrent()]

    def set_row_start(self, row_start: Optional[torch.Tensor]) -> None:
        """First real slot of every row; kept in one buffer so that a captured step stays valid."""
        if row_start is None or self.row_start is None or self.row_start.shape != row_start.shape:
            self.row_start = None if row_start is None else row_start.to(torch.int64).contiguous()
        else:
            self.row_start.copy_(row_start)

    def get_seq_length(self, layer_idx: Optional[int] = 0) -> int:
        return self._seen_tokens

    def get_max_length(self) -> Optional[int]:
        return self.max_cache_len

    def get_max_cache_shape(self) -> Optional[int]:
        return self.max_cache_len

    def grow_cache(self, capacity: int, max_capacity: Optional[int] = None) -> None:
        capacity = _next_pow2(capacity)
        if max_capacity is not None:
            capacity = min(capacity, max_capacity)
        if self.max_cache_len >= capacity:
            return
        for s in self._states():
            s.grow(capacity)
        self.max_cache_len = capacity

    def reset(self) -> None:
        for s in self._states():
            s.reset()
        self._seen_tokens = 0
        self.row_start = None


class MuiCachePool:
    """Caches by request: one is taken at a request's first tokens, given back at its end, and serves
    a later request after reset()."""

    def __init__(self, new_cache):
        self._new_cache = new_cache
        self._free: List[MuiCache] = []
        self._live = {}

    def get(self, request) -> MuiCache:
        cache = self._live.get(request)
        if cache is None:
            if self._free:
                cache = self._free.pop()
                cache.reset()
            else:
                cache = self._new_cache()
            self._live[request] = cache
        return cache

    def release(self, request) -> None:
        cache = self._live.pop(request, None)
        if cache is not None:
            self._free.append(cache)
