"""MuiLatentAttention: attention whose keys and values are linear maps of one cached latent row per token
plus a rotated key part shared by all heads, with queries through a latent of their own and a sliding
window. Kernels: csrc/latent_attention.hip.

A layer may read another layer's cached rows (kv_source) instead of keeping its own: it then has no key /
value down projection, only its own up projections, queries and window."""
from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn as nn

from ... import _lib, hybrid_ops
from ...engineconfig import MuiEngineConfig
from ..kvcache.hybridcache import MuiHybridCache, MuiLatentState
from ..linear import MuiLinear
from ..module import MuiModule
from ..multilinear import MuiMultiLinear


@dataclass
class MuiLatentAttentionConfig:
    heads: int
    dim: int        # unrotated query / key dimensions per head
    rot_dim: int    # rotated ones
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    window: int = 0            # keys a query sees, itself included (0: all)
    kv_source: Optional[int] = None  # layer whose latent rows this one reads

    def __post_init__(self):
        if self.rot_dim % 2:
            raise ValueError("rot_dim must be even")


class MuiLatentAttention(MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, hidden: int, config: MuiLatentAttentionConfig, layer_idx: int,
                 eps: float, device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        c = self.config = config
        self.layer_idx, self.eps = layer_idx, eps
        self.own_rows = c.kv_source is None
        kw = dict(device=device, dtype=dtype)
        outs = [c.q_rank] + ([c.kv_rank, c.rot_dim] if self.own_rows else [])
        self.down = MuiMultiLinear(engine_config, hidden, outs, bias=False, **kw)
        self.q_norm = nn.Parameter(torch.ones(c.q_rank, **kw), requires_grad=False)
        self.kv_norm = nn.Parameter(torch.ones(c.kv_rank, **kw), requires_grad=False) if self.own_rows else None
        self.up_q = MuiLinear(engine_config, c.q_rank, c.heads * (c.dim + c.rot_dim), bias=False, **kw)
        # rows of the key map, then rows of the value map
        self.up_kv = MuiLinear(engine_config, c.kv_rank, c.heads * (c.dim + c.vdim), bias=False, **kw)
        self.out_proj = MuiLinear(engine_config, c.heads * c.vdim, hidden, bias=False, **kw)
        half = torch.arange(c.rot_dim // 2, dtype=torch.float64)
        self.register_buffer("inv_freq", (float(c.rot_base) ** (-2.0 * half / c.rot_dim)).to(device), persistent=False)

    def new_state(self, batch: int, capacity: int, device, dtype) -> Optional[MuiLatentState]:
        if not self.own_rows:
            return None
        return MuiLatentState(batch, capacity, self.config.kv_rank, self.config.rot_dim, device, dtype)

    def forward(self, h: torch.Tensor, cache: MuiHybridCache, cache_position: torch.Tensor) -> torch.Tensor:
        """h [B, T, hidden] (normed) -> [B, T, hidden]; the tokens' rows go to slots cache_position."""
        c = self.config
        b, t = h.shape[0], h.shape[1]
        state: MuiLatentState = cache.layers[self.layer_idx if self.own_rows else c.kv_source]
        q_latent, cos_sin = hybrid_ops.latent_prepare(self.down.linear(h), self.q_norm, self.kv_norm, self.eps, self.inv_freq,
                                                      cache_position, cache.row_start, state.c, state.r)
        q = self.up_q(q_latent)
        route = hybrid_ops.latent_route(h.dtype, t, c.heads, c.dim, c.rot_dim, c.vdim, c.kv_rank)
        w = self.up_kv.weight
        if route == _lib.MUI_LATENT_PREFILL:
            # keys and values of everything the tokens can see, once per call
            q_first = cache.get_seq_length()
            kv_first = max(0, q_first - c.window + 1) if c.window else 0
            kv = [self.up_kv(state.c[i, kv_first:q_first + t]) for i in range(b)]
            o = hybrid_ops.latent_prefill_attention(q, cos_sin, kv, kv_first, state.r, cache.row_start, q_first, c.heads, c.dim,
                                                    c.vdim, c.scale, c.window)
        else:
            o = hybrid_ops.latent_attention(q, cos_sin, w[:c.heads * c.dim], w[c.heads * c.dim:], state.c, state.r,
                                            cache_position, cache.row_start, c.heads, c.dim, c.vdim, c.scale, c.window, route)
        return self.out_proj(o)
