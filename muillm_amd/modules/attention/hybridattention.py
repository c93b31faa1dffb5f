"""MuiHybridAttention: grouped-query attention of native designs: one projection q | k | v | output gate, RMS norms over
the whole of q and of k, rotary positions on the first dimensions of every head (pairs 2 i, 2 i + 1), capped scores, a
sliding window that keeps the first tokens of a sequence visible. Kernels: csrc/hybrid_attention.hip."""
from dataclasses import dataclass
from typing import Any, Dict, Optional

import torch
import torch.nn as nn

from ... import hybrid_ops
from ...engineconfig import MuiEngineConfig
from ..kvcache.hybridcache import MuiHybridCache, MuiKeyValueState
from ..linear import MuiLinear
from ..module import MuiModule
from ..multilinear import MuiMultiLinear
from .rotaryembedding import compute_rope_inv_freq


@dataclass
class MuiHybridAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[Dict[str, Any]] = None  # as compute_rope_inv_freq takes it for "llama3"
    softcap: float = 0.0  # 0: scores as they are
    window: int = 0       # keys a query sees, itself included (0: all)
    keep_first: int = 0   # first tokens that stay visible beyond the window
    qk_norm: bool = True
    gated: bool = True

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} query heads over {self.kv_heads} key/value heads")
        if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
            raise ValueError(f"cannot rotate {self.rot_dims} of {self.dim} dimensions")
        if self.window < 0 or self.keep_first < 0 or self.softcap < 0:
            raise ValueError("window, keep_first and softcap cannot be negative")


class MuiHybridAttention(MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, hidden: int, config: MuiHybridAttentionConfig, layer_idx: int, eps: float,
                 device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        c = self.config = config
        self.layer_idx, self.eps = layer_idx, eps
        kw = dict(device=device, dtype=dtype)
        nq, nk = c.heads * c.dim, c.kv_heads * c.dim
        outs = [nq, nk, c.kv_heads * c.vdim] + ([c.heads * c.vdim] if c.gated else [])
        self.proj = MuiMultiLinear(engine_config, hidden, outs, bias=False, **kw)
        self.q_norm = nn.Parameter(torch.ones(nq, **kw), requires_grad=False) if c.qk_norm else None
        self.k_norm = nn.Parameter(torch.ones(nk, **kw), requires_grad=False) if c.qk_norm else None
        self.out_proj = MuiLinear(engine_config, c.heads * c.vdim, hidden, bias=False, **kw)
        inv_freq = torch.zeros(0, dtype=torch.float64)
        if c.rot_dims:
            inv_freq, _ = compute_rope_inv_freq("llama3" if c.rot_scaling else None, c.rot_base, c.rot_dims, c.rot_scaling,
                                                dtype=torch.float64)
        self.register_buffer("inv_freq", inv_freq.to(device), persistent=False)

    def new_state(self, batch: int, capacity: int, device, dtype) -> MuiKeyValueState:
        return MuiKeyValueState(batch, capacity, self.config.kv_heads, self.config.dim, self.config.vdim, device, dtype)

    def forward(self, h: torch.Tensor, cache: MuiHybridCache, cache_position: torch.Tensor) -> torch.Tensor:
        """h [B, T, hidden] -> [B, T, hidden]; the tokens' rows go to slots cache_position."""
        c, state = self.config, cache.layers[self.layer_idx]
        proj = self.proj.linear(h)
        q = hybrid_ops.hybrid_prepare(proj, c.heads, c.kv_heads, c.dim, c.vdim, self.q_norm, self.k_norm, self.eps, self.inv_freq,
                                      cache_position, cache.row_start, state.k, state.v)
        gate = proj[..., self.proj.slice_starts[3]:] if c.gated else None
        return self.out_proj(hybrid_ops.hybrid_attention(q, state.k, state.v, gate, cache_position, cache.row_start, c.heads,
                                                         c.kv_heads, c.scale, c.softcap, c.window, c.keep_first))
