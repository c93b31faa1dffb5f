"""MuiMLstm: a matrix memory per head with exponential input gate, forget gate and running maximum (the
mLSTM layer of xLSTM), head-wise normalised output behind a sigmoid gate. Kernels: csrc/mlstm.hip."""
from dataclasses import dataclass

import torch
import torch.nn as nn

from ... import hybrid_ops
from ...engineconfig import MuiEngineConfig
from ..kvcache.hybridcache import MuiHybridCache, MuiRecurrentState
from ..linear import MuiLinear
from ..module import MuiModule
from ..multilinear import MuiMultiLinear


@dataclass
class MuiMLstmConfig:
    heads: int
    dim: int    # query / key size per head
    vdim: int
    gate_cap: float


class MuiMLstm(MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, hidden: int, config: MuiMLstmConfig, layer_idx: int, eps: float,
                 device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        c = self.config = config
        self.layer_idx, self.eps = layer_idx, eps
        kw = dict(device=device, dtype=dtype)
        qk, v = c.heads * c.dim, c.heads * c.vdim
        self.proj = MuiMultiLinear(engine_config, hidden, [qk, qk, v, v], bias=False, **kw)  # q | k | v | output gate
        # input gate rows, then forget gate rows: their pre-activations stay in 32 bits
        self.gate_weight = nn.Parameter(torch.zeros((2 * c.heads, hidden), **kw), requires_grad=False)
        self.gate_bias = nn.Parameter(torch.zeros(2 * c.heads, **kw), requires_grad=False)
        self.head_norm = nn.Parameter(torch.ones(v, **kw), requires_grad=False)
        self.out_proj = MuiLinear(engine_config, v, hidden, bias=False, **kw)

    def new_state(self, batch: int, capacity: int, device, dtype) -> MuiRecurrentState:
        c, slices = self.config, hybrid_ops.mlstm_slices(self.config.vdim)
        return MuiRecurrentState(torch.zeros((batch, c.heads, c.dim, c.vdim), dtype=torch.float32, device=device),
                                 torch.zeros((batch, c.heads, slices, c.dim), dtype=torch.float32, device=device),
                                 torch.zeros((batch, c.heads, slices), dtype=torch.float32, device=device))

    def forward(self, h: torch.Tensor, cache: MuiHybridCache, cache_position: torch.Tensor) -> torch.Tensor:
        c = self.config
        b, t = h.shape[0], h.shape[1]
        q, k, v, gate = self.proj(h)
        gates = hybrid_ops.linear_f32(h, self.gate_weight, self.gate_bias).view(b, t, 2 * c.heads)
        o = hybrid_ops.mlstm(q, k, v, gates, cache.layers[self.layer_idx].values, c.dim ** -0.5, c.gate_cap, cache_position,
                             cache.row_start, c.heads)
        return self.out_proj(hybrid_ops.mlstm_output(o, self.head_norm, gate, self.eps))
