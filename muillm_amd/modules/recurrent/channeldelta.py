"""MuiChannelDelta: gated delta rule with one decay per head and key channel. Queries, keys and values pass short
causal convolutions; decays and the output gate come from low-rank projections. Kernels: csrc/channel_delta.hip."""
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
class MuiChannelDeltaConfig:
    heads: int
    kv_heads: int    # query / key heads
    dim: int         # query / key size per head
    vdim: int
    taps: int        # of the convolutions
    decay_rank: int
    gate_rank: int

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} value heads over {self.kv_heads} query/key heads")
        if self.taps < 1:
            raise ValueError("a convolution needs a tap")


def _up8(n: int) -> int:
    return (n + 7) // 8 * 8


class MuiChannelDelta(MuiModule):
    """Everything that reads h is one projection q | k | v | a1 | g1 | b. The low-rank parts and b are padded with zero
    rows (and a2, g2 with zero columns) to multiples of eight, so that every part starts on a 16-byte boundary."""

    def __init__(self, engine_config: MuiEngineConfig, hidden: int, config: MuiChannelDeltaConfig, layer_idx: int, eps: float,
                 device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        c = self.config = config
        self.layer_idx, self.eps = layer_idx, eps
        kw = dict(device=device, dtype=dtype)
        qk, v, ra, rg = c.kv_heads * c.dim, c.heads * c.vdim, _up8(c.decay_rank), _up8(c.gate_rank)
        self.proj = MuiMultiLinear(engine_config, hidden, [qk, qk, v, ra, rg, _up8(c.heads)], bias=False, **kw)

        def weight(*shape, value=0.0):
            return nn.Parameter(torch.full(shape, value, **kw), requires_grad=False)

        with torch.no_grad():
            self.proj.linear.weight[2 * qk + v:].zero_()
        self.conv = weight(2 * qk + v, c.taps)
        self.decay_up = weight(c.heads * c.dim, ra)
        self.dt_bias = weight(c.heads * c.dim)
        self.a_log = weight(c.heads)
        self.gate_up = weight(v, rg)
        self.head_norm = weight(c.vdim, value=1.0)
        self.out_proj = MuiLinear(engine_config, v, hidden, bias=False, **kw)

    def layer(self) -> hybrid_ops.ChannelDelta:
        c = self.config
        return hybrid_ops.ChannelDelta(c.heads, c.kv_heads, c.dim, c.vdim, tuple(self.proj.slice_starts), self.conv, self.decay_up,
                                       self.dt_bias, self.a_log, self.gate_up, self.head_norm, self.eps)

    def new_state(self, batch: int, capacity: int, device, dtype) -> MuiRecurrentState:
        """The memory, and the convolutions' last inputs as a ring of rows by slot."""
        c, layer = self.config, self.layer()
        return MuiRecurrentState(torch.zeros((batch, c.heads, c.dim, c.vdim), dtype=torch.float32, device=device),
                                 torch.zeros((batch, layer.ring_rows, layer.channels), dtype=dtype, device=device))

    def forward(self, h: torch.Tensor, cache: MuiHybridCache, cache_position: torch.Tensor) -> torch.Tensor:
        memory, ring = cache.layers[self.layer_idx].values
        return self.out_proj(hybrid_ops.channel_delta(self.layer(), self.proj.linear(h), memory, ring, cache_position,
                                                      cache.row_start))
