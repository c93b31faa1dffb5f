"""MuiMoE: mixture of small clamped-SwiGLU experts with identity experts. Kernels: csrc/moe.hip.

Router in 32 bits: scores are a softmax over all outputs, the choice uses scores + correction, the weights
are the chosen scores as they are. The result is handed on as a MoEOutput: its weighted sum is taken by the
kernel that adds it to the residual stream."""
from dataclasses import dataclass

import torch
import torch.nn as nn

from .. import hybrid_ops
from ..engineconfig import MuiEngineConfig
from .module import MuiModule


@dataclass
class MuiMoEConfig:
    experts: int   # with matrices
    identity: int  # without: their output is the block's input
    top: int
    ff: int
    limit: float   # gate clamped from above, up from both sides

    def __post_init__(self):
        if self.experts < 1 or not 1 <= self.top <= self.experts + self.identity:
            raise ValueError(f"a router cannot choose {self.top} of {self.experts} + {self.identity} experts")


class MuiMoE(MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, hidden: int, config: MuiMoEConfig, device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        c = self.config = config
        kw = dict(device=device, dtype=dtype)
        outputs = c.experts + c.identity

        def weight(*shape):
            return nn.Parameter(torch.empty(shape, **kw), requires_grad=False)

        self.router = weight(outputs, hidden)
        self.correction = nn.Parameter(torch.zeros(outputs, **kw), requires_grad=False)
        self.gate_proj = weight(c.experts, c.ff, hidden)
        self.up_proj = weight(c.experts, c.ff, hidden)
        self.down_proj = weight(c.experts, hidden, c.ff)

    def forward(self, h: torch.Tensor) -> hybrid_ops.MoEOutput:
        c = self.config
        x = h.reshape(-1, h.shape[-1])
        tile = hybrid_ops.moe_tile_pairs(x.dtype, x.shape[0], c.top, c.experts, x.shape[1], c.ff)
        logits = hybrid_ops.linear_f32(x, self.router)
        expert, weight, pairs, tiles = hybrid_ops.moe_route(logits, self.correction, c.experts, c.top, tile)
        out = hybrid_ops.moe_experts(x, self.gate_proj, self.up_proj, self.down_proj, c.limit, expert, pairs, tiles, tile)
        return hybrid_ops.MoEOutput(out, x, expert, weight, c.experts)
