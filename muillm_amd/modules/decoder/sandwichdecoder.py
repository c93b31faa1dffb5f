"""Decoder layers with norms around each sublayer and an fp32 residual stream:
x <- x + m post_norm(mixer(pre_norm(x))), then the same with an optional feed-forward. The pre norms can be
left out: the sublayers then read x itself, rounded to the activations' type.

A sublayer's post norm, the residual sum and the next sublayer's input (its pre norm) are one kernel
(hybrid_ops.residual_norm), so a layer hands its last sublayer's output on unjoined: run_layers joins it
together with the input of whatever comes next."""
from typing import List, Optional

import torch
import torch.nn as nn

from ... import hybrid_ops
from ...engineconfig import MuiEngineConfig
from ..module import MuiModule
from ..norm.rmsnorm import MuiRMSNorm


class MuiSandwichDecoderLayer(MuiModule):
    """mixer: a module with forward(h, cache, cache_position) and new_state(...); mlp: a module with
    forward(h), or None for a layer without feed-forward. branch_scale: m."""

    def __init__(self, engine_config: MuiEngineConfig, hidden: int, mixer: MuiModule, mlp: Optional[MuiModule], eps: float,
                 device=None, dtype=None, pre_norms: bool = True, branch_scale: float = 1.0):
        super().__init__(engine_config=engine_config)

        def norm(there: bool):
            return MuiRMSNorm(engine_config, hidden, eps=eps, device=device, dtype=dtype) if there else None

        self.mixer, self.mlp, self.branch_scale = mixer, mlp, branch_scale
        self.pre_mixer_norm, self.post_mixer_norm = norm(pre_norms), norm(True)
        self.pre_mlp_norm, self.post_mlp_norm = norm(pre_norms and mlp is not None), norm(mlp is not None)


def run_layers(layers: List[MuiSandwichDecoderLayer], x: torch.Tensor, h: torch.Tensor, final_norm: MuiRMSNorm, eps: float,
               cache, cache_position: torch.Tensor, collect: Optional[list] = None, final_scale: float = 1.0) -> torch.Tensor:
    """x (fp32 residual stream) and h (the first sublayer's input) [B, T, hidden] through all layers; returns
    final_scale times the final norm's output. collect: a list that receives the residual stream after every layer."""
    shape = h.shape

    def join(x, y, post: MuiRMSNorm, m: float, following: Optional[MuiRMSNorm], scale: float = 1.0):
        return hybrid_ops.residual_norm(x, y, post.weight, None if following is None else following.weight, eps,
                                        branch_scale=m, next_scale=scale, emit=True)

    for i, layer in enumerate(layers):
        last, m = i + 1 == len(layers), layer.branch_scale
        following = (final_norm, final_scale) if last else (layers[i + 1].pre_mixer_norm,)
        y, post = layer.mixer(h, cache, cache_position), layer.post_mixer_norm
        if layer.mlp is not None:
            x, h = join(x, y, post, m, layer.pre_mlp_norm)
            y, post = layer.mlp(h), layer.post_mlp_norm
        x, h = join(x, y, post, m, *following)
        h = h.reshape(shape)
        if collect is not None:
            collect.append(x.clone())
    return h
