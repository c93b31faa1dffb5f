"""Decoder layers with a norm before and after each sublayer around an fp32 residual stream:
x <- x + post_norm(mixer(pre_norm(x))), then the same with an optional feed-forward.

A sublayer's post norm, the residual sum and the next sublayer's pre norm are one kernel
(hybrid_ops.residual_norm), so a layer hands its last sublayer's output on unjoined: run_layers joins it
together with the norm of whatever comes next."""
from typing import List, Optional

import torch
import torch.nn as nn

from ... import hybrid_ops
from ...engineconfig import MuiEngineConfig
from ..module import MuiModule
from ..norm.rmsnorm import MuiRMSNorm


class MuiSandwichDecoderLayer(MuiModule):
    """mixer: a module with forward(h, cache, cache_position) and new_state(...); mlp: a module with
    forward(h), or None for a layer without feed-forward."""

    def __init__(self, engine_config: MuiEngineConfig, hidden: int, mixer: MuiModule, mlp: Optional[MuiModule], eps: float,
                 device=None, dtype=None):
        super().__init__(engine_config=engine_config)

        def norm():
            return MuiRMSNorm(engine_config, hidden, eps=eps, device=device, dtype=dtype)

        self.mixer, self.mlp = mixer, mlp
        self.pre_mixer_norm, self.post_mixer_norm = norm(), norm()
        self.pre_mlp_norm, self.post_mlp_norm = (norm(), norm()) if mlp is not None else (None, None)


def run_layers(layers: List[MuiSandwichDecoderLayer], inputs: torch.Tensor, input_scale: float, final_norm: MuiRMSNorm, eps: float,
               cache, cache_position: torch.Tensor, collect: Optional[list] = None) -> torch.Tensor:
    """inputs [B, T, hidden] (embedding rows, scaled here) through all layers; returns the final norm's
    output. collect: a list that receives the fp32 residual stream after every layer."""
    join = hybrid_ops.residual_norm
    x, h = join(None, inputs, None, layers[0].pre_mixer_norm.weight, eps, y_scale=input_scale)
    for i, layer in enumerate(layers):
        last = i + 1 == len(layers)
        following = final_norm.weight if last else layers[i + 1].pre_mixer_norm.weight
        y = layer.mixer(h, cache, cache_position)
        if layer.mlp is not None:
            x, h = join(x, y, layer.post_mixer_norm.weight, layer.pre_mlp_norm.weight, eps)
            y = layer.mlp(h)
            x, h = join(x, y, layer.post_mlp_norm.weight, following, eps)
        else:
            x, h = join(x, y, layer.post_mixer_norm.weight, following, eps)
        h = h.reshape(inputs.shape)
        if collect is not None:
            collect.append(x.clone())
    return h
