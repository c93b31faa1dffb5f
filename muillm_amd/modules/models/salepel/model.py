"""MuiSalepelModel / MuiSalepelForCausalLM: a decoder of latent-attention and mLSTM layers with
mixture-of-experts feed-forwards, norms on both sides of every sublayer and an fp32 residual stream.

The mechanisms live beside their relatives (modules/attention/latentattention.py, modules/recurrent/mlstm.py,
modules/moe.py, modules/decoder/sandwichdecoder.py, modules/kvcache/hybridcache.py), the step, loading and what
generate() expects in ../native.py; this file puts the modules together and names the tensors of a checkpoint."""
from typing import Iterator, Tuple

import torch
import torch.nn as nn

from .... import hybrid_ops
from ....engineconfig import MuiEngineConfig
from ...attention.latentattention import MuiLatentAttention, MuiLatentAttentionConfig
from ...decoder.sandwichdecoder import MuiSandwichDecoderLayer
from ...embedding import MuiEmbedding
from ...moe import MuiMoE
from ...recurrent.mlstm import MuiMLstm
from ..native import MuiNativeForCausalLM, MuiNativeModel
from .config import MuiSalepelConfig


def _mixer_tensors(mixer) -> Iterator[Tuple[str, torch.Tensor]]:
    """(name in the checkpoint, the (slice of a) parameter it fills) of a mixer."""
    if isinstance(mixer, MuiLatentAttention):
        c, down = mixer.config, mixer.down.linear.weight
        yield "dq", down[:c.q_rank]
        yield "dq.norm", mixer.q_norm
        if mixer.own_rows:
            yield "dkv", down[c.q_rank:]
            yield "dkv.norm", mixer.kv_norm
        yield "uq", mixer.up_q.weight
        yield "uk", mixer.up_kv.weight[:c.heads * c.dim]
        yield "uv", mixer.up_kv.weight[c.heads * c.dim:]
    else:
        h, w = mixer.config.heads, mixer.proj.linear.weight
        for name, lo, hi in zip("qkvg", mixer.proj.slice_starts, mixer.proj.slice_ends):
            yield name, w[lo:hi]
        yield "norm", mixer.head_norm
        yield "i", mixer.gate_weight[:h]
        yield "i.b", mixer.gate_bias[:h]
        yield "f", mixer.gate_weight[h:]
        yield "f.b", mixer.gate_bias[h:]
    yield "o", mixer.out_proj.weight


class MuiSalepelModel(MuiNativeModel):
    def __init__(self, engine_config: MuiEngineConfig, config: MuiSalepelConfig, device=None, dtype=None):
        super().__init__(engine_config, config)
        hid, eps = config.hidden_size, config.rms_norm_eps
        kw = dict(device=device, dtype=dtype)
        self.embed_tokens = MuiEmbedding(engine_config, config.vocab_size, hid, **kw)
        layers = []
        for i, layer in enumerate(config.layers):
            kind = MuiLatentAttention if isinstance(layer.mixer, MuiLatentAttentionConfig) else MuiMLstm
            mixer = kind(engine_config, hid, layer.mixer, i, eps, **kw)
            mlp = None if layer.mlp is None else MuiMoE(engine_config, hid, layer.mlp, **kw)
            layers.append(MuiSandwichDecoderLayer(engine_config, hid, mixer, mlp, eps, **kw))
        self.layers = nn.ModuleList(layers)
        self.norm = self.final_norm(**kw)
        self.finalize_init()

    def start(self, input_ids, inputs_embeds, cache, cache_position):
        rows = self.embed_tokens(input_ids) if inputs_embeds is None else inputs_embeds
        return hybrid_ops.residual_norm(None, rows, None, self.layers[0].pre_mixer_norm.weight, self.config.rms_norm_eps,
                                        y_scale=self.config.embedding_scale)


class MuiSalepelForCausalLM(MuiNativeForCausalLM):
    model_class = MuiSalepelModel
    config_class = MuiSalepelConfig

    def checkpoint_tensors(self) -> Iterator[Tuple[str, torch.Tensor]]:
        m = self.model
        yield "embed", m.embed_tokens.weight
        for i, layer in enumerate(m.layers):
            p = f"l{i}."
            yield p + "norm1", layer.pre_mixer_norm.weight
            yield p + "norm1b", layer.post_mixer_norm.weight
            for name, t in _mixer_tensors(layer.mixer):
                yield p + "mix." + name, t
            if layer.mlp is not None:
                yield p + "norm2", layer.pre_mlp_norm.weight
                yield p + "norm2b", layer.post_mlp_norm.weight
                for e in range(layer.mlp.config.experts):
                    yield f"{p}mlp.e{e}.gate", layer.mlp.gate_proj[e]
                    yield f"{p}mlp.e{e}.up", layer.mlp.up_proj[e]
                    yield f"{p}mlp.e{e}.down", layer.mlp.down_proj[e]
                yield p + "mlp.router", layer.mlp.router
                yield p + "mlp.correction", layer.mlp.correction
        yield "final.norm", m.norm.weight
        yield "head", self.lm_head.weight
