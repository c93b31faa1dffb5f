"""MuiZufadraModel / MuiZufadraForCausalLM: a decoder of windowed attention with sinks and of gated delta-rule layers in
any order, dense feed-forwards, norms on the sublayers' outputs only, an fp32 residual stream and a bigram embedding.

The mechanisms live beside their relatives (modules/attention/hybridattention.py, modules/recurrent/channeldelta.py,
modules/gateupdownmlp.py, modules/embedding.py, modules/decoder/sandwichdecoder.py, modules/kvcache/hybridcache.py), the
step, loading and what generate() expects in ../native.py; this file puts the modules together and names the tensors
of a checkpoint."""
from typing import Iterator, Tuple

import torch
import torch.nn as nn

from .... import hybrid_ops
from ....engineconfig import MuiEngineConfig
from ...attention.hybridattention import MuiHybridAttention, MuiHybridAttentionConfig
from ...decoder.sandwichdecoder import MuiSandwichDecoderLayer
from ...embedding import MuiBigramEmbedding, MuiEmbedding
from ...gateupdownmlp import MuiGateUpDownMLP
from ...recurrent.channeldelta import MuiChannelDelta
from ..native import MuiNativeForCausalLM, MuiNativeModel
from .config import MuiZufadraConfig


def _mixer_tensors(mixer) -> Iterator[Tuple[str, torch.Tensor]]:
    """(name in the checkpoint, the (slice of a) parameter it fills) of a mixer."""
    w, starts = mixer.proj.linear.weight, mixer.proj.slice_starts
    if isinstance(mixer, MuiHybridAttention):
        for name, lo, hi in zip("qkvg", starts, mixer.proj.slice_ends):
            yield name, w[lo:hi]
        yield "q.norm", mixer.q_norm
        yield "k.norm", mixer.k_norm
    else:
        c = mixer.config
        qk, v = c.kv_heads * c.dim, c.heads * c.vdim
        rows = {"q": qk, "k": qk, "v": v, "a1": c.decay_rank, "g1": c.gate_rank, "b": c.heads}
        for (name, n), lo in zip(rows.items(), starts):
            yield name, w[lo:lo + n]
        for name, lo, n in (("q", 0, qk), ("k", qk, qk), ("v", 2 * qk, v)):
            yield name + ".conv", mixer.conv[lo:lo + n]
        yield "a2", mixer.decay_up[:, :c.decay_rank]
        yield "dt_bias", mixer.dt_bias
        yield "A_log", mixer.a_log
        yield "g2", mixer.gate_up[:, :c.gate_rank]
        yield "norm", mixer.head_norm
    yield "o", mixer.out_proj.weight


class MuiZufadraModel(MuiNativeModel):
    def __init__(self, engine_config: MuiEngineConfig, config: MuiZufadraConfig, device=None, dtype=None):
        super().__init__(engine_config, config)
        hid, eps, bg = config.hidden_size, config.rms_norm_eps, config.bigram
        kw = dict(device=device, dtype=dtype)
        self.logit_scale = config.logit_scale
        if bg is None:
            self.embed_tokens = MuiEmbedding(engine_config, config.vocab_size, hid, **kw)
        else:
            self.embed_tokens = MuiBigramEmbedding(engine_config, config.vocab_size, hid, config.embedding_scale, bg.buckets,
                                                   bg.mul_prev, bg.mul_cur, **kw)
        layers = []
        for i, layer in enumerate(config.layers):
            kind = MuiHybridAttention if isinstance(layer.mixer, MuiHybridAttentionConfig) else MuiChannelDelta
            mixer = kind(engine_config, hid, layer.mixer, i, eps, **kw)
            mlp = None if layer.ff is None else MuiGateUpDownMLP(engine_config, hid, layer.ff, nn.SiLU(), bias=True, **kw)
            layers.append(MuiSandwichDecoderLayer(engine_config, hid, mixer, mlp, eps, pre_norms=False,
                                                  branch_scale=config.residual_mult, **kw))
        self.layers = nn.ModuleList(layers)
        self.norm = self.final_norm(**kw)
        self.finalize_init()

    @property
    def front(self):
        return self.embed_tokens if isinstance(self.embed_tokens, MuiBigramEmbedding) else None

    def start(self, input_ids, inputs_embeds, cache, cache_position):
        if self.front is None:
            rows = self.embed_tokens(input_ids) if inputs_embeds is None else inputs_embeds
            return hybrid_ops.residual_norm(None, rows, None, None, 0.0, y_scale=self.config.embedding_scale, emit=True)
        if input_ids is None:
            raise ValueError("a bigram embedding needs the token ids")
        return self.embed_tokens(input_ids, cache, cache_position)


class MuiZufadraForCausalLM(MuiNativeForCausalLM):
    model_class = MuiZufadraModel
    config_class = MuiZufadraConfig

    def checkpoint_tensors(self) -> Iterator[Tuple[str, torch.Tensor]]:
        m = self.model
        yield "embed", m.embed_tokens.weight
        if m.front is not None:
            yield "bigram", m.embed_tokens.bigram
        for i, layer in enumerate(m.layers):
            p = f"l{i}."
            yield p + "norm1", layer.post_mixer_norm.weight
            for name, t in _mixer_tensors(layer.mixer):
                yield p + "mix." + name, t
            if layer.mlp is not None:
                yield p + "norm2", layer.post_mlp_norm.weight
                for name in ("gate", "up", "down"):
                    part = getattr(layer.mlp, name + "_proj")
                    yield f"{p}mlp.{name}", part.weight
                    yield f"{p}mlp.{name}.b", part.bias
        yield "final.norm", m.norm.weight
        yield "head", self.lm_head.weight
