"""MuiSalepelModel / MuiSalepelForCausalLM: a decoder of latent-attention and mLSTM layers with
mixture-of-experts feed-forwards, norms on both sides of every sublayer and an fp32 residual stream.

The mechanisms live beside their relatives (modules/attention/latentattention.py, modules/recurrent/mlstm.py,
modules/moe.py, modules/decoder/sandwichdecoder.py, modules/kvcache/hybridcache.py); this file names the
tensors of a checkpoint and offers what the decode loop and generate() expect of a causal LM."""
import os
from typing import Callable, Dict, Iterator, Optional, Tuple, Union

import torch
import torch.nn as nn

from .... import muillm_ext
from ....engineconfig import MuiEngineConfig
from ...attention.latentattention import MuiLatentAttention, MuiLatentAttentionConfig
from ...decoder.sandwichdecoder import MuiSandwichDecoderLayer, run_layers
from ...embedding import MuiEmbedding
from ...kvcache.hybridcache import MuiHybridCache
from ...linear import MuiLinear
from ...module import MuiModule
from ...moe import MuiMoE
from ...norm.rmsnorm import MuiRMSNorm
from ...recurrent.mlstm import MuiMLstm
from ..generation import MuiGenerationMixin
from ..llama.model import MuiCausalLMOutput, MuiModelOutput
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


class MuiSalepelModel(MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, config: MuiSalepelConfig, device=None, dtype=None):
        super().__init__(engine_config=engine_config)
        self.config = config
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
        self.norm = MuiRMSNorm(engine_config, hid, eps=eps, **kw)
        self.finalize_init()

    def finalize_init(self):
        self.mdevice = self.embed_tokens.weight.device
        self.mdtype = self.embed_tokens.weight.dtype

    def create_cache(self, batch_size: int, seq_len: int) -> MuiHybridCache:
        return MuiHybridCache(self.engine_config, [l.mixer for l in self.layers], batch_size, seq_len, self.mdevice, self.mdtype)

    def forward(self, input_ids: Optional[torch.LongTensor] = None, attention_mask: Optional[torch.Tensor] = None,
                past_key_values: Optional[MuiHybridCache] = None, inputs_embeds: Optional[torch.Tensor] = None,
                output_hidden_states: Optional[bool] = None, cache_position: Optional[torch.LongTensor] = None) -> MuiModelOutput:
        """inputs_embeds are rows of the embedding table (the embedding scale is applied here).
        attention_mask [B, T] of 0 / 1 marks left padding of the tokens an empty cache starts with.
        hidden_states: the fp32 residual stream after every layer."""
        if (input_ids is None) == (inputs_embeds is None):
            raise ValueError("specify either input_ids or inputs_embeds")
        rows = self.embed_tokens(input_ids) if inputs_embeds is None else inputs_embeds
        b, t = rows.shape[0], rows.shape[1]
        cache = past_key_values
        if cache is None:
            cache = self.create_cache(b, t)
        elif not isinstance(cache, MuiHybridCache):
            raise ValueError("the layers of this model need a MuiHybridCache")
        past = cache.get_seq_length()
        if b > cache.max_batch_size:
            raise ValueError(f"batch {b} exceeds the cache's max_batch_size {cache.max_batch_size}")
        if not cache.device_length_mode:
            cache.grow_cache(past + t)
        if attention_mask is not None and past == 0:
            cache.set_row_start(self._left_padding(attention_mask))
        if cache_position is None:
            cache_position = torch.arange(past, past + t, device=rows.device)
        collect = [] if output_hidden_states else None
        h = run_layers(self.layers, rows, self.config.embedding_scale, self.norm, self.config.rms_norm_eps, cache,
                       cache_position, collect)
        cache.set_seen_tokens(past + t)
        return MuiModelOutput(last_hidden_state=h, past_key_values=cache,
                              hidden_states=None if collect is None else tuple(collect))

    @staticmethod
    def _left_padding(attention_mask: torch.Tensor) -> Optional[torch.Tensor]:
        am = attention_mask.to(torch.int64)
        if bool((am == 1).all()):
            return None
        pads = (am == 0).sum(-1)
        if am.dim() != 2 or bool((am.cumsum(-1).eq(0).sum(-1) != pads).any()) or bool((pads >= am.shape[1]).any()):
            raise ValueError("padding must be on the left of at least one real token")
        return pads


class MuiSalepelForCausalLM(MuiGenerationMixin, MuiModule):
    def __init__(self, engine_config: MuiEngineConfig, config: MuiSalepelConfig, device=None, dtype=None):
        MuiModule.__init__(self, engine_config=engine_config)
        self.config = config
        self.model = MuiSalepelModel(engine_config, config, device=device, dtype=dtype)
        self.lm_head = MuiLinear(engine_config, config.hidden_size, config.vocab_size, bias=False, device=device, dtype=dtype)
        self._graph_decoder = None

    # ---- weights -----------------------------------------------------------------------------
    def checkpoint_tensors(self) -> Iterator[Tuple[str, torch.Tensor]]:
        """(name, parameter or slice of one that it fills), every tensor of a checkpoint once."""
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

    @torch.no_grad()
    def load_tensors(self, names, get: Callable[[str], torch.Tensor]) -> None:
        """Fill every parameter from get(name); names: what the checkpoint holds (nothing may be left over)."""
        left = set(names)
        for name, dst in self.checkpoint_tensors():
            if name not in left:
                raise ValueError(f"the checkpoint has no tensor {name}")
            src = get(name)
            if tuple(src.shape) != tuple(dst.shape):
                raise ValueError(f"{name} has shape {tuple(src.shape)}, expected {tuple(dst.shape)}")
            dst.copy_(src)
            left.discard(name)
        if left:
            raise ValueError(f"the checkpoint holds tensors this model has no place for: {sorted(left)[:8]}")

    @staticmethod
    def _new(engine_config, config, dtype, device) -> "MuiSalepelForCausalLM":
        lm = MuiSalepelForCausalLM(engine_config or MuiEngineConfig(), config, device=device, dtype=dtype)
        lm.eval()
        lm.requires_grad_(False)
        return lm

    def _finalize(self) -> "MuiSalepelForCausalLM":
        from ....engine import _finalize_module
        _finalize_module(self)
        self.muillm_config = self.engine_config
        return self

    @staticmethod
    def from_tensors(config: MuiSalepelConfig, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda",
                     engine_config: Optional[MuiEngineConfig] = None) -> "MuiSalepelForCausalLM":
        lm = MuiSalepelForCausalLM._new(engine_config, config, dtype, device)
        lm.load_tensors(tensors.keys(), tensors.__getitem__)
        return lm._finalize()

    @staticmethod
    def from_pretrained(path: str, dtype=torch.bfloat16, device="cuda",
                        engine_config: Optional[MuiEngineConfig] = None) -> "MuiSalepelForCausalLM":
        """A folder with config.json and model.safetensors."""
        from safetensors import safe_open

        lm = MuiSalepelForCausalLM._new(engine_config, MuiSalepelConfig.from_pretrained(path), dtype, device)
        with safe_open(os.path.join(path, "model.safetensors"), framework="pt", device="cpu") as f:
            lm.load_tensors(f.keys(), f.get_tensor)
        return lm._finalize()

    @staticmethod
    def from_config(engine_config: Optional[MuiEngineConfig], config: MuiSalepelConfig, dtype=torch.bfloat16, device="cuda",
                    seed: int = 0, init_std: float = 0.02) -> "MuiSalepelForCausalLM":
        """Randomly initialised (matrices ~ N(0, init_std), norm gains 1, biases 0), for benchmarks."""
        lm = MuiSalepelForCausalLM._new(engine_config, config, dtype, device)
        gen = torch.Generator(device=device)
        gen.manual_seed(seed)
        with torch.no_grad():
            for _, t in lm.checkpoint_tensors():
                if t.dim() == 2:
                    t.normal_(0.0, init_std, generator=gen)
        return lm._finalize()

    # ---- what the decode loop asks of a causal LM -----------------------------------------------
    pads_in_cache = True  # left padding is a property of the cache; no additive mask travels with a step

    def create_cache(self, batch_size: int, seq_len: int) -> MuiHybridCache:
        return self.model.create_cache(batch_size, seq_len)

    def max_positions(self) -> Optional[int]:
        return None

    def get_input_embeddings(self):
        return self.model.embed_tokens

    def get_output_embeddings(self):
        return self.lm_head

    @torch.no_grad()
    def forward(self, input_ids: Optional[torch.LongTensor] = None, attention_mask: Optional[torch.Tensor] = None,
                position_ids: Optional[torch.LongTensor] = None, past_key_values: Optional[MuiHybridCache] = None,
                inputs_embeds: Optional[torch.Tensor] = None, use_cache: Optional[bool] = None,
                output_hidden_states: Optional[bool] = None, cache_position: Optional[torch.LongTensor] = None,
                all_ones_mask: Optional[bool] = None, num_logits_to_keep: int = 0,
                logits_positions: Union[None, list, torch.Tensor] = None, float_logits: bool = True) -> MuiCausalLMOutput:
        """One step over the tokens given, from the state the cache holds. position_ids are accepted for the
        decode loop's sake: a token's position is its slot minus its row's first slot. logits_positions: the
        places among the tokens whose logits are wanted (default all; num_logits_to_keep: the last ones)."""
        out = self.model(input_ids=input_ids, attention_mask=attention_mask, past_key_values=past_key_values,
                         inputs_embeds=inputs_embeds, output_hidden_states=output_hidden_states, cache_position=cache_position)
        h = out.last_hidden_state
        if logits_positions is not None:
            h = h[:, logits_positions, :]
        elif num_logits_to_keep:
            h = h[:, -num_logits_to_keep:, :]
        logits = None
        if h.shape[1]:
            logits = self.lm_head(h.contiguous())
            if float_logits:
                logits = logits.float()
        return MuiCausalLMOutput(logits=logits, past_key_values=out.past_key_values, hidden_states=out.hidden_states)
