"""What the native designs (config.json with an `architecture` of this library) have in common: one step over
the layers from the state a MuiHybridCache holds, loading by tensor name, and what the decode loop and
generate() expect of a causal LM. A design adds its configuration, its modules and its tensor names."""
import os
from typing import Callable, Dict, Iterator, Optional, Tuple, Union

import torch
import torch.nn as nn

from ...engineconfig import MuiEngineConfig
from ..decoder.sandwichdecoder import run_layers
from ..kvcache.hybridcache import MuiHybridCache
from ..linear import MuiLinear
from ..module import MuiModule
from ..norm.rmsnorm import MuiRMSNorm
from .generation import MuiGenerationMixin
from .llama.model import MuiCausalLMOutput, MuiModelOutput


class MuiNativeModel(MuiModule):
    """Needs of a subclass: __init__ that sets embed_tokens, layers and norm and calls finalize_init();
    start(); `front`: a module of its own state in front of the layers, or None."""

    front: Optional[nn.Module] = None
    logit_scale = 1.0  # rides on the final norm's output

    def __init__(self, engine_config: MuiEngineConfig, config):
        super().__init__(engine_config=engine_config)
        self.config = config

    def final_norm(self, **kw) -> MuiRMSNorm:
        return MuiRMSNorm(self.engine_config, self.config.hidden_size, eps=self.config.rms_norm_eps, **kw)

    def finalize_init(self):
        self.mdevice = self.embed_tokens.weight.device
        self.mdtype = self.embed_tokens.weight.dtype

    def create_cache(self, batch_size: int, seq_len: int) -> MuiHybridCache:
        return MuiHybridCache(self.engine_config, [l.mixer for l in self.layers], batch_size, seq_len, self.mdevice, self.mdtype,
                              front=self.front)

    def start(self, input_ids, inputs_embeds, cache: MuiHybridCache, cache_position) -> Tuple[torch.Tensor, torch.Tensor]:
        """(residual stream in front of the first layer, fp32; the first sublayer's input), both [B, T, hidden]."""
        raise NotImplementedError

    def forward(self, input_ids: Optional[torch.LongTensor] = None, attention_mask: Optional[torch.Tensor] = None,
                past_key_values: Optional[MuiHybridCache] = None, inputs_embeds: Optional[torch.Tensor] = None,
                output_hidden_states: Optional[bool] = None, cache_position: Optional[torch.LongTensor] = None) -> MuiModelOutput:
        """inputs_embeds are rows of the embedding table (their scale is applied here).
        attention_mask [B, T] of 0 / 1 marks left padding of the tokens an empty cache starts with.
        hidden_states: the fp32 residual stream after every layer."""
        if (input_ids is None) == (inputs_embeds is None):
            raise ValueError("specify either input_ids or inputs_embeds")
        src = input_ids if inputs_embeds is None else inputs_embeds
        b, t = src.shape[0], src.shape[1]
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
            cache_position = torch.arange(past, past + t, device=src.device)
        collect = [] if output_hidden_states else None
        x, h = self.start(input_ids, inputs_embeds, cache, cache_position)
        h = run_layers(self.layers, x, h, self.norm, self.config.rms_norm_eps, cache, cache_position, collect,
                       final_scale=self.logit_scale)
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


class MuiNativeForCausalLM(MuiGenerationMixin, MuiModule):
    """Needs of a subclass: model_class, config_class, checkpoint_tensors()."""

    model_class = None
    config_class = None

    def __init__(self, engine_config: MuiEngineConfig, config, device=None, dtype=None):
        MuiModule.__init__(self, engine_config=engine_config)
        self.config = config
        self.model = self.model_class(engine_config, config, device=device, dtype=dtype)
        self.lm_head = MuiLinear(engine_config, config.hidden_size, config.vocab_size, bias=False, device=device, dtype=dtype)
        self._graph_decoder = None

    # ---- weights -----------------------------------------------------------------------------
    def checkpoint_tensors(self) -> Iterator[Tuple[str, torch.Tensor]]:
        """(name, parameter or slice of one that it fills), every tensor of a checkpoint once."""
        raise NotImplementedError

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

    @classmethod
    def _new(cls, engine_config, config, dtype, device):
        lm = cls(engine_config or MuiEngineConfig(), config, device=device, dtype=dtype)
        lm.eval()
        lm.requires_grad_(False)
        return lm

    def _finalize(self):
        from ...engine import _finalize_module
        _finalize_module(self)
        self.muillm_config = self.engine_config
        return self

    @classmethod
    def from_tensors(cls, config, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda",
                     engine_config: Optional[MuiEngineConfig] = None):
        config = config.with_tensor_shapes({k: tuple(t.shape) for k, t in tensors.items()})
        lm = cls._new(engine_config, config, dtype, device)
        lm.load_tensors(tensors.keys(), tensors.__getitem__)
        return lm._finalize()

    @classmethod
    def from_pretrained(cls, path: str, dtype=torch.bfloat16, device="cuda", engine_config: Optional[MuiEngineConfig] = None):
        """A folder with config.json and model.safetensors."""
        from safetensors import safe_open

        with safe_open(os.path.join(path, "model.safetensors"), framework="pt", device="cpu") as f:
            names = list(f.keys())
            config = cls.config_class.from_pretrained(path).with_tensor_shapes({k: tuple(f.get_slice(k).get_shape()) for k in names})
            lm = cls._new(engine_config, config, dtype, device)
            lm.load_tensors(names, f.get_tensor)
        return lm._finalize()

    @classmethod
    def from_config(cls, engine_config: Optional[MuiEngineConfig], config, dtype=torch.bfloat16, device="cuda", seed: int = 0,
                    init_std: float = 0.02):
        """Randomly initialised (matrices ~ N(0, init_std), norm gains 1, biases 0), for benchmarks."""
        lm = cls._new(engine_config, config, dtype, device)
        gen = torch.Generator(device=device)
        gen.manual_seed(seed)
        with torch.no_grad():
            for _, t in lm.checkpoint_tensors():
                if t.dim() == 2:
                    t.normal_(0.0, init_std, generator=gen)
        return lm._finalize()

    # ---- what the decode loop asks of a causal LM -----------------------------------------------
    pads_in_cache = True  # left padding is a property of the cache; no additive mask travels with a step

    @property
    def takes_embeddings(self) -> bool:
        """False: a step needs the token ids themselves, an embedding row is not enough."""
        return self.model.front is None

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
