"""Configuration of a Zufadra decoder, read from its config.json: every size and constant comes from there (the ranks of
the low-rank projections from the checkpoint's tensors); a key that this build does not know is reported."""
import json
import os
from dataclasses import dataclass, field, replace
from typing import Any, Dict, List, Optional, Tuple, Union

from ...attention.hybridattention import MuiHybridAttentionConfig
from ...recurrent.channeldelta import MuiChannelDeltaConfig
from ..nativeconfig import take_section

ARCHITECTURE = "Zufadra"


@dataclass
class MuiBigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int

    def __post_init__(self):
        if self.buckets < 1 or self.mul_prev < 0 or self.mul_cur < 0:
            raise ValueError("a bigram table needs buckets and multipliers that are not negative")


@dataclass
class MuiZufadraLayerConfig:
    mixer: Union[MuiHybridAttentionConfig, MuiChannelDeltaConfig]
    ff: Optional[int] = None  # inner size of the feed-forward; None: the layer has none


def _attention(mx: Dict[str, Any], where: str) -> MuiHybridAttentionConfig:
    take_section(mx, where, ("dim", "heads", "kv_heads", "scale", "vdim"), ("mask", "rot", "softcap"))
    mask, rot = mx.get("mask"), mx.get("rot")
    kw: Dict[str, Any] = {}
    if mask is not None:
        take_section(mask, where + ".mask", ("size",), ("keep_first",))
        if mask["size"] < 1:
            raise ValueError(f"{where}: a window of {mask['size']}")
        kw.update(window=mask["size"], keep_first=mask.get("keep_first", 0))
    if rot is not None:
        take_section(rot, where + ".rot", ("base", "dims"), ("scaling",))
        scaling = rot.get("scaling")
        if scaling is not None:
            take_section(scaling, where + ".rot.scaling", ("factor", "high", "low", "original"))
            scaling = {"factor": scaling["factor"], "low_freq_factor": scaling["low"], "high_freq_factor": scaling["high"],
                       "original_max_position_embeddings": scaling["original"]}
        kw.update(rot_dims=rot["dims"], rot_base=float(rot["base"]), rot_scaling=scaling)
    return MuiHybridAttentionConfig(heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"],
                                    scale=float(mx["scale"]), softcap=float(mx.get("softcap") or 0.0), **kw)


def _channel_delta(mx: Dict[str, Any], where: str) -> MuiChannelDeltaConfig:
    take_section(mx, where, ("conv", "dim", "heads", "kv_heads", "vdim"))
    return MuiChannelDeltaConfig(heads=mx["heads"], kv_heads=mx["kv_heads"], dim=mx["dim"], vdim=mx["vdim"], taps=mx["conv"],
                                 decay_rank=mx["dim"], gate_rank=mx["vdim"])


_MIXERS = {"attention": _attention, "channel_delta": _channel_delta}


def _mlp(ff: Optional[Dict[str, Any]], where: str) -> Optional[int]:
    if ff is None:
        return None
    take_section(ff, where, ("ff", "kind"))
    if ff["kind"] != "dense":
        raise ValueError(f"{where}: unknown feed-forward {ff['kind']!r}")
    return ff["ff"]


@dataclass
class MuiZufadraConfig:
    vocab_size: int
    hidden_size: int
    rms_norm_eps: float
    embedding_scale: float
    residual_mult: float
    logit_scale: float
    bigram: Optional[MuiBigramConfig] = None
    layers: List[MuiZufadraLayerConfig] = field(default_factory=list)
    pad_token_id: Optional[int] = None
    # no table of positions: angles are computed where they are needed, sequences end with the memory
    max_position_embeddings: Optional[int] = None

    def __post_init__(self):
        if not self.layers:
            raise ValueError("a decoder needs layers")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def with_tensor_shapes(self, shapes: Dict[str, Tuple[int, ...]]) -> "MuiZufadraConfig":
        """The same with the ranks that only the checkpoint's tensors tell."""
        layers = []
        for i, layer in enumerate(self.layers):
            if isinstance(layer.mixer, MuiChannelDeltaConfig):
                ranks = [shapes.get(f"l{i}.mix.{n}", (0,))[0] for n in ("a1", "g1")]
                if min(ranks) < 1:
                    raise ValueError(f"layer {i}: the checkpoint has no low-rank projections")
                layer = replace(layer, mixer=replace(layer.mixer, decay_rank=ranks[0], gate_rank=ranks[1]))
            layers.append(layer)
        return replace(self, layers=layers)

    @staticmethod
    def from_dict(cfg: Dict[str, Any]) -> "MuiZufadraConfig":
        take_section(cfg, "config", ("architecture", "embedding", "layers", "logit_scale", "norm", "residual_mult", "vocab", "width"))
        if cfg["architecture"] != ARCHITECTURE:
            raise ValueError(f"architecture {cfg['architecture']!r} is not {ARCHITECTURE}")
        layers = []
        for i, layer in enumerate(cfg["layers"]):
            where = f"layers[{i}]"
            take_section(layer, where, ("type", "mixer"), ("mlp",))
            if layer["type"] not in _MIXERS:
                raise ValueError(f"{where}: unknown mixer {layer['type']!r}")
            layers.append(MuiZufadraLayerConfig(_MIXERS[layer["type"]](layer["mixer"], where + ".mixer"),
                                                _mlp(layer.get("mlp"), where + ".mlp")))
        embedding = take_section(cfg["embedding"], "embedding", ("scale",), ("bigram",))
        bigram = embedding.get("bigram")
        if bigram is not None:
            bigram = MuiBigramConfig(**take_section(bigram, "embedding.bigram", ("buckets", "mul_cur", "mul_prev")))
        return MuiZufadraConfig(vocab_size=cfg["vocab"], hidden_size=cfg["width"],
                                rms_norm_eps=float(take_section(cfg["norm"], "norm", ("eps",))["eps"]),
                                embedding_scale=float(embedding["scale"]), residual_mult=float(cfg["residual_mult"]),
                                logit_scale=float(cfg["logit_scale"]), bigram=bigram, layers=layers)

    @staticmethod
    def from_pretrained(path: str) -> "MuiZufadraConfig":
        with open(os.path.join(path, "config.json")) as f:
            return MuiZufadraConfig.from_dict(json.load(f))
