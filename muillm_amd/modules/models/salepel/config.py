"""Configuration of a Salepel decoder, read from its config.json: every size and constant comes from there;
a key that this build does not know is reported."""
import json
import os
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Union

from ...attention.latentattention import MuiLatentAttentionConfig
from ...moe import MuiMoEConfig
from ...recurrent.mlstm import MuiMLstmConfig
from ..nativeconfig import take_section

ARCHITECTURE = "Salepel"


@dataclass
class MuiSalepelLayerConfig:
    mixer: Union[MuiLatentAttentionConfig, MuiMLstmConfig]
    mlp: Optional[MuiMoEConfig] = None


def _latent_attention(mx: Dict[str, Any], where: str) -> MuiLatentAttentionConfig:
    take_section(mx, where, ("dim", "heads", "kv_rank", "mask", "q_rank", "rot", "rot_dim", "scale", "vdim"), ("kv_from",))
    mask = take_section(mx["mask"], where + ".mask", ("size",))
    rot = take_section(mx["rot"], where + ".rot", ("base", "dims"))
    if rot["dims"] != mx["rot_dim"]:
        raise ValueError(f"{where}: rot.dims {rot['dims']} is not rot_dim {mx['rot_dim']}")
    if mask["size"] < 1:
        raise ValueError(f"{where}: a window of {mask['size']}")
    return MuiLatentAttentionConfig(heads=mx["heads"], dim=mx["dim"], rot_dim=mx["rot_dim"], vdim=mx["vdim"],
                                    q_rank=mx["q_rank"], kv_rank=mx["kv_rank"], scale=float(mx["scale"]),
                                    rot_base=float(rot["base"]), window=mask["size"], kv_source=mx.get("kv_from"))


def _mlstm(mx: Dict[str, Any], where: str) -> MuiMLstmConfig:
    take_section(mx, where, ("dim", "gate_cap", "heads", "vdim"))
    return MuiMLstmConfig(heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"], gate_cap=float(mx["gate_cap"]))


_MIXERS = {"latent_attention": _latent_attention, "mlstm": _mlstm}


def _mlp(ff: Optional[Dict[str, Any]], where: str) -> Optional[MuiMoEConfig]:
    if ff is None:
        return None
    take_section(ff, where, ("kind", "expert", "router"))
    if ff["kind"] != "moe":
        raise ValueError(f"{where}: unknown feed-forward {ff['kind']!r}")
    expert = take_section(ff["expert"], where + ".expert", ("ff", "limit"))
    router = take_section(ff["router"], where + ".router", ("experts", "top"), ("identity",))
    return MuiMoEConfig(experts=router["experts"], identity=router.get("identity", 0), top=router["top"], ff=expert["ff"],
                        limit=float(expert["limit"]))


@dataclass
class MuiSalepelConfig:
    vocab_size: int
    hidden_size: int
    rms_norm_eps: float
    embedding_scale: float
    layers: List[MuiSalepelLayerConfig] = field(default_factory=list)
    pad_token_id: Optional[int] = None
    # no table of positions: angles are computed where they are needed, sequences end with the memory
    max_position_embeddings: Optional[int] = None

    def __post_init__(self):
        if not self.layers:
            raise ValueError("a decoder needs layers")
        for i, layer in enumerate(self.layers):
            mx = layer.mixer
            src = getattr(mx, "kv_source", None)
            if src is None:
                continue
            other = self.layers[src].mixer if 0 <= src < i else None
            if not isinstance(other, MuiLatentAttentionConfig) or other.kv_source is not None:
                raise ValueError(f"layer {i} reads the latent rows of layer {src}, which keeps none before it")
            if (other.kv_rank, other.rot_dim, other.rot_base) != (mx.kv_rank, mx.rot_dim, mx.rot_base):
                raise ValueError(f"layers {src} and {i} share latent rows but differ in kv_rank, rot_dim or rotation")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def with_tensor_shapes(self, shapes) -> "MuiSalepelConfig":
        return self  # the configuration says every size

    @staticmethod
    def from_dict(cfg: Dict[str, Any]) -> "MuiSalepelConfig":
        take_section(cfg, "config", ("architecture", "embedding", "layers", "norm", "vocab", "width"))
        if cfg["architecture"] != ARCHITECTURE:
            raise ValueError(f"architecture {cfg['architecture']!r} is not {ARCHITECTURE}")
        layers = []
        for i, layer in enumerate(cfg["layers"]):
            where = f"layers[{i}]"
            take_section(layer, where, ("type", "mixer"), ("mlp",))
            if layer["type"] not in _MIXERS:
                raise ValueError(f"{where}: unknown mixer {layer['type']!r}")
            layers.append(MuiSalepelLayerConfig(_MIXERS[layer["type"]](layer["mixer"], where + ".mixer"),
                                                _mlp(layer.get("mlp"), where + ".mlp")))
        return MuiSalepelConfig(vocab_size=cfg["vocab"], hidden_size=cfg["width"],
                                rms_norm_eps=float(take_section(cfg["norm"], "norm", ("eps",))["eps"]),
                                embedding_scale=float(take_section(cfg["embedding"], "embedding", ("scale",))["scale"]), layers=layers)

    @staticmethod
    def from_pretrained(path: str) -> "MuiSalepelConfig":
        with open(os.path.join(path, "config.json")) as f:
            return MuiSalepelConfig.from_dict(json.load(f))
