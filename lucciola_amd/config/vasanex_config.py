"""Typed configuration of the Vasanex decoder, read from the keys of its config.json.

The file lists the layers one by one (``layers``: each with its ``type``, "attention" or "mlstm", the mixer's sizes
under ``mixer`` and its feed-forward under ``mlp``, which may be null), the model's ``width`` and ``vocab``, the norms'
``eps`` under ``norm`` and the embedding's ``scale`` under ``embedding``.  Every size and constant is a field read from
the file; nothing is assumed equal between layers, except that the layers that mix values have values of one shape.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .model_config import ConfigError, read_config_json
from .pubodra_config import _get, _int
from .rununex_config import RotaryConfig, _float, _heads, _read_rotary

ARCHITECTURE = "Vasanex"


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int]
    rot: Optional[RotaryConfig]
    v_mix: bool


@dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class MlpConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class LayerConfig:
    type: str                       # "attention" or "mlstm"
    mixer: Any                      # AttentionConfig or MatrixMemoryConfig
    mlp: Optional[MlpConfig]


@dataclass(frozen=True)
class VasanexConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[LayerConfig, ...]
    initializer_range: float = 0.02
    eos_token_ids: Tuple[int, ...] = ()
    raw: Optional[Dict[str, Any]] = None    # the dict it was read from, for writing it out again

    @staticmethod
    def from_dict(data: Dict[str, Any]) -> "VasanexConfig":
        layers = _get(data, "layers", "the model")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        parsed = tuple(_read_layer(entry, i) for i, entry in enumerate(layers))
        mixing = [(i, layer.mixer) for i, layer in enumerate(parsed) if layer.type == "attention" and layer.mixer.v_mix]
        for i, m in mixing[1:]:
            first = mixing[0][1]
            if (m.kv_heads, m.vdim) != (first.kv_heads, first.vdim):
                raise ConfigError(f"config.json: layers[{i}] mixes values of {m.kv_heads} x {m.vdim} entries with "
                                  f"layers[{mixing[0][0]}]'s of {first.kv_heads} x {first.vdim}")
        eps = _float(_get(data, "norm", "the model"), "eps", "norm")
        if not eps > 0:
            raise ConfigError("config.json: norm.eps must be positive")
        embedding = data.get("embedding") or {}
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in eos) if isinstance(eos, (list, tuple)) else (int(eos),)
        return VasanexConfig(
            vocab=_int(data, "vocab", "the model"), width=_int(data, "width", "the model"), norm_eps=eps,
            embedding_scale=_float(embedding, "scale", "embedding") if "scale" in embedding else 1.0, layers=parsed,
            initializer_range=float(data.get("initializer_range", 0.02)), eos_token_ids=eos_ids, raw=dict(data))

    @staticmethod
    def from_folder(folder: str) -> "VasanexConfig":
        return VasanexConfig.from_dict(read_config_json(folder))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw) if self.raw is not None else {}


def _read_attention(m, where) -> AttentionConfig:
    heads, kv_heads = _heads(m, where)
    dim = _int(m, "dim", where)
    mask = m.get("mask")
    window = _int(mask, "size", where + ".mask") if mask and mask.get("size") is not None else None
    v_mix = m.get("v_mix", False)
    if not isinstance(v_mix, bool):
        raise ConfigError(f"config.json: {where}.v_mix must be true or false, got {v_mix!r}")
    return AttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=_int(m, "vdim", where),
                           scale=_float(m, "scale", where), window=window, rot=_read_rotary(m, where, dim), v_mix=v_mix)


def _read_matrix_memory(m, where) -> MatrixMemoryConfig:
    cap = _float(m, "gate_cap", where)
    if not cap > 0:
        raise ConfigError(f"config.json: {where}.gate_cap must be positive, got {cap}")
    return MatrixMemoryConfig(heads=_int(m, "heads", where), dim=_int(m, "dim", where), vdim=_int(m, "vdim", where),
                              gate_cap=cap)


def _read_layer(entry: Dict[str, Any], i: int) -> LayerConfig:
    where = f"layers[{i}]"
    kind = str(_get(entry, "type", where))
    m = _get(entry, "mixer", where)
    if kind == "attention":
        mixer = _read_attention(m, where + ".mixer")
    elif kind == "mlstm":
        mixer = _read_matrix_memory(m, where + ".mixer")
    else:
        raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this design (attention, mlstm)")
    mlp = entry.get("mlp")
    mlp_cfg = None
    if mlp:
        lw = where + ".mlp"
        mkind = str(mlp.get("kind", "dense"))
        if mkind != "dense":
            raise ConfigError(f"config.json: {lw}.kind '{mkind}' is not a feed-forward of this design (dense)")
        mlp_cfg = MlpConfig(ff=_int(mlp, "ff", lw), limit=_float(mlp, "limit", lw))
        if not mlp_cfg.limit > 0:
            raise ConfigError(f"config.json: {lw}.limit must be positive, got {mlp_cfg.limit}")
    return LayerConfig(kind, mixer, mlp_cfg)
