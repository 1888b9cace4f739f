"""Typed configuration of the Nogosun decoder, read from the keys of its config.json.

The file lists the layers one by one (``layers``: each with its ``type``, "attention", "channel_delta" or "parallel", the
mixer's sizes under ``mixer`` and its feed-forward under ``mlp``, which may be null), the model's ``width`` and ``vocab``,
the norms' ``eps`` under ``norm`` and the embedding's ``scale`` under ``embedding``.  A layer with ``weights_of``: j uses
layer j's tensors and is otherwise the same.  Every size and constant is a field read from the file; nothing is assumed
equal between other layers.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any, Dict, Optional, Tuple

from .model_config import ConfigError, read_config_json
from .pubodra_config import YarnScaling, _get, _int
from .rununex_config import _float, _heads

ARCHITECTURE = "Nogosun"


@dataclass(frozen=True)
class RotaryConfig:
    base: float
    dims: int
    scaling: Optional[YarnScaling] = None


@dataclass(frozen=True)
class KeyValueAttentionConfig:
    """Attention whose values are its keys."""

    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: Optional[int]
    keep_first: int
    rot: Optional[RotaryConfig]


@dataclass(frozen=True)
class CappedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float
    temperature: Tuple[float, float]        # (coef, every)


@dataclass(frozen=True)
class GatedLinearConfig:
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class ParallelConfig:
    left: CappedAttentionConfig
    right: GatedLinearConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class ChannelDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class MoeConfig:
    ff: int
    experts: int
    top: int


@dataclass(frozen=True)
class LayerConfig:
    type: str                       # "attention", "channel_delta" or "parallel"
    mixer: Any                      # KeyValueAttentionConfig, ChannelDeltaConfig or ParallelConfig
    mlp: Optional[MoeConfig]
    weights_of: int                 # the layer whose tensors it uses (its own place: it has its own)


@dataclass(frozen=True)
class NogosunConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[LayerConfig, ...]
    initializer_range: float = 0.02
    eos_token_ids: Tuple[int, ...] = ()
    raw: Optional[Dict[str, Any]] = None    # the dict it was read from, for writing it out again

    @staticmethod
    def from_dict(data: Dict[str, Any]) -> "NogosunConfig":
        layers = _get(data, "layers", "the model")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        parsed = [_read_layer(entry, i) for i, entry in enumerate(layers)]
        owners = [_owner(parsed, i) for i in range(len(parsed))]
        for i, j in enumerate(owners):
            if (parsed[i].type, parsed[i].mixer, parsed[i].mlp) != (parsed[j].type, parsed[j].mixer, parsed[j].mlp):
                raise ConfigError(f"config.json: layers[{i}] uses the tensors of layers[{j}] and must equal it")
        parsed = tuple(replace(layer, weights_of=owner) for layer, owner in zip(parsed, owners))
        eps = _float(_get(data, "norm", "the model"), "eps", "norm")
        if not eps > 0:
            raise ConfigError("config.json: norm.eps must be positive")
        embedding = data.get("embedding") or {}
        eos = data.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in eos) if isinstance(eos, (list, tuple)) else (int(eos),)
        return NogosunConfig(
            vocab=_int(data, "vocab", "the model"), width=_int(data, "width", "the model"), norm_eps=eps,
            embedding_scale=_float(embedding, "scale", "embedding") if "scale" in embedding else 1.0, layers=parsed,
            initializer_range=float(data.get("initializer_range", 0.02)), eos_token_ids=eos_ids, raw=dict(data))

    @staticmethod
    def from_folder(folder: str) -> "NogosunConfig":
        return NogosunConfig.from_dict(read_config_json(folder))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw) if self.raw is not None else {}


def _owner(layers, i: int) -> int:
    """The layer whose tensors layer i uses in the end: a borrowed layer may itself borrow."""
    seen, at = {i}, i
    while layers[at].weights_of != at:
        at = layers[at].weights_of
        if not 0 <= at < len(layers):
            raise ConfigError(f"config.json: layers[{i}].weights_of leads to layer {at} of {len(layers)}")
        if at in seen:
            raise ConfigError(f"config.json: layers[{i}].weights_of goes round in a circle")
        seen.add(at)
    return at


def _positive(data, key, where) -> float:
    value = _float(data, key, where)
    if not value > 0:
        raise ConfigError(f"config.json: {where}.{key} must be positive, got {value}")
    return value


def _read_rotary(m, where, dim: int) -> Optional[RotaryConfig]:
    rot = m.get("rot")
    if not rot or not rot.get("dims"):
        return None
    rw = where + ".rot"
    dims = _int(rot, "dims", rw, 2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"config.json: {rw}.dims ({dims}) must be even and at most dim ({dim})")
    base = _float(rot, "base", rw)
    if not base > 1:
        raise ConfigError(f"config.json: {rw}.base must be above 1")
    scaling = rot.get("scaling")
    yarn = None
    if scaling:
        sw = rw + ".scaling"
        yarn = YarnScaling(*(_positive(scaling, key, sw) for key in ("factor", "original", "fast", "slow")))
    return RotaryConfig(base, dims, yarn)


def _read_attention(m, where) -> KeyValueAttentionConfig:
    heads, kv_heads = _heads(m, where)
    dim = _int(m, "dim", where)
    if "vdim" in m and _int(m, "vdim", where) != dim:
        raise ConfigError(f"config.json: {where}.vdim ({m['vdim']}) must be dim ({dim}): the values are the keys")
    mask = m.get("mask") or {}
    window = _int(mask, "size", where + ".mask") if mask.get("size") is not None else None
    keep = _int(mask, "keep_first", where + ".mask", 0) if mask.get("keep_first") is not None else 0
    return KeyValueAttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, scale=_float(m, "scale", where), window=window,
                                   keep_first=keep, rot=_read_rotary(m, where, dim))


def _read_parallel(m, where) -> ParallelConfig:
    left, right = _get(m, "left", where), _get(m, "right", where)
    lw, rw = where + ".left", where + ".right"
    heads, kv_heads = _heads(left, lw)
    temperature = _get(left, "q_temp", lw)
    left_cfg = CappedAttentionConfig(
        heads=heads, kv_heads=kv_heads, dim=_int(left, "dim", lw), vdim=_int(left, "vdim", lw),
        scale=_float(left, "scale", lw), softcap=_positive(left, "softcap", lw),
        temperature=(_float(temperature, "coef", lw + ".q_temp"), _positive(temperature, "every", lw + ".q_temp")))
    right_cfg = GatedLinearConfig(heads=_int(right, "heads", rw), dim=_int(right, "dim", rw), vdim=_int(right, "vdim", rw),
                                  tau=_positive(right, "tau", rw))
    return ParallelConfig(left_cfg, right_cfg, _float(m, "left_scale", where), _float(m, "right_scale", where))


def _read_channel_delta(m, where) -> ChannelDeltaConfig:
    heads, kv_heads = _heads(m, where)
    return ChannelDeltaConfig(heads=heads, kv_heads=kv_heads, dim=_int(m, "dim", where), vdim=_int(m, "vdim", where),
                              conv=_int(m, "conv", where))


_MIXERS = {"attention": _read_attention, "channel_delta": _read_channel_delta, "parallel": _read_parallel}


def _read_layer(entry: Dict[str, Any], i: int) -> LayerConfig:
    where = f"layers[{i}]"
    kind = str(_get(entry, "type", where))
    if kind not in _MIXERS:
        raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this design ({', '.join(_MIXERS)})")
    mixer = _MIXERS[kind](_get(entry, "mixer", where), where + ".mixer")
    mlp = entry.get("mlp")
    mlp_cfg = None
    if mlp:
        lw = where + ".mlp"
        mkind = str(mlp.get("kind", "moe"))
        if mkind != "moe":
            raise ConfigError(f"config.json: {lw}.kind '{mkind}' is not a feed-forward of this design (moe)")
        router = _get(mlp, "router", lw)
        mlp_cfg = MoeConfig(ff=_int(_get(mlp, "expert", lw), "ff", lw + ".expert"),
                            experts=_int(router, "experts", lw + ".router"), top=_int(router, "top", lw + ".router"))
        if mlp_cfg.top > mlp_cfg.experts:
            raise ConfigError(f"config.json: {lw}.router.top ({mlp_cfg.top}) exceeds its {mlp_cfg.experts} experts")
    owner = _int(entry, "weights_of", where, 0) if entry.get("weights_of") is not None else i
    if entry.get("weights_of") == i:
        raise ConfigError(f"config.json: {where}.weights_of names the layer itself")
    return LayerConfig(kind, mixer, mlp_cfg, owner)
