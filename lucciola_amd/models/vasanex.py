"""The Vasanex decoder as data: how its configuration becomes a :class:`ModelSpec`.

The embedding's row is multiplied by a number.  Every layer is x + mixer(norm(x)), then x + ff(norm(x)) where it
has a feed-forward; the norms are RMS norms whose weight is stored around zero.  The mixer is attention (biases on all
four projections, q and k normed as whole rows, the first entries of every head rotated in halves, a sliding window,
a sink, and values that are mixed with those of the first layer that says so) or the mLSTM's matrix memory.  The
feed-forward is gated, its gate and up entries held below a limit.  The head is the embedding's table without its factor.

Tensor names: ``embed``, ``final.norm`` and, for layer i, ``l<i>.norm1|norm2``, ``l<i>.mix.{q,k,v,o}``(``.b``),
``l<i>.mix.{q,k}.norm``, ``l<i>.mix.{vmix,sink}`` (attention) or ``l<i>.mix.{q,k,v,g,o,norm}`` and
``l<i>.mix.{i,f}``(``.b``) (mlstm), ``l<i>.mlp.{gate,up,down}``.
"""
from __future__ import annotations

from typing import Optional

from ..config.registry import ARCHITECTURES, Architecture
from ..config.specs import ModelSpec, PartSpec, RunEntry, mixer_only_layer, prenorm_layer
from ..config.vasanex_config import ARCHITECTURE, LayerConfig, VasanexConfig

GATE_SLOPE = 1.702      # the feed-forward's gate is g sigmoid(1.702 g)
UP_SHIFT = 1.0          # and multiplies up + 1
MEMORY_FLOOR = 1e-6     # what the matrix memory's denominator holds beside its normaliser


def _norm(cfg: VasanexConfig) -> PartSpec:
    return PartSpec("rms", {"size": cfg.width, "eps": cfg.norm_eps, "one_plus": True})


def vasanex_layer(cfg: VasanexConfig, i: int, layer: LayerConfig, values: Optional[str]):
    p = f"l{i}."
    m = layer.mixer
    names = {"mixer_norm.weight": p + "norm1"}
    if layer.type == "attention":
        position = None
        if m.rot is not None:
            position = PartSpec("rotary", {"rotary_dim": m.rot.dims, "theta": m.rot.base, "pairing": "half"})
        mixer = PartSpec("masked_attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
            "value_dim": m.vdim, "scale": m.scale, "eps": cfg.norm_eps, "position": position, "window": m.window,
            "sink": True, "bias": True, "row_norm": True, "values": values})
        names.update({"mixer." + k: p + "mix." + k for k in ("q", "k", "v", "o", "sink")})
        names.update({f"mixer.{k}_bias": p + f"mix.{k}.b" for k in ("q", "k", "v", "o")})
        names.update({f"mixer.{k}_norm": p + f"mix.{k}.norm" for k in ("q", "k")})
        if values is not None:
            names["mixer.vmix"] = p + "mix.vmix"
    else:
        mixer = PartSpec("mlstm", {
            "hidden_size": cfg.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "cap": m.gate_cap,
            "norm_eps": cfg.norm_eps, "floor": MEMORY_FLOOR})
        names.update({"mixer." + k: p + "mix." + k for k in ("q", "k", "v", "g", "i", "f", "norm", "o")})
        names.update({f"mixer.{k}_bias": p + f"mix.{k}.b" for k in ("i", "f")})
    if layer.mlp is None:
        return mixer_only_layer(mixer, _norm(cfg), names)
    feed_forward = PartSpec("gated_mlp", {
        "hidden_size": cfg.width, "intermediate_size": layer.mlp.ff, "activation": "silu", "limit": layer.mlp.limit,
        "slope": GATE_SLOPE, "shift": UP_SHIFT})
    names["feed_forward_norm.weight"] = p + "norm2"
    names.update({f"feed_forward.{k}_proj": p + f"mlp.{k}" for k in ("gate", "up", "down")})
    return prenorm_layer(mixer, feed_forward, _norm(cfg), _norm(cfg), names)


def vasanex_model_spec(cfg: VasanexConfig) -> ModelSpec:
    layers, kept = [], False
    for i, layer in enumerate(cfg.layers):
        values = None
        if layer.type == "attention" and layer.mixer.v_mix:
            # the first layer that mixes keeps its values for the others
            values, kept = ("mix" if kept else "keep"), True
        layers.append(vasanex_layer(cfg, i, layer, values))
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab, embedding_name="embed", layers=layers,
        run_order=[RunEntry(i) for i in range(len(layers))],
        final_norm=_norm(cfg), final_norm_names={"weight": "final.norm"},
        head_name=None, init_std=cfg.initializer_range, max_positions=0,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width,
                                               "scale": cfg.embedding_scale}))


ARCHITECTURES.register(ARCHITECTURE, Architecture(
    name=ARCHITECTURE, read_config=VasanexConfig.from_dict, model_spec=vasanex_model_spec))
