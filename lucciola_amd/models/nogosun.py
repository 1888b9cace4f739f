"""The Nogosun decoder as data: how its configuration becomes a :class:`ModelSpec`.

The embedding's row is multiplied by a number.  Every layer is x + mixer(norm_1(x)) + ff(norm_2(x)), both branches of the
same x behind RMS norms of their own.  The mixer is attention whose values are its keys before their rotation (biases on
q and k, the first entries of every head rotated in halves with stretched frequencies, a sliding window beside the
sequence's first tokens), the gated delta rule with a decay per key channel, or two mixers side by side on the same
input: attention without a rotation (biases on q, k and v, a norm per head, a query temperature that grows with the
position, capped scores, one added to the softmax's denominator, an output gate) beside gated linear attention; their
outputs are added with a scale each.  The feed-forward is a mixture of two-matrix experts with the exact GELU, weighed
by a softmax over all experts that is not renormalised; or none.  The head is a table of its own.

A layer may use an earlier layer's tensors with a cache or state of its own: it is one more entry of the run order that
names that layer.

Tensor names: ``embed``, ``final.norm``, ``head`` and, for a layer i with tensors of its own, ``l<i>.norm1|norm2``,
``l<i>.mix.{q,k}``(``.b``) and ``l<i>.mix.o`` (attention), ``l<i>.mix.{q,k,v}``(``.conv``) and
``l<i>.mix.{b,A_log,norm,a1,a2,dt_bias,g1,g2,o}`` (channel_delta) or ``l<i>.mix.left.{q,k,v}``(``.b``),
``l<i>.mix.left.{q,k}.norm``, ``l<i>.mix.left.{g,o}`` and ``l<i>.mix.right.{q,k,v,g,o,norm,a1,a2,a2.b}`` (parallel),
``l<i>.mlp.router``, ``l<i>.mlp.e<k>.{up,down}``.
"""
from __future__ import annotations

from ..config.nogosun_config import ARCHITECTURE, LayerConfig, NogosunConfig
from ..config.registry import ARCHITECTURES, Architecture
from ..config.specs import ModelSpec, PartSpec, RunEntry, parallel_layer

ONE_MORE = 0.0      # the score of what the capped attention's softmax adds to its denominator
UNIT_EPS = 1e-6     # under the root of the delta rule's unit vectors


def _norm(cfg: NogosunConfig) -> PartSpec:
    return PartSpec("rms", {"size": cfg.width, "eps": cfg.norm_eps})


def nogosun_layer(cfg: NogosunConfig, i: int, layer: LayerConfig):
    p = f"l{i}."
    m = layer.mixer
    names = {"mixer_norm.weight": p + "norm1"}
    if layer.type == "attention":
        position = None
        if m.rot is not None:
            position = PartSpec("rotary", {"rotary_dim": m.rot.dims, "theta": m.rot.base, "pairing": "half",
                                           "scaling": m.rot.scaling.to_dict() if m.rot.scaling else None})
        mixer = PartSpec("masked_attention", {
            "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
            "value_dim": m.dim, "scale": m.scale, "eps": cfg.norm_eps, "position": position, "window": m.window,
            "keep_first": m.keep_first, "bias": True, "output_bias": False, "values": "keys"})
        names.update({"mixer." + k: p + "mix." + k for k in ("q", "k", "o")})
        names.update({f"mixer.{k}_bias": p + f"mix.{k}.b" for k in ("q", "k")})
    elif layer.type == "channel_delta":
        mixer = PartSpec("channel_delta", {
            "hidden_size": cfg.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim,
            "value_dim": m.vdim, "conv_taps": m.conv, "norm_eps": cfg.norm_eps, "unit_eps": UNIT_EPS})
        names.update({"mixer." + k: p + "mix." + k for k in ("q", "k", "v", "norm", "o")})
        names.update({f"mixer.{k}_conv": p + f"mix.{k}.conv" for k in ("q", "k", "v")})
        names.update({"mixer." + ours: p + "mix." + theirs for ours, theirs in (
            ("beta", "b"), ("rate_log", "A_log"), ("rate_in", "a1"), ("rate_out", "a2"), ("rate_bias", "dt_bias"),
            ("gate_in", "g1"), ("gate_out", "g2"))})
    else:
        left = PartSpec("masked_attention", {
            "hidden_size": cfg.width, "num_heads": m.left.heads, "num_kv_heads": m.left.kv_heads,
            "head_dim": m.left.dim, "value_dim": m.left.vdim, "scale": m.left.scale, "eps": cfg.norm_eps, "bias": True,
            "output_bias": False, "head_norm": True, "temperature": m.left.temperature, "softcap": m.left.softcap,
            "sink": ONE_MORE, "gate": True})
        right = PartSpec("gated_linear", {
            "hidden_size": cfg.width, "num_heads": m.right.heads, "key_dim": m.right.dim, "value_dim": m.right.vdim,
            "tau": m.right.tau, "norm_eps": cfg.norm_eps})
        mixer = PartSpec("parallel", {"left": left, "right": right, "left_scale": m.left_scale,
                                      "right_scale": m.right_scale})
        q = p + "mix.left."
        names.update({"mixer.left." + k: q + k for k in ("q", "k", "v", "g", "o")})
        names.update({f"mixer.left.{k}_bias": q + k + ".b" for k in ("q", "k", "v")})
        names.update({f"mixer.left.{k}_norm": q + k + ".norm" for k in ("q", "k")})
        names.update({"mixer.right." + ours: p + "mix.right." + theirs for ours, theirs in (
            ("q", "q"), ("k", "k"), ("v", "v"), ("gate", "g"), ("o", "o"), ("norm", "norm"), ("rate_in", "a1"),
            ("rate_out", "a2"), ("rate_bias", "a2.b"))})
    if layer.mlp is None:
        return parallel_layer(mixer, None, _norm(cfg), None, names)
    mlp = layer.mlp
    feed_forward = PartSpec("routed_mlp", {
        "hidden_size": cfg.width, "intermediate_size": mlp.ff, "experts": mlp.experts, "top": mlp.top,
        "activation": "gelu", "scores": "softmax", "renormalise": False})
    names["feed_forward_norm.weight"] = p + "norm2"
    names["feed_forward.router"] = p + "mlp.router"
    for k in range(mlp.experts):
        for which in ("up", "down"):
            names[f"feed_forward.experts.{k}.{which}"] = p + f"mlp.e{k}.{which}"
    return parallel_layer(mixer, feed_forward, _norm(cfg), _norm(cfg), names)


def nogosun_model_spec(cfg: NogosunConfig) -> ModelSpec:
    owners = [i for i, layer in enumerate(cfg.layers) if layer.weights_of == i]
    place = {i: n for n, i in enumerate(owners)}
    sizes = {"vocab_size": cfg.vocab, "hidden_size": cfg.width}
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab, embedding_name="embed",
        layers=[nogosun_layer(cfg, i, cfg.layers[i]) for i in owners],
        run_order=[RunEntry(place[layer.weights_of]) for layer in cfg.layers],
        final_norm=_norm(cfg), final_norm_names={"weight": "final.norm"},
        head_name="head", init_std=cfg.initializer_range, max_positions=0,
        embedding=PartSpec("token_embedding", {**sizes, "scale": cfg.embedding_scale}))


ARCHITECTURES.register(ARCHITECTURE, Architecture(
    name=ARCHITECTURE, read_config=NogosunConfig.from_dict, model_spec=nogosun_model_spec))
