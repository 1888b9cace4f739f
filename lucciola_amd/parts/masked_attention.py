"""Attention whose heads may differ from the plain kind in several ways, each a parameter:

- keys and values of sizes of their own (``head_dim``, ``value_dim``), G key/value heads for H query heads;
- ``maps`` = 2, differential attention: a head has two queries and a kv head two keys ([map 1, map 2] side by
  side); each map is a softmax attention of its own over the same values, and the head's output is
  a_1 - lambda a_2 with lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + ``difference`` from four learned vectors, then
  divided by its root mean square over the value entries and multiplied by 1 - ``difference``;
- ``conv_taps`` > 0: q, k and v pass a short causal convolution per channel right behind their projection
  (no bias, no activation); the last ``conv_taps`` - 1 projected rows of a request are state;
- ``position``: a rotary encoding on the first entries of every map of every head;
- ``bias``: q, k and v and the output projection have biases;
- ``row_norm``: all of a token's q, before it is split into heads, is divided by its root mean square and
  multiplied by a weight of its size, and so is all of its k, before the rotation;
- ``values``: the layer's values go to later layers or are mixed with an earlier layer's values of the same
  token, (1 - lambda) v + lambda v_earlier with one learned number (tensor ``vmix``), before they are cached:
  "keep": the values as projected stay for later layers of the pass; "mix": they are mixed with those that the last
  "keep" layer before this one left (a "keep" layer has the tensor too and does not use it);
  or "keys": there is no value projection, the values are the keys as projected (bias included, before any norm or
  rotation);
- ``output_bias`` False: biases on q, k and v only;
- ``head_norm``: every q head is divided by its root mean square and multiplied by a weight of the head's size that all
  heads share, and so is every k head with another one, before the rotation;
- ``temperature`` (coef, every): q at position p is multiplied by 1 + coef ln(floor((p + 1) / every) + 1);
- ``unit_qk``: every q and k head is divided by its root mean square (no weight);
- ``distance_bias``: r1_h ln(1 + r2_h (i - j)) is taken off the score of query i and key j (two learned numbers a
  head);
- ``softcap``: the scores become softcap tanh(score / softcap);
- ``sink``: a learned number s_h a head whose exp(s_h) is one more term of the softmax's denominator; or a number, the
  same constant for every head (0.0: one is added to the denominator) and no tensor;
- ``gate``: the heads' outputs times sigmoid(W_g h), entry by entry, before the output projection;
- ``chunk``: position i sees j <= i only inside its own chunk of that many positions, counted from the sequence's
  start; ``window``: only the last so many positions; ``keep_first``: the first so many positions are seen
  by every later one beside those (their pages are not given back).

The projections leave as float32; one kernel makes q, k and v of them (convolution, rotation of interleaved pairs,
unit norm; or, with ``bias``, ``row_norm``, ``values`` or rotation of halves, the kernel that knows those:
``ops.attention_rows``; or, with ``head_norm``, ``temperature`` or values that are the keys, ``ops.attention_heads``) and
writes k and v into the cache (keys token-major, values transposed inside a page).  Scores, softmax, bias, sink
and the maps' combination are float32 whatever the cache's type; with a bfloat16 cache of sizes that fit, the two
products run on the matrix cores (``ops.masked_attention``), else in float32 multiply-adds.
"""
from __future__ import annotations

import math
from typing import Dict, Optional, Sequence, Union

import torch

from ..cache.specs import FixedStates, PagedRows
from ..config.registry import MIXERS, POSITION_ENCODINGS
from ..config.specs import PartSpec
from ..kernels import ops
from ..weights.loader import ParamDecl
from .base import BuildContext, Part, build_part
from .feed_forward import stack_rows


def _f32(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.float32).contiguous()


PASSED_VALUES = "values"        # under which a "keep" layer leaves its values in the batch


@MIXERS.register("masked_attention")
class MaskedAttention(Part):
    graph_safe = True   # launches only kernels whose arguments stay put between steps

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 scale: float, eps: float, maps: int = 1, difference: float = 0.0, conv_taps: int = 0,
                 position: Optional[PartSpec] = None, unit_qk: bool = False, distance_bias: bool = False,
                 sink: Union[bool, float] = False, gate: bool = False, chunk: Optional[int] = None,
                 window: Optional[int] = None, bias: bool = False, row_norm: bool = False, values: Optional[str] = None,
                 output_bias: bool = True, head_norm: bool = False, temperature: Optional[Sequence[float]] = None,
                 softcap: float = 0.0, keep_first: int = 0):
        super().__init__(hidden_size=hidden_size, num_heads=num_heads, num_kv_heads=num_kv_heads, head_dim=head_dim,
                         value_dim=value_dim, scale=scale, eps=eps, maps=maps, difference=difference,
                         conv_taps=conv_taps, position=position, unit_qk=unit_qk, distance_bias=distance_bias,
                         sink=sink, gate=gate, chunk=chunk, window=window, bias=bias, row_norm=row_norm,
                         values=values, output_bias=output_bias, head_norm=head_norm, temperature=temperature,
                         softcap=softcap, keep_first=keep_first)
        if num_heads % num_kv_heads:
            raise ValueError(f"masked_attention: {num_heads} heads are not a multiple of {num_kv_heads} kv heads")
        if maps not in (1, 2):
            raise ValueError(f"masked_attention: {maps} score maps a head (1 or 2)")
        self.H, self.nh, self.nkv = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.d, self.dv, self.maps = int(head_dim), int(value_dim), int(maps)
        if max(self.d, self.dv) > ops.MASKED_ATTENTION_MAX:
            raise ValueError(f"masked_attention: heads of {self.d}/{self.dv} entries are above the kernel's "
                             f"{ops.MASKED_ATTENTION_MAX}")
        self.scale, self.eps, self.difference = float(scale), float(eps), float(difference)
        self.taps = int(conv_taps)
        if not 0 <= self.taps <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError(f"masked_attention: {self.taps} taps are above the kernel's {ops.SHORT_CONV_MAX_TAPS}")
        # a sink of one constant for all heads is no tensor
        self.sink_constant = None if isinstance(sink, bool) else float(sink)
        self.unit_qk, self.distance_bias, self.has_sink, self.has_gate = (bool(unit_qk), bool(distance_bias),
                                                                          sink is True, bool(gate))
        self.chunk, self.window = int(chunk) if chunk else 0, int(window) if window else 0
        self.keep_first, self.softcap = int(keep_first), float(softcap)
        if self.keep_first < 0 or self.softcap < 0:
            raise ValueError("masked_attention: keep_first and softcap must not be negative")
        self.position = build_part(POSITION_ENCODINGS, position) if position else None
        self.has_bias, self.row_norm, self.values = bool(bias), bool(row_norm), values
        if values not in (None, "keep", "mix", "keys"):
            raise ValueError(f"masked_attention: values '{values}' are neither 'keep' nor 'mix' nor 'keys'")
        self.has_output_bias, self.head_norm = self.has_bias and bool(output_bias), bool(head_norm)
        self.temperature = tuple(float(v) for v in temperature) if temperature is not None else None
        if self.temperature is not None and (len(self.temperature) != 2 or not self.temperature[1] > 0):
            raise ValueError("masked_attention: a temperature is (coef, every) with every > 0")
        self.values_are_keys = values == "keys"
        if self.values_are_keys and self.dv != self.d:
            raise ValueError(f"masked_attention: values that are the keys have {self.d} entries, not {self.dv}")
        pairing = getattr(self.position, "pairing", None)
        if self.position is not None and pairing not in ("half", "interleaved"):
            raise ValueError(f"masked_attention: no prologue kernel rotates with the pairing '{pairing}'")
        self.half = pairing == "half"
        # which of the prologue kernels makes q, k and v
        self.by_heads = self.head_norm or self.temperature is not None or self.values_are_keys
        self.by_rows = not self.by_heads and (self.has_bias or self.row_norm or self.values is not None or self.half)
        if self.by_heads and (self.row_norm or self.taps or self.unit_qk or self.maps > 1 or values in ("keep", "mix")):
            raise ValueError("masked_attention: head_norm, temperature and values that are the keys go without row_norm, "
                             "convolutions, unit_qk, several maps and mixed values (no prologue kernel has both)")
        if self.by_rows and (self.taps or self.unit_qk):
            raise ValueError("masked_attention: convolutions and unit_qk go without bias, row_norm, values and "
                             "rotation of halves (no prologue kernel has both)")
        if self.position is not None:
            if self.position.rotary_dim > self.d:
                raise ValueError(f"masked_attention: {self.position.rotary_dim} rotated entries in heads of {self.d}")
        self.nq_cols = self.nh * self.maps * self.d
        self.nk_cols = self.nkv * self.maps * self.d
        self.nv_cols = self.nkv * self.dv
        # columns of the projection: q | k | v, or q | k where the values are the keys (what passes the convolutions)
        self.channels = self.nq_cols + self.nk_cols + (0 if self.values_are_keys else self.nv_cols)

    def declare(self) -> Dict[str, ParamDecl]:
        out = {"q": ParamDecl((self.nq_cols, self.H)), "k": ParamDecl((self.nk_cols, self.H)),
               "v": ParamDecl((self.nv_cols, self.H)), "o": ParamDecl((self.H, self.nh * self.dv))}
        if self.values_are_keys:
            del out["v"]
        if self.taps:
            out.update({"q_conv": ParamDecl((self.nq_cols, self.taps), role="vector"),
                        "k_conv": ParamDecl((self.nk_cols, self.taps), role="vector"),
                        "v_conv": ParamDecl((self.nv_cols, self.taps), role="vector")})
        if self.maps == 2:
            for name in ("lq1", "lk1", "lq2", "lk2"):
                out[name] = ParamDecl((self.d,), role="vector")
        if self.distance_bias:
            out["r1"] = ParamDecl((self.nh,), role="vector", init="ones_plus_normal")
            out["r2"] = ParamDecl((self.nh,), role="vector", init="ones_plus_normal")
        if self.has_sink:
            out["sink"] = ParamDecl((self.nh,), role="vector")
        if self.has_gate:
            out["g"] = ParamDecl((self.nh * self.dv, self.H))
        if self.has_bias:
            for name, size in (("q_bias", self.nq_cols), ("k_bias", self.nk_cols), ("v_bias", self.nv_cols),
                               ("o_bias", self.H)):
                if (name != "v_bias" or not self.values_are_keys) and (name != "o_bias" or self.has_output_bias):
                    out[name] = ParamDecl((size,), role="vector")
        if self.row_norm:
            out["q_norm"] = ParamDecl((self.nq_cols,), role="vector", init="ones_plus_normal")
            out["k_norm"] = ParamDecl((self.nk_cols,), role="vector", init="ones_plus_normal")
        if self.head_norm:
            out["q_norm"] = ParamDecl((self.d,), role="vector", init="ones_plus_normal")
            out["k_norm"] = ParamDecl((self.d,), role="vector", init="ones_plus_normal")
        if self.values in ("keep", "mix"):
            out["vmix"] = ParamDecl((), role="vector")
        return out

    def bind(self, tensors, ctx: BuildContext) -> None:
        self.dtype = ctx.dtype
        projected = ("q", "k") if self.values_are_keys else ("q", "k", "v")
        mats = [tensors[k] for k in projected] + ([tensors["g"]] if self.has_gate else [])
        self.proj = stack_rows(mats)
        self.o = tensors["o"]
        self.conv = None
        if self.taps:
            self.conv = torch.cat([_f32(tensors[k]) for k in ("q_conv", "k_conv", "v_conv")], dim=0).contiguous()
        self.subtract = 0.0
        if self.maps == 2:
            # one number for the layer; read once, at load
            lq1, lk1, lq2, lk2 = (tensors[k].to(torch.float64).cpu() for k in ("lq1", "lk1", "lq2", "lk2"))
            self.subtract = math.exp(float((lq1 * lk1).sum())) - math.exp(float((lq2 * lk2).sum())) + self.difference
        self.r1 = _f32(tensors["r1"]) if self.distance_bias else None
        self.r2 = _f32(tensors["r2"]) if self.distance_bias else None
        self.sink = _f32(tensors["sink"]) if self.has_sink else None
        if self.sink_constant is not None:
            self.sink = torch.full((self.nh,), self.sink_constant, dtype=torch.float32, device=ctx.device)
        self.bias = self.o_bias = self.q_norm = self.k_norm = None
        if self.has_bias:
            self.bias = torch.cat([_f32(tensors[k + "_bias"]) for k in projected]).contiguous()
            self.o_bias = _f32(tensors["o_bias"]) if self.has_output_bias else None
        if self.row_norm or self.head_norm:
            self.q_norm, self.k_norm = _f32(tensors["q_norm"]), _f32(tensors["k_norm"])
        # one number for the layer; read once, at load
        self.mix = float(tensors["vmix"].to(torch.float32).item()) if self.values == "mix" else 0.0
        if self.position is not None:
            self.position.bind({}, ctx)

    def cache_need(self):
        rows = PagedRows(self.nk_cols, self.nv_cols, self.window or None,
                         self.keep_first if self.window else 0)
        if self.taps > 1:
            return rows, FixedStates(((self.taps - 1, self.channels),))
        return rows

    def batch_planner(self):
        # the step's tokens in tiles of up to 16 of one request: the matrix-core kernel's work items
        return ops.LATENT_PLAN, ops.plan_latent_attention

    def tables_epoch(self) -> int:
        return self.position.tables_epoch() if self.position is not None else 0

    def ready(self, position: int) -> bool:
        return self.position.ready(position) if self.position is not None else True

    def forward(self, x: torch.Tensor, site) -> torch.Tensor:
        batch = site.batch
        paged = site.part(0)
        k_cache, v_cache = paged.cache
        pages = paged.pages
        tail = site.part(1).cache[0] if self.taps > 1 else None
        proj = ops.gemm(x, self.proj, torch.float32)
        table, rot = None, 0
        if self.position is not None:
            table, rot = self.position.rotary_table(batch.max_position), self.position.rotary_dim
        slots = pages.slots if site.writes_cache else None
        if self.by_heads:
            q = ops.attention_heads(
                proj, self.nh, self.nkv, self.nkv, self.d, self.dv, self.dtype, k_cache, v_cache, slots,
                values_are_keys=self.values_are_keys, bias=self.bias, q_weight=self.q_norm, k_weight=self.k_norm,
                eps=self.eps, table=table, rot=rot, half=self.half, positions=batch.positions,
                temperature=self.temperature)
        elif self.by_rows:
            q = self._by_rows(proj, site, k_cache, v_cache, table, rot)
        else:
            q = ops.attention_prepare(
                proj, self.nh * self.maps, self.nkv * self.maps, self.nkv, self.d, self.dv, self.dtype, k_cache, v_cache,
                slots, taps=self.conv, tail=tail, tok_req=batch.tok_req, q_offsets=batch.q_offsets,
                slot_ids=batch.slot_ids, table=table, rot=rot, positions=batch.positions,
                unit_eps=self.eps if self.unit_qk else None)
        if self.taps > 1:
            ops.conv_tail_update(proj, tail, self.channels, self.taps, batch.q_offsets, batch.slot_ids,
                                 batch.num_requests)
        o = ops.masked_attention(
            q, k_cache, v_cache, batch.tok_req, batch.positions, pages.block_table, pages.page_size, self.nh, self.nkv,
            self.maps, self.d, self.dv, self.scale, chunk=self.chunk, window=self.window,
            keep=self.keep_first if self.window or self.chunk else 0, cap=self.softcap, r1=self.r1, r2=self.r2,
            sink=self.sink, subtract=self.subtract, unit_eps=self.eps if self.maps == 2 else None,
            out_scale=1.0 - self.difference if self.maps == 2 else 1.0,
            gate=proj if self.has_gate else None, gate_column=self.channels, plan=batch.plans.get(ops.LATENT_PLAN),
            max_ctx=batch.max_ctx)
        y = ops.gemm(o, self.o, self.dtype, defer=True)
        return ops.BiasedBranch(y, self.o_bias) if self.o_bias is not None else y

    def _by_rows(self, proj: torch.Tensor, site, k_cache, v_cache, table, rot: int) -> torch.Tensor:
        batch, earlier = site.batch, None
        if self.values == "mix":
            earlier = batch.passing.get(PASSED_VALUES)
            if earlier is None:
                raise ValueError("masked_attention: no earlier layer has left values to mix in")
        q, own = ops.attention_rows(
            proj, self.nh * self.maps, self.nkv * self.maps, self.nkv, self.d, self.dv, self.dtype, k_cache, v_cache,
            site.part(0).pages.slots if site.writes_cache else None, bias=self.bias, q_weight=self.q_norm,
            k_weight=self.k_norm, eps=self.eps, table=table, rot=rot, half=self.half, positions=batch.positions,
            mix_from=earlier, mix=self.mix, keep_values=self.values == "keep")
        if own is not None:
            batch.passing[PASSED_VALUES] = own
        return q
