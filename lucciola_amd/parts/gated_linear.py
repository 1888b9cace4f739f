"""Gated linear attention as a part: linear attention whose state forgets per key channel at a rate that the token
decides.

With h the mixer's input, H heads, ``key_dim`` query/key and ``value_dim`` value entries a head:
  q = W_q h / sqrt(key_dim), k = W_k h, v = W_v h, head by head;
  alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau), one number per head and key channel;
  per head, from a state S [key, value] of zeros:  S <- diag(alpha) S + k v^T,  o = S^T q;
  every head's o divided by its root mean square (``norm_eps`` inside the root) and weighed (one weight for all
  heads), the heads side by side times silu(W_g h), then W_o.
The state is float32 and belongs to the request (a slot per live request, zeroed when it starts there); the projections
leave as float32 and everything up to the gated read-out stays float32.  The recurrence is the framework's scan
(``ops.delta_scan``) without a removal term, with decay = alpha, write = k, read = q: a step's tokens are walked in order
within each request from the slot's state, whatever the cut of the prompt.
"""
from __future__ import annotations

from typing import Dict

import torch

from ..cache.specs import FixedStates
from ..config.registry import MIXERS
from ..kernels import ops
from ..weights.loader import ParamDecl
from .base import BuildContext, Part
from .feed_forward import low_rank_outer, stack_rows


@MIXERS.register("gated_linear")
class GatedLinear(Part):
    graph_safe = True   # launches only kernels whose arguments stay put between steps

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, tau: float, norm_eps: float):
        super().__init__(hidden_size=hidden_size, num_heads=num_heads, key_dim=key_dim, value_dim=value_dim, tau=tau,
                         norm_eps=norm_eps)
        self.H, self.nh, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.tau, self.norm_eps = float(tau), float(norm_eps)
        if not self.tau > 0:
            raise ValueError(f"gated_linear: tau {tau} must be positive")
        ops.check_delta_sizes("gated_linear", self.dk, self.dv)

    def declare(self) -> Dict[str, ParamDecl]:
        nk, nv = self.nh * self.dk, self.nh * self.dv
        # the inner size of the decay's two small matrices is whatever the checkpoint holds
        return {"q": ParamDecl((nk, self.H)), "k": ParamDecl((nk, self.H)), "v": ParamDecl((nv, self.H)),
                "gate": ParamDecl((nv, self.H)), "rate_in": ParamDecl((-1, self.H)), "rate_out": ParamDecl((nk, -1)),
                "rate_bias": ParamDecl((nk,), role="vector"),
                "norm": ParamDecl((self.dv,), role="vector", init="ones_plus_normal"), "o": ParamDecl((self.H, nv))}

    def bind(self, tensors, ctx: BuildContext) -> None:
        self.dtype = ctx.dtype
        # the decay's inner product rides along in the projection
        self.proj = stack_rows([tensors[k] for k in ("q", "k", "v", "gate", "rate_in")])
        self.gate_column = self.nh * (2 * self.dk + self.dv)
        self.rank_column, self.rank = self.gate_column + self.nh * self.dv, tensors["rate_in"].shape[0]
        self.outer = low_rank_outer((tensors["rate_in"],), (tensors["rate_out"],), ctx.dtype == torch.bfloat16)
        self.rate_bias, self.norm = (tensors[k].to(torch.float32).contiguous() for k in ("rate_bias", "norm"))
        self.o = tensors["o"]

    def cache_need(self):
        return FixedStates(((self.nh, self.dv, self.dk),))

    def forward(self, x: torch.Tensor, site) -> torch.Tensor:
        batch = site.batch
        (state,) = site.cache
        proj = ops.gemm(x, self.proj, torch.float32)
        inner = ops.columns(proj, self.rank_column, self.rank, self.outer.shape[1], self.dtype)
        rates = ops.gemm(inner, self.outer, torch.float32)
        coef, v = ops.gated_linear_prepare(proj, rates, 0, self.rate_bias, 1.0 / self.tau, self.dk ** -0.5, self.nh,
                                           self.dk, self.dv)
        o = ops.delta_scan(coef, v, state, batch.q_offsets, batch.slot_ids, batch.num_requests, self.nh, self.dk,
                           self.dv)
        y = ops.head_gate_norm(o, proj, self.gate_column, self.norm, False, self.norm_eps, "silu", self.nh, self.dv, self.dtype)
        return ops.gemm(y, self.o, self.dtype, defer=True)
