"""The matrix memory of the xLSTM (mLSTM) as a part: a linear attention whose input and forget gates are
exponentials of learned functions of the token, held in range by a running reference point.

With h the mixer's input, H heads, ``key_dim`` query/key and ``value_dim`` value entries a head, ``cap`` > 0:
  q = W_q h / sqrt(key_dim), k = W_k h, v = W_v h, head by head;
  i = cap tanh((W_i h + b_i) / cap),  f = logsigmoid(cap tanh((W_f h + b_f) / cap)), one number a head each;
  per head, from S [key, value], n [key] and m of zeros:
    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- e^(f + m - m') n + e^(i - m') k;  m <- m'
    o = S^T q / (max(|n . q|, e^(-m)) + floor)
  each head's o divided by its root mean square (``norm_eps`` inside the root); the heads side by side times a
  weight, times sigmoid(W_g h), then W_o.
S, n and m are float32 and belong to the request (a slot per live request, zeroed when it starts there); the
projections leave as float32 and everything up to the gated read-out stays float32.  The normaliser n is kept as one
more value channel of S whose value is always 1, and the recurrence is the framework's scan (``ops.delta_scan``)
without a removal term, with decay = e^(f + m - m') in every key channel, write = e^(i - m') k, read = q: a step's
tokens are walked in order within each request from the slot's state, whatever the cut of the prompt.
"""
from __future__ import annotations

from typing import Dict

import torch

from ..cache.specs import FixedStates
from ..config.registry import MIXERS
from ..kernels import ops
from ..weights.loader import ParamDecl
from .base import BuildContext, Part
from .feed_forward import stack_rows


@MIXERS.register("mlstm")
class MatrixMemory(Part):
    graph_safe = True   # launches only kernels whose arguments stay put between steps

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, cap: float, norm_eps: float,
                 floor: float = 1e-6):
        super().__init__(hidden_size=hidden_size, num_heads=num_heads, key_dim=key_dim, value_dim=value_dim, cap=cap,
                         norm_eps=norm_eps, floor=floor)
        self.H, self.nh, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.cap, self.norm_eps, self.floor = float(cap), float(norm_eps), float(floor)
        if not self.cap > 0:
            raise ValueError(f"mlstm: the gates' cap {cap} must be positive")
        ops.check_delta_sizes("mlstm", self.dk, self.dv)

    def declare(self) -> Dict[str, ParamDecl]:
        nk, nv = self.nh * self.dk, self.nh * self.dv
        return {"q": ParamDecl((nk, self.H)), "k": ParamDecl((nk, self.H)), "v": ParamDecl((nv, self.H)),
                "g": ParamDecl((nv, self.H)), "i": ParamDecl((self.nh, self.H)), "f": ParamDecl((self.nh, self.H)),
                "i_bias": ParamDecl((self.nh,), role="vector"), "f_bias": ParamDecl((self.nh,), role="vector"),
                "norm": ParamDecl((nv,), role="vector", init="ones_plus_normal"), "o": ParamDecl((self.H, nv))}

    def bind(self, tensors, ctx: BuildContext) -> None:
        self.dtype = ctx.dtype
        self.proj = stack_rows([tensors[k] for k in ("q", "k", "v", "g", "i", "f")])
        self.gate_column = self.nh * (2 * self.dk + self.dv)
        self.i_column = self.gate_column + self.nh * self.dv
        self.i_bias, self.f_bias, self.norm = (tensors[k].to(torch.float32).contiguous()
                                               for k in ("i_bias", "f_bias", "norm"))
        self.o = tensors["o"]

    def cache_need(self):
        return FixedStates(((self.nh, self.dv + 1, self.dk), (self.nh,)))

    def forward(self, x: torch.Tensor, site) -> torch.Tensor:
        batch = site.batch
        state, reference = site.cache
        proj = ops.gemm(x, self.proj, torch.float32)
        coef, v, bottoms = ops.mlstm_prepare(proj, self.nh, self.dk, self.dv, self.i_column, self.i_column + self.nh,
                                             self.i_bias, self.f_bias, self.cap, self.dk ** -0.5, reference,
                                             batch.q_offsets, batch.slot_ids, batch.num_requests)
        o = ops.delta_scan(coef, v, state, batch.q_offsets, batch.slot_ids, batch.num_requests, self.nh, self.dk,
                           self.dv + 1)
        y = ops.mlstm_readout(o, bottoms, self.floor, proj, self.gate_column, self.norm, self.norm_eps, self.nh,
                              self.dv, self.dtype)
        return ops.gemm(y, self.o, self.dtype, defer=True)
