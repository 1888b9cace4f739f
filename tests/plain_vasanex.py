"""The Vasanex decoder in plain, slow PyTorch on the CPU: one function per mechanism, written from the design's
equations, sharing no code with the engine.  Everything is computed in the dtype of the tensors it is given (the
tests hand it float64 copies of the weights); a whole sequence at a time, token by token where a recurrence asks
for it.

Notation: h [T, width] is a mixer's or feed-forward's input for the T tokens of one sequence, positions
0 .. T - 1; ``w`` maps tensor names to tensors; ``p`` is the prefix of the part's tensors.
"""
from __future__ import annotations

from typing import Dict, List

import torch

GATE_SLOPE = 1.702


def divided_by_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def one_plus_rms_norm(x, weight, eps):
    return divided_by_rms(x, eps) * (1.0 + weight)


def biased(h, w, name):
    return h @ w[name].T + w[name + ".b"]


def rotate_halves(x, positions, dims, base):
    """x [T, heads, d]: entry i meets entry i + dims / 2, i < dims / 2; entries from ``dims`` on pass."""
    half = dims // 2
    freqs = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    angle = positions.to(torch.float64)[:, None] * freqs[None, :]
    cos, sin = torch.cos(angle).to(x.dtype)[:, None, :], torch.sin(angle).to(x.dtype)[:, None, :]
    out = x.clone()
    out[..., :half] = x[..., :half] * cos - x[..., half:dims] * sin
    out[..., half:dims] = x[..., half:dims] * cos + x[..., :half] * sin
    return out


def visible(T, size):
    """[T, T]: row i sees column j where 0 <= i - j < size (size None: every j <= i)."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (back >= 0) if size is None else (back >= 0) & (back < size)


def softmax_with_sink(scores, mask, sink):
    """Rows of weights; exp(sink) is one more term of the denominator."""
    scores = scores.masked_fill(~mask, float("-inf"))
    top = torch.maximum(scores.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def attention(h, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, first_values=None):
    """Returns (output, this layer's values before any mixing)."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = divided_by_rms(biased(h, w, p + "q"), eps) * w[p + "q.norm"]      # the whole row at once
    k = divided_by_rms(biased(h, w, p + "k"), eps) * w[p + "k.norm"]
    own = biased(h, w, p + "v")
    v = own
    if m.get("v_mix") and first_values is not None:
        v = (1.0 - w[p + "vmix"]) * own + w[p + "vmix"] * first_values
    q, k, v = q.view(T, H, d), k.view(T, G, d), v.view(T, G, dv)
    rot = m.get("rot")
    if rot and rot.get("dims"):
        positions = torch.arange(T)
        q = rotate_halves(q, positions, rot["dims"], rot["base"])
        k = rotate_halves(k, positions, rot["dims"], rot["base"])
    mask = visible(T, m["mask"]["size"] if m.get("mask") else None)
    heads = []
    for head in range(H):
        g = head // (H // G)
        weights = softmax_with_sink((q[:, head] @ k[:, g].T) * m["scale"], mask, w[p + "sink"][head])
        heads.append(weights @ v[:, g])
    return biased(torch.cat(heads, dim=-1), w, p + "o"), own


def capped(x, cap):
    return cap * torch.tanh(x / cap)


def matrix_memory(h, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    """The mLSTM mixer, token by token."""
    T = h.shape[0]
    H, d, dv, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ w[p + "q"].T).view(T, H, d) / d ** 0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, dv)
    log_in = capped(biased(h, w, p + "i"), cap)
    log_keep = torch.nn.functional.logsigmoid(capped(biased(h, w, p + "f"), cap))
    out = h.new_zeros((T, H, dv))
    for head in range(H):
        S, n, top = h.new_zeros((d, dv)), h.new_zeros(d), h.new_zeros(())
        for t in range(T):
            new_top = torch.maximum(log_keep[t, head] + top, log_in[t, head])
            keep, write = torch.exp(log_keep[t, head] + top - new_top), torch.exp(log_in[t, head] - new_top)
            S = keep * S + write * torch.outer(k[t, head], v[t, head])
            n = keep * n + write * k[t, head]
            top = new_top
            bottom = torch.maximum((n @ q[t, head]).abs(), torch.exp(-top)) + 1e-6
            out[t, head] = (S.T @ q[t, head]) / bottom
    y = divided_by_rms(out, eps).reshape(T, H * dv) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    return y @ w[p + "o"].T


def clamped_gated_mlp(h, w, p: str, limit: float):
    gate = (h @ w[p + "gate"].T).clamp(max=limit)
    up = (h @ w[p + "up"].T).clamp(min=-limit, max=limit)
    return (gate * torch.sigmoid(GATE_SLOPE * gate) * (up + 1.0)) @ w[p + "down"].T


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], keep_layers: bool = False):
    """Logits [T, vocab] of one sequence; with ``keep_layers`` also the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    first_values, after = None, []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = one_plus_rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y, own = attention(h, w, p + "mix.", m, eps, first_values)
            if m.get("v_mix") and first_values is None:
                first_values = own
        elif layer["type"] == "mlstm":
            y = matrix_memory(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp"):
            x = x + clamped_gated_mlp(one_plus_rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"]["limit"])
        after.append(x)
    logits = one_plus_rms_norm(x, w["final.norm"], eps) @ w["embed"].T
    return (logits, after) if keep_layers else logits
