"""The Nogosun decoder in plain, slow PyTorch on the CPU: one function per mechanism, written from the design's
equations, sharing no code with the engine.  Everything is computed in the dtype of the tensors it is given (the
tests hand it float64 copies of the weights); a whole sequence at a time, token by token where a recurrence asks
for it.

Notation: h [T, width] is a mixer's or feed-forward's input for the T tokens of one sequence, positions
0 .. T - 1; ``w`` maps tensor names to tensors; ``p`` is the prefix of the part's tensors.
"""
from __future__ import annotations

import math
from typing import Dict, List

import torch


def divided_by_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return divided_by_rms(x, eps) * weight


def linear(h, w, name):
    return h @ w[name].T


def biased(h, w, name):
    return linear(h, w, name) + w[name + ".b"]


# ------------------------------------------------------------------ positions
def stretched_frequencies(dims, base, scaling):
    """(frequency of each pair, factor of cosines and sines)."""
    freqs = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freqs, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_with(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))

    low = max(math.floor(pair_with(scaling["fast"])), 0)
    high = min(math.ceil(pair_with(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(x, positions, rot):
    """x [T, heads, d]: entry i meets entry i + dims / 2, i < dims / 2; entries from ``dims`` on pass."""
    dims, half = rot["dims"], rot["dims"] // 2
    freqs, magnitude = stretched_frequencies(dims, rot["base"], rot.get("scaling"))
    angle = positions.to(torch.float64)[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :]
    cos = (torch.cos(angle) * magnitude).to(x.dtype)[:, None, :]
    sin = (torch.sin(angle) * magnitude).to(x.dtype)[:, None, :]
    out = x.clone()
    out[..., :half] = x[..., :half] * cos - x[..., half:dims] * sin
    out[..., half:dims] = x[..., half:dims] * cos + x[..., :half] * sin
    return out


def query_temperature(positions, coef, every):
    return 1.0 + coef * torch.log(torch.floor((positions.to(torch.float64) + 1) / every) + 1)


# ------------------------------------------------------------------ attention
def visible(T, size=None, keep_first=0):
    """[T, T]: row i sees column j <= i where i - j < size or j < keep_first (size None: every j <= i)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen if size is None else seen & ((i - j < size) | (j < keep_first))


def softmax(scores, mask, one_more=False):
    """Rows of weights over the visible; ``one_more``: 1 is added to the denominator."""
    scores = scores.masked_fill(~mask, float("-inf"))
    top = scores.max(dim=-1, keepdim=True).values
    if one_more:
        top = top.clamp(min=0.0)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + (torch.exp(-top) if one_more else 0.0))


def softcapped(scores, cap):
    return cap * torch.tanh(scores / cap)


def attention_values_are_keys(h, w: Dict[str, torch.Tensor], p: str, m: dict):
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q, k = biased(h, w, p + "q").view(T, H, d), biased(h, w, p + "k").view(T, G, d)
    v = k
    if m.get("rot"):
        positions = torch.arange(T)
        q, k = rotate_halves(q, positions, m["rot"]), rotate_halves(k, positions, m["rot"])
    mask = visible(T, m["mask"]["size"], m["mask"].get("keep_first", 0)) if m.get("mask") else visible(T)
    heads = []
    for head in range(H):
        g = head // (H // G)
        heads.append(softmax((q[:, head] @ k[:, g].T) * m["scale"], mask) @ v[:, g])
    return linear(torch.cat(heads, dim=-1), w, p + "o")


def attention_capped(h, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(biased(h, w, p + "q").view(T, H, d), w[p + "q.norm"], eps)
    k = rms_norm(biased(h, w, p + "k").view(T, G, d), w[p + "k.norm"], eps)
    v = biased(h, w, p + "v").view(T, G, dv)
    t = m["q_temp"]
    q = q * query_temperature(torch.arange(T), t["coef"], t["every"]).to(q.dtype)[:, None, None]
    heads = []
    for head in range(H):
        g = head // (H // G)
        scores = softcapped((q[:, head] @ k[:, g].T) * m["scale"], m["softcap"])
        heads.append(softmax(scores, visible(T), one_more=True) @ v[:, g])
    return linear(torch.cat(heads, dim=-1) * torch.sigmoid(linear(h, w, p + "g")), w, p + "o")


# ------------------------------------------------------------------ recurrences
def gated_linear_attention(h, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = linear(h, w, p + "q").view(T, H, d) * d ** -0.5
    k, v = linear(h, w, p + "k").view(T, H, d), linear(h, w, p + "v").view(T, H, dv)
    z = linear(linear(h, w, p + "a1"), w, p + "a2") + w[p + "a2.b"]
    keep = (torch.sigmoid(z) ** (1.0 / m["tau"])).view(T, H, d)
    out = h.new_zeros((T, H, dv))
    for head in range(H):
        S = h.new_zeros((d, dv))
        for t in range(T):
            S = keep[t, head][:, None] * S + torch.outer(k[t, head], v[t, head])
            out[t, head] = S.T @ q[t, head]
    y = rms_norm(out, w[p + "norm"], eps).reshape(T, H * dv)
    return linear(y * torch.nn.functional.silu(linear(h, w, p + "g")), w, p + "o")


def parallel(h, w, p, m, eps):
    return (m["left_scale"] * attention_capped(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * gated_linear_attention(h, w, p + "right.", m["right"], eps))


def short_convolution(x, taps):
    """x [T, channels], taps [channels, K]: the last column meets the current token, zeros before the start."""
    K = taps.shape[1]
    padded = torch.cat([x.new_zeros((K - 1, x.shape[1])), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(K))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_delta(h, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    silu = torch.nn.functional.silu
    q, k, v = (silu(short_convolution(linear(h, w, p + n), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d)), v.view(T, H, dv)
    beta = torch.sigmoid(linear(h, w, p + "b"))
    step = torch.nn.functional.softplus(linear(linear(h, w, p + "a1"), w, p + "a2") + w[p + "dt_bias"]).view(T, H, d)
    keep = torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * step)
    out = h.new_zeros((T, H, dv))
    for head in range(H):
        g = head // (H // G)
        S = h.new_zeros((d, dv))
        for t in range(T):
            S = keep[t, head][:, None] * S
            u = beta[t, head] * (v[t, head] - S.T @ k[t, g])
            S = S + torch.outer(k[t, g], u)
            out[t, head] = S.T @ q[t, g]
    y = rms_norm(out, w[p + "norm"], eps).reshape(T, H * dv)
    return linear(y * torch.sigmoid(linear(linear(h, w, p + "g1"), w, p + "g2")), w, p + "o")


# ------------------------------------------------------------------ feed-forward
def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def routing(h, router, top):
    """(chosen experts [T, top], their scores)."""
    scores = torch.softmax(h @ router.T, dim=-1)
    picked = scores.topk(top, dim=-1)
    return picked.indices, picked.values


def experts(h, w: Dict[str, torch.Tensor], p: str, mlp: dict):
    ids, weights = routing(h, w[p + "router"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t].tolist(), weights[t]):
            out[t] += s * (w[f"{p}e{e}.down"] @ gelu_erf(w[f"{p}e{e}.up"] @ h[t]))
    return out


# ------------------------------------------------------------------ the whole
def weights_of(cfg: dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], keep_layers: bool = False):
    """Logits [T, vocab] of one sequence; with ``keep_layers`` also the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{weights_of(cfg, i)}.", layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = attention_values_are_keys(h, w, p + "mix.", m)
        elif layer["type"] == "channel_delta":
            y = channel_delta(h, w, p + "mix.", m, eps)
        elif layer["type"] == "parallel":
            y = parallel(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        if layer.get("mlp"):
            y = y + experts(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
        x = x + y
        after.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return (logits, after) if keep_layers else logits
