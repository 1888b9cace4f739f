"""Tiny Nogosun configurations for the tests.  They differ in every size and option: the order of the three kinds of
layer, heads and kv heads (equal, one kv head for all, groups), key and value sizes (equal or not, multiples of four or
not), windows (one token, short, over several pages, none) and kept first tokens (none, one, over a page's edge, more than
the window), rotated entries (all, some, none; stretched or not), taps, the query temperature's steps, caps, the decay's
root, scales, experts (all of them chosen, one), layers without a feed-forward, layers that use another one's tensors (once,
twice, one that itself borrows) and the embedding's factor."""


def attention(heads, kv_heads, dim, scale, window=None, keep=None, rot_dims=None, base=10000.0, stretch=None):
    """``stretch``: (factor, original, fast, slow)"""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
        if keep is not None:
            m["mask"]["keep_first"] = keep
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
        if stretch:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), stretch))
    return {"type": "attention", "mixer": m}


def channel_delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def parallel(left, right, left_scale, right_scale):
    """``left``: (heads, kv_heads, dim, vdim, scale, softcap, coef, every); ``right``: (heads, dim, vdim, tau)"""
    heads, kv_heads, dim, vdim, scale, softcap, coef, every = left
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap,
                 "q_temp": {"coef": coef, "every": every}},
        "right": dict(zip(("heads", "dim", "vdim", "tau"), right)), "left_scale": left_scale, "right_scale": right_scale}}


def layer(mixer, ff=None, experts=None, top=None):
    return dict(mixer, mlp={"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}} if ff else None)


def borrows(layers, j):
    """One more layer with layer j's tensors."""
    return dict(layers[j], weights_of=j)


_A = [
    layer(attention(4, 2, 16, 0.3, 9, 3, rot_dims=8, base=100.0, stretch=(3.0, 40, 6.0, 1.0)), 20, 5, 2),
    layer(parallel((4, 2, 12, 16, 0.4, 6.0, 0.7, 8), (2, 8, 12, 4.0), 0.7, 1.4), 16, 4, 1),
]
_A += [borrows(_A, 0), layer(channel_delta(4, 2, 8, 16, 3), None), borrows(_A, 1)]
N_A = {"architecture": "Nogosun", "vocab": 210, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
       "layers": _A}

# nothing divides by four; a window of one token, none in another layer; no rotation; all experts chosen; a single tap
_B = [
    layer(channel_delta(3, 3, 7, 5, 1), 11, 3, 3),
    layer(attention(3, 3, 10, 0.31, 1, 1, rot_dims=6, base=77.0), None),
    layer(attention(6, 2, 7, 0.4), 13, 6, 2),
    layer(parallel((3, 1, 10, 7, 0.35, 2.5, 1.3, 5), (3, 5, 9, 1.0), 1.0, -0.6), None),
]
_B += [borrows(_B, 3), borrows(_B, 2), layer(channel_delta(6, 2, 9, 3, 5), 9, 2, 1)]
_B.append(dict(_B[4], weights_of=4))
N_B = {"architecture": "Nogosun", "vocab": 131, "width": 50, "norm": {"eps": 3e-4}, "embedding": {"scale": 0.7},
       "layers": _B}

# sizes in powers of two, which every kernel with a fast form takes; a short window beside more kept tokens than it, and
# one over several pages
_C = [
    layer(attention(8, 2, 32, 0.18, 20, 37, rot_dims=16, base=100000.0, stretch=(4.0, 64, 32.0, 1.0)), 128, 8, 2),
    layer(parallel((8, 2, 64, 32, 0.125, 12.0, 0.6, 32), (4, 32, 64, 12.0), 1.3, 0.8), 64, 16, 4),
    layer(channel_delta(4, 2, 64, 32, 4), 128, 4, 2),
]
_C += [borrows(_C, 1), borrows(_C, 2), layer(attention(4, 4, 64, 0.12, 50, 5, rot_dims=64, base=500.0), None)]
N_C = {"architecture": "Nogosun", "vocab": 384, "width": 128, "norm": {"eps": 1e-6}, "embedding": {"scale": 9.3},
       "layers": _C}

ALL = {"A": (N_A, 4, 31), "B": (N_B, 8, 32), "C": (N_C, 16, 33)}
STD = 0.06      # spread of the random weights: every branch moves the logits


def random_configuration(seed):
    """A configuration drawn at random: every size, the layers' order and kinds, the masks, who borrows from whom."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 6)):
        if layers and rng.random() < 0.3:
            layers.append(borrows(layers, rng.randrange(len(layers))))
            continue
        kv = rng.choice([1, 2, 3])
        heads, dim, vdim = kv * rng.choice([1, 2, 3]), rng.choice([4, 6, 8, 12, 16, 32]), rng.choice([4, 5, 8, 16, 20])
        kind = rng.choice(["attention", "parallel", "delta"])
        if kind == "attention":
            rot = rng.choice([None, 2, 4, dim])
            window = rng.choice([None, 1, 2, 5, 16, 31, 64])
            mixer = attention(heads, kv, dim, rng.choice([0.1, 0.2, 0.35]), window, rng.choice([None, 0, 1, 4, 9, 40]),
                              rot_dims=min(rot, dim) if rot else None, base=rng.choice([100.0, 10000.0, 500000.0]),
                              stretch=rng.choice([None, (2.0, 32, 8.0, 1.0), (8.0, 100, 20.0, 2.0)]))
        elif kind == "parallel":
            mixer = parallel((heads, kv, dim, vdim, rng.choice([0.1, 0.3]), rng.choice([1.5, 8.0, 30.0]),
                              rng.choice([0.2, 0.9]), rng.choice([1, 7, 16])),
                             (rng.choice([1, 2, 4]), rng.choice([4, 7, 16]), rng.choice([5, 8, 24]), rng.choice([1.0, 8.0])),
                             rng.choice([0.5, 1.0, 1.3]), rng.choice([0.8, -1.1]))
        else:
            mixer = channel_delta(heads, kv, dim, vdim, rng.choice([1, 2, 4, 6]))
        experts = rng.choice([1, 3, 8])
        layers.append(layer(mixer, *((rng.choice([8, 12, 24]), experts, rng.randint(1, experts)) if rng.random() < 0.7 else ())))
    cfg = {"architecture": "Nogosun", "vocab": rng.choice([50, 257, 400]), "width": rng.choice([24, 40, 64, 72, 128]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}, "layers": layers}
    if rng.random() < 0.8:
        cfg["embedding"] = {"scale": rng.choice([0.5, 4.0, 9.5])}
    return cfg, rng.choice([4, 8, 16, 32])


def telling_weights(weights, seed):
    """The random weights with every learned number that sits behind the projections of a size at which leaving it out or
    taking another one's shows: the norms' weights, biases, the decays, taps; scores and routers with some spread."""
    import torch
    g = torch.Generator().manual_seed(seed)
    out = dict(weights)

    def fill(name, values):
        out[name] = values.to(weights[name].dtype)
    for name in sorted(weights):
        shape, last = tuple(weights[name].shape), name.split(".")[-1]
        if "norm" in last:
            fill(name, 1 + torch.randn(shape, generator=g) * 0.3)
        elif last == "b" and len(shape) == 1:
            fill(name, torch.randn(shape, generator=g) * (1.5 if ".a2." in name else 0.4))
        elif last in ("A_log", "dt_bias"):
            fill(name, torch.randn(shape, generator=g) - 1.0)
        elif last == "conv":
            fill(name, torch.randn(shape, generator=g) * 0.6)
        elif last in ("q", "k"):
            fill(name, weights[name].float() * 2.0)
        elif last in ("a2", "g2", "b"):
            fill(name, weights[name].float() * 8.0)
        elif last == "router":
            fill(name, weights[name].float() * 5.0)
    return out
