"""Tiny Vasanex configurations for the tests.  They differ in every size and option: the order of the two kinds of
layer, heads and kv heads (equal, one kv head for all, a group of three), key and value sizes (equal or not, multiples
of four or not), windows that differ between layers (one token, short, long, none), rotated entries (all of a head's,
some, none), which layers mix values (not the first attention layer, only one, none), the gates' caps, the
feed-forwards' widths and limits (or no feed-forward, behind either kind of mixer) and the embedding's factor."""


def attention(heads, kv_heads, dim, vdim, scale, window=None, rot_dims=None, base=10000.0, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix}
    if window:
        m["mask"] = {"size": window}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
    return {"type": "attention", "mixer": m}


def mlstm(heads, dim, vdim, gate_cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}}


def layer(mixer, ff=None, limit=None):
    return dict(mixer, mlp={"kind": "dense", "ff": ff, "limit": limit} if ff else None)


# attention first; the first attention layer mixes nothing; windows of 9 and 21; a feed-forward behind a memory
V_A = {
    "architecture": "Vasanex", "vocab": 210, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
    "layers": [
        layer(attention(4, 2, 16, 24, 0.3, 9, rot_dims=8, base=100.0), 40, 0.7),
        layer(mlstm(2, 16, 8, 5.0), 32, 2.0),
        layer(attention(2, 1, 12, 16, 0.25, 21, rot_dims=12, base=500.0, v_mix=True), None),
        layer(mlstm(3, 8, 24, 9.0), None),
        layer(attention(6, 1, 8, 16, 0.4, 14, v_mix=True), 48, 0.4),
    ],
}

# nothing divides by four; a window of one token, none in another layer; no rotation; every head its own kv head
V_B = {
    "architecture": "Vasanex", "vocab": 131, "width": 50, "norm": {"eps": 3e-6}, "embedding": {"scale": 0.7},
    "layers": [
        layer(mlstm(3, 7, 5, 2.5), None),
        layer(attention(3, 3, 10, 7, 0.31, None, rot_dims=6, base=77.0, v_mix=True), 30, 1.1),
        layer(attention(6, 3, 14, 7, 0.22, 1, rot_dims=14, base=900.0, v_mix=True), 22, 3.0),
        layer(attention(9, 3, 6, 7, 0.5, 6, v_mix=True), None),
        layer(mlstm(1, 11, 9, 15.0), 34, 0.5),
    ],
}

# sizes in powers of two, which every kernel with a fast form takes; a short window and one over several pages
V_C = {
    "architecture": "Vasanex", "vocab": 384, "width": 128, "norm": {"eps": 1e-6}, "embedding": {"scale": 11.3},
    "layers": [
        layer(attention(8, 2, 32, 64, 0.18, 100, rot_dims=16, base=100000.0, v_mix=True), 256, 1.5),
        layer(mlstm(4, 32, 32, 12.0), 128, 0.8),
        layer(mlstm(2, 64, 64, 6.0), None),
        layer(attention(16, 2, 64, 64, 0.125, 33, rot_dims=64, base=10000.0, v_mix=True), 128, 6.0),
        layer(attention(4, 4, 16, 32, 0.25, None, rot_dims=8), 256, 1.0),
    ],
}

ALL = {"A": (V_A, 4, 21), "B": (V_B, 8, 22), "C": (V_C, 16, 23)}
STD = 0.05      # spread of the random weights: every branch moves the logits


def random_configuration(seed):
    """A configuration drawn at random: every size, the layers' order and kinds, the windows, what is mixed."""
    import random
    rng = random.Random(seed)
    layers, values = [], (rng.choice([1, 2, 3]), rng.choice([4, 7, 8, 16, 24]))
    for _ in range(rng.randint(1, 5)):
        if rng.random() < 0.6:
            v_mix = rng.random() < 0.6
            kv, vdim = values if v_mix else (rng.choice([1, 2]), rng.choice([4, 5, 16]))
            dim = rng.choice([4, 6, 8, 12, 16, 32])
            rot = rng.choice([None, 2, 4, dim])
            mixer = attention(kv * rng.choice([1, 2, 3, 5]), kv, dim, vdim, rng.choice([0.1, 0.2, 0.35]),
                              rng.choice([None, 1, 2, 5, 16, 31, 64]), rot_dims=min(rot, dim) if rot else None,
                              base=rng.choice([100.0, 10000.0, 500000.0]), v_mix=v_mix)
        else:
            mixer = mlstm(rng.choice([1, 2, 3, 4]), rng.choice([4, 7, 8, 16, 32]), rng.choice([4, 5, 8, 16, 31]),
                          rng.choice([1.5, 6.0, 15.0]))
        layers.append(layer(mixer, *((rng.choice([16, 24, 40]), rng.choice([0.3, 1.0, 7.0])) if rng.random() < 0.7 else ())))
    cfg = {"architecture": "Vasanex", "vocab": rng.choice([50, 257, 400]), "width": rng.choice([24, 40, 64, 72, 128]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}, "layers": layers}
    if rng.random() < 0.8:
        cfg["embedding"] = {"scale": rng.choice([0.5, 4.0, 9.5])}
    return cfg, rng.choice([4, 8, 16, 32])


def telling_weights(weights, seed):
    """The random weights with every learned number that sits behind the projections of a size at which leaving it out or
    taking another one's shows: biases, sinks, the mixing numbers, the norms' weights, the memory's gates (their rows
    so large that the gates move by several units from token to token)."""
    import torch
    g = torch.Generator().manual_seed(seed)
    out = dict(weights)

    def fill(name, values):
        out[name] = values.to(weights[name].dtype)
    for name in sorted(weights):
        shape, last = tuple(weights[name].shape), name.split(".")[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            fill(name, torch.randn(shape, generator=g) * 0.3)
        elif last == "norm":
            fill(name, 1 + torch.randn(shape, generator=g) * 0.3)
        elif last == "sink":
            fill(name, torch.randn(shape, generator=g) * 1.5)
        elif last == "vmix":
            fill(name, torch.rand(shape, generator=g) * 0.6 + 0.2)
        elif last == "b":
            fill(name, torch.randn(shape, generator=g) * (1.5 if name.split(".")[-2] in ("i", "f") else 0.4))
        elif last in ("i", "f"):
            fill(name, weights[name].float() * 8.0)
        elif last in ("q", "k"):
            fill(name, weights[name].float() * 2.0)
    return out
