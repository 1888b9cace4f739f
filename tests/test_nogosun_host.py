"""The Nogosun design on the CPU: its configuration and what is refused, its tensors, what its layers need of the cache,
the plain implementation's mechanisms against hand-made cases, and the engine's host logic (step function, cache, state
slots, kept pages, layers that borrow tensors, batches) with the plain torch versions of the kernels put in their place,
against the plain whole-sequence implementation."""
import copy
import math

import pytest
import torch

import nogosun_configs as nc
import plain_nogosun
import reference_ops
import traces
from helpers import compare, make_runner, prompts_for, random_weights, replay
from lucciola_amd import models  # noqa: F401  (registers the architectures)
from lucciola_amd.cache.manager import CacheManager
from lucciola_amd.cache.specs import FixedStates, PagedRows
from lucciola_amd.config.engine_config import EngineConfig
from lucciola_amd.config.model_config import ConfigError
from lucciola_amd.config.nogosun_config import NogosunConfig
from lucciola_amd.config.registry import architecture_for
from lucciola_amd.engine.batch import StepEntry
from lucciola_amd.engine.llm_engine import LLMEngine
from lucciola_amd.engine.loading import _build
from lucciola_amd.kernels import ops
from lucciola_amd.models.causal_lm import declared_tensors
from lucciola_amd.models.nogosun import nogosun_model_spec
from lucciola_amd.parts.delta_rule import ChannelDelta
from lucciola_amd.parts.feed_forward import RoutedMLP, low_rank_outer
from lucciola_amd.parts.gated_linear import GatedLinear
from lucciola_amd.parts.masked_attention import MaskedAttention
from lucciola_amd.sampling.sampler import SamplingParams
from lucciola_amd.weights.loader import DictSource

LENGTHS = {"A": [1, 12, 45], "B": [2, 40, 21], "C": [70, 9]}


def weights_for(cfg, seed, std=nc.STD):
    return nc.telling_weights(random_weights(cfg, seed, std=std), seed)


def plain_weights(weights):
    return {k: v.to(torch.float64) for k, v in weights.items()}


def plain_logits(cfg, weights, prompts):
    w = plain_weights(weights)
    return {n: plain_nogosun.forward(cfg, w, ids) for n, ids in prompts.items()}


def greedy(cfg, weights, prompt, count):
    w = plain_weights(weights)
    ids = list(prompt)
    for _ in range(count):
        ids.append(int(torch.argmax(plain_nogosun.forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]


# ------------------------------------------------------------------ configuration, tensors, cache
def test_configuration_is_read_layer_by_layer():
    cfg = NogosunConfig.from_dict(nc.N_A)
    assert (cfg.vocab, cfg.width, cfg.norm_eps, cfg.embedding_scale) == (210, 64, 1e-5, 3.0)
    assert [l.type for l in cfg.layers] == ["attention", "parallel", "attention", "channel_delta", "parallel"]
    a = cfg.layers[0].mixer
    assert (a.heads, a.kv_heads, a.dim, a.scale, a.window, a.keep_first) == (4, 2, 16, 0.3, 9, 3)
    assert (a.rot.dims, a.rot.base) == (8, 100.0)
    assert a.rot.scaling.to_dict() == {"factor": 3.0, "original": 40.0, "fast": 6.0, "slow": 1.0}
    p = cfg.layers[1].mixer
    assert (p.left.heads, p.left.kv_heads, p.left.dim, p.left.vdim, p.left.scale, p.left.softcap) == (4, 2, 12, 16, 0.4, 6.0)
    assert p.left.temperature == (0.7, 8.0) and (p.left_scale, p.right_scale) == (0.7, 1.4)
    assert (p.right.heads, p.right.dim, p.right.vdim, p.right.tau) == (2, 8, 12, 4.0)
    d = cfg.layers[3].mixer
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.conv) == (4, 2, 8, 16, 3) and cfg.layers[3].mlp is None
    assert (cfg.layers[0].mlp.ff, cfg.layers[0].mlp.experts, cfg.layers[0].mlp.top) == (20, 5, 2)
    assert [l.weights_of for l in cfg.layers] == [0, 1, 0, 3, 1]
    other = NogosunConfig.from_dict({k: v for k, v in nc.N_B.items() if k != "embedding"})
    assert other.embedding_scale == 1.0
    assert [l.weights_of for l in other.layers] == [0, 1, 2, 3, 3, 2, 6, 3]
    assert other.layers[2].mixer.window is None and other.layers[2].mixer.rot is None
    assert other.layers[1].mixer.rot.scaling is None
    assert architecture_for(nc.N_B).name == "Nogosun"


def _at(i, *keys):
    def find(c):
        d = c["layers"][i]
        for k in keys:
            d = d[k]
        return d
    return find


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="mlstm"), "not a mixer"),
    (lambda c: _at(0, "mixer")(c).update(kv_heads=3), "multiple"),
    (lambda c: _at(0, "mixer")(c).update(vdim=8), "values are the keys"),
    (lambda c: _at(0, "mixer", "rot")(c).update(dims=7), "even"),
    (lambda c: _at(0, "mixer", "rot")(c).update(dims=18), "at most"),
    (lambda c: _at(0, "mixer", "rot")(c).update(base=1.0), "base"),
    (lambda c: _at(0, "mixer", "rot", "scaling")(c).pop("slow"), "slow"),
    (lambda c: _at(0, "mixer", "rot", "scaling")(c).update(factor=0), "positive"),
    (lambda c: _at(0, "mixer", "mask")(c).update(size=0), "at least 1"),
    (lambda c: _at(0, "mixer", "mask")(c).update(keep_first=-1), "at least 0"),
    (lambda c: _at(0, "mixer")(c).pop("scale"), "scale"),
    (lambda c: _at(1, "mixer", "left")(c).update(softcap=0.0), "positive"),
    (lambda c: _at(1, "mixer", "left")(c).pop("q_temp"), "q_temp"),
    (lambda c: _at(1, "mixer", "left", "q_temp")(c).update(every=0), "positive"),
    (lambda c: _at(1, "mixer", "right")(c).update(tau=0.0), "positive"),
    (lambda c: _at(1, "mixer")(c).pop("left_scale"), "left_scale"),
    (lambda c: _at(1, "mlp", "router")(c).update(top=9), "exceeds"),
    (lambda c: _at(1, "mlp")(c).update(kind="dense"), "not a feed-forward"),
    (lambda c: _at(3, "mixer")(c).update(conv=0), "at least 1"),
    (lambda c: c["layers"][2].update(weights_of=7), "leads to layer"),
    (lambda c: c["layers"][2].update(weights_of=2), "itself"),
    (lambda c: (c["layers"][0].update(weights_of=2)), "circle"),
    (lambda c: c["layers"][2].update(weights_of=1), "must equal"),
    (lambda c: c["layers"][2].update(mlp=None), "must equal"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c.update(layers=[]), "at least one"),
])
def test_configuration_refuses(change, message):
    cfg = copy.deepcopy(nc.N_A)
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        NogosunConfig.from_dict(cfg)


def test_tensors_blocks_and_borrowed_layers():
    spec = nogosun_model_spec(NogosunConfig.from_dict(nc.N_B))
    assert [e.layer for e in spec.run_order] == [0, 1, 2, 3, 3, 2, 4, 3]
    assert all(e.cache_of is None for e in spec.run_order)
    assert [l.block for l in spec.layers] == ["parallel_residual", "parallel_mixer", "parallel_residual", "parallel_mixer",
                                              "parallel_residual"]
    names = declared_tensors(spec)
    shapes = {n: d.shape for n, d in names.items()}
    assert shapes["embed"] == shapes["head"] == (131, 50) and shapes["final.norm"] == (50,)
    assert shapes["l0.mix.q"] == (21, 50) and shapes["l0.mix.q.conv"] == (21, 1) and shapes["l0.mix.v"] == (15, 50)
    assert shapes["l0.mix.b"] == (3, 50) and shapes["l0.mix.A_log"] == (3,) and shapes["l0.mix.dt_bias"] == (21,)
    assert shapes["l0.mix.a1"] == (-1, 50) and shapes["l0.mix.g2"] == (15, -1) and shapes["l0.mix.norm"] == (5,)
    assert shapes["l1.mix.k"] == (30, 50) and shapes["l1.mix.k.b"] == (30,) and shapes["l1.mix.o"] == (50, 30)
    assert not any(n in shapes for n in ("l1.mix.v", "l1.mix.o.b", "l1.norm2", "l1.mlp.router", "l4.norm1", "l5.mix.q"))
    assert shapes["l2.mix.q"] == (42, 50) and shapes["l2.mlp.e5.up"] == (13, 50) and shapes["l2.mlp.router"] == (6, 50)
    assert shapes["l3.mix.left.v.b"] == (7,) and shapes["l3.mix.left.q.norm"] == (10,) and shapes["l3.mix.left.g"] == (21, 50)
    assert shapes["l3.mix.right.a2"] == (15, -1) and shapes["l3.mix.right.a2.b"] == (15,)
    assert shapes["l6.mix.k.conv"] == (18, 5) and shapes["l6.mix.dt_bias"] == (54,) and shapes["l6.mix.norm"] == (3,)
    assert "l3.mix.left.sink" not in shapes


def test_what_the_layers_keep(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg, page, seed = nc.ALL["A"]
    runner = make_runner(cfg, weights_for(cfg, seed), page, 8, "float32", "cpu", max_seqs=3)
    windowed, both = PagedRows(32, 32, 9, 3), (PagedRows(24, 32), FixedStates(((2, 12, 8),)))
    assert runner.model.site_needs() == [windowed, both, windowed, FixedStates(((4, 16, 8), (2, 96))), both]
    assert len(runner.cache.groups) == 2 and runner.cache.has_fixed_state
    # a layer that borrows tensors has memory of its own
    assert runner.cache.storage[0][0][0].data_ptr() != runner.cache.storage[2][0][0].data_ptr()
    assert runner.cache.storage[1][1][0].data_ptr() != runner.cache.storage[4][1][0].data_ptr()


@pytest.mark.parametrize("keep,first_kept", [(0, 0), (1, 1), (4, 1), (5, 2), (30, 8)])
def test_pages_of_the_first_positions_stay(keep, first_kept):
    """Window 6, pages of 4: after 33 tokens the window needs positions 28 on, and the first pages if they are kept."""
    cache = CacheManager([PagedRows(8, 8, 6, keep)], 4, 20, 1)
    cache.admit("r")
    for n in (10, 3, 1, 1, 9, 2, 7):
        cache.reserve("r", n)
        cache.commit("r")
        cache.check()
    table = cache.block_table(0, "r")
    assert len(table) == 9
    kept = [i for i, page in enumerate(table) if page >= 0]
    assert kept == sorted(set(range(first_kept)) | {7, 8})
    cache.release("r")
    assert cache.num_free_blocks() == 20


def test_parts_refuse_what_no_kernel_has():
    sizes = dict(hidden_size=8, num_heads=2, num_kv_heads=1, head_dim=4, value_dim=4, scale=1.0, eps=1e-6)
    for more in (dict(head_norm=True, row_norm=True), dict(temperature=(1.0, 2.0), conv_taps=2),
                 dict(values="keys", maps=2), dict(head_norm=True, values="mix")):
        with pytest.raises(ValueError, match="no prologue kernel has both"):
            MaskedAttention(**sizes, **more)
    with pytest.raises(ValueError, match="values that are the keys"):
        MaskedAttention(**dict(sizes, value_dim=8), values="keys")
    with pytest.raises(ValueError, match="coef, every"):
        MaskedAttention(**sizes, temperature=(1.0, 0.0))
    with pytest.raises(ValueError, match="negative"):
        MaskedAttention(**sizes, softcap=-1.0)
    with pytest.raises(ValueError, match="tau"):
        GatedLinear(8, 1, 4, 4, 0.0, 1e-6)
    with pytest.raises(ValueError, match="multiple"):
        ChannelDelta(8, 3, 2, 4, 4, 2, 1e-6)
    with pytest.raises(ValueError, match="no kernel"):
        RoutedMLP(8, 8, 2, 1, activation="silu")
    with pytest.raises(ValueError, match="do not fit each other"):
        low_rank_outer((torch.zeros(3, 8),), (torch.zeros(5, 4),), False)


def test_low_rank_products_on_one_diagonal():
    g = torch.Generator().manual_seed(1)
    a1, a2, b1, b2 = (torch.randn(s, generator=g) for s in ((3, 8), (5, 3), (4, 8), (6, 4)))
    x = torch.randn(7, 8, generator=g)
    want = torch.cat([x @ a1.T @ a2.T, x @ b1.T @ b2.T], dim=1)
    for pad, rank in ((False, 7), (True, 128)):
        outer = low_rank_outer((a1, b1), (a2, b2), pad)
        assert outer.shape == (11, rank)
        inner = reference_ops.columns(torch.cat([x, x @ a1.T, x @ b1.T], dim=1), 8, 7, rank, torch.float32)
        assert torch.allclose(inner @ outer.T, want, atol=1e-5)


def test_branches_that_wait_together(monkeypatch):
    reference_ops.install(monkeypatch)
    a, b, c = (torch.full((2, 3), v) for v in (1.0, 10.0, 100.0))
    both = ops.summed((ops.summed((a, 2.0), (b, 0.5)), 3.0), (c, 1.0))
    assert [scale for _, scale in both.branches] == [6.0, 1.5, 1.0]
    assert both.value().tolist() == [[121.0] * 3] * 2
    assert ops.value(ops.summed((a, 4.0))).tolist() == [[4.0] * 3] * 2


# ------------------------------------------------------------------ the plain implementation by hand
def test_the_mask_by_hand():
    mask = plain_nogosun.visible(9, 3, 2)
    for i in range(9):
        assert mask[i].tolist() == [j <= i and (i - j < 3 or j < 2) for j in range(9)]
    assert plain_nogosun.visible(4).tolist() == [[j <= i for j in range(4)] for i in range(4)]


def test_the_stretched_rotation_by_hand():
    scaling = {"factor": 4.0, "original": 100, "fast": 5.0, "slow": 0.5}
    freqs, magnitude = plain_nogosun.stretched_frequencies(6, 50.0, scaling)
    low = max(math.floor(6 * math.log(100 / (2 * math.pi * 5)) / (2 * math.log(50))), 0)
    high = min(math.ceil(6 * math.log(100 / (2 * math.pi * 0.5)) / (2 * math.log(50))), 5)
    assert (low, high) == (0, 3)
    for i in range(3):
        f, ramp = 50.0 ** (-2 * i / 6), i / 3
        assert freqs[i] == pytest.approx(f / 4 * ramp + f * (1 - ramp))
    assert magnitude == pytest.approx(1 + 0.1 * math.log(4))
    x = torch.arange(1.0, 9.0, dtype=torch.float64).view(1, 1, 8)
    got = plain_nogosun.rotate_halves(x, torch.tensor([3]), {"dims": 6, "base": 50.0, "scaling": scaling})[0, 0].tolist()
    for i in range(3):
        c, s = magnitude * math.cos(3 * freqs[i]), magnitude * math.sin(3 * freqs[i])
        assert got[i] == pytest.approx((i + 1) * c - (i + 4) * s) and got[i + 3] == pytest.approx((i + 4) * c + (i + 1) * s)
    assert got[6:] == [7.0, 8.0]


def test_the_temperature_and_the_cap_by_hand():
    t = plain_nogosun.query_temperature(torch.arange(8), 0.5, 4).tolist()
    assert t[:3] == [1.0] * 3 and t[3:7] == pytest.approx([1 + 0.5 * math.log(2)] * 4)
    assert t[7] == pytest.approx(1 + 0.5 * math.log(3))
    s = plain_nogosun.softcapped(torch.tensor([-1e9, 0.0, 3.0, 1e9]), 2.0).tolist()
    assert s == pytest.approx([-2.0, 0.0, 2 * math.tanh(1.5), 2.0])


def test_one_more_in_the_denominator_by_hand():
    scores = torch.tensor([[0.0, 1.0], [-3.0, -2.0]], dtype=torch.float64)
    mask = torch.tensor([[True, False], [True, True]])
    w = plain_nogosun.softmax(scores, mask, one_more=True)
    assert w[0].tolist() == pytest.approx([0.5, 0.0])
    total = 1 + math.exp(-3) + math.exp(-2)
    assert w[1].tolist() == pytest.approx([math.exp(-3) / total, math.exp(-2) / total])
    assert plain_nogosun.softmax(scores, mask)[0].tolist() == [1.0, 0.0]


def test_values_are_the_keys_before_the_rotation_by_hand():
    """One head that sees only itself gives out its own biased key, whatever the rotation does to it."""
    e = torch.eye(4, dtype=torch.float64)
    w = {"x.q": e, "x.q.b": torch.zeros(4).double(), "x.k": 2 * e, "x.k.b": torch.ones(4).double(), "x.o": e}
    m = {"heads": 1, "kv_heads": 1, "dim": 4, "scale": 1.0, "mask": {"size": 1, "keep_first": 0},
         "rot": {"dims": 4, "base": 10.0}}
    h = torch.arange(12.0, dtype=torch.float64).view(3, 4)
    assert torch.allclose(plain_nogosun.attention_values_are_keys(h, w, "x.", m), 2 * h + 1)


def test_gated_linear_attention_by_hand():
    """One head of two key channels and one value: the state's channels forget at rates of their own."""
    h = torch.tensor([[1.0, 0.3], [-2.0, 0.8], [0.5, -1.1]], dtype=torch.float64)
    e = torch.eye(2, dtype=torch.float64)
    w = {"q": e, "k": e.flip(0), "v": e[:1], "g": e[1:], "norm": torch.tensor([2.0]).double(), "o": torch.ones(1, 1).double(),
         "a1": e[1:], "a2": torch.tensor([[1.0], [-2.0]]).double(), "a2.b": torch.tensor([0.1, 0.4]).double()}
    w = {"x." + k: v for k, v in w.items()}
    got = plain_nogosun.gated_linear_attention(h, w, "x.", {"heads": 1, "dim": 2, "vdim": 1, "tau": 3.0}, 1e-2)
    S = [0.0, 0.0]
    for t in range(3):
        a, b = h[t].tolist()
        z = [b + 0.1, -2 * b + 0.4]
        S = [(1 / (1 + math.exp(-z[c]))) ** (1 / 3) * S[c] + (b, a)[c] * a for c in range(2)]
        o = (S[0] * a + S[1] * b) / math.sqrt(2)
        assert got[t].item() == pytest.approx(2 * o / math.sqrt(o * o + 1e-2) * b / (1 + math.exp(-b)))


def test_the_channel_delta_rule_by_hand():
    """One head of two key channels and one value, one tap: the write sees the state after its decay, the read after the
    write."""
    h = torch.tensor([[1.0, 0.3], [-2.0, 0.8], [0.5, -1.1]], dtype=torch.float64)
    e = torch.eye(2, dtype=torch.float64)
    w = {"q": e, "k": e.flip(0), "v": e[:1], "b": e[1:], "A_log": torch.tensor([-0.5]).double(), "a1": e[1:],
         "a2": torch.tensor([[1.0], [-2.0]]).double(), "dt_bias": torch.tensor([0.1, 0.4]).double(), "g1": e[:1],
         "g2": torch.tensor([[0.7]]).double(), "norm": torch.tensor([2.0]).double(), "o": torch.ones(1, 1).double(),
         "q.conv": torch.ones(2, 1).double(), "k.conv": torch.ones(2, 1).double(), "v.conv": torch.tensor([[3.0]]).double()}
    w = {"x." + k: v for k, v in w.items()}
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 1, "conv": 1}
    got = plain_nogosun.channel_delta(h, w, "x.", m, 1e-2)

    def silu(z):
        return z / (1 + math.exp(-z))
    S = [0.0, 0.0]
    for t in range(3):
        a, b = h[t].tolist()
        size = math.sqrt(silu(a) ** 2 + silu(b) ** 2 + 1e-6)
        q, k = [silu(a) / size / math.sqrt(2), silu(b) / size / math.sqrt(2)], [silu(b) / size, silu(a) / size]
        step = [math.log1p(math.exp(b + 0.1)), math.log1p(math.exp(-2 * b + 0.4))]
        S = [math.exp(-math.exp(-0.5) * step[c]) * S[c] for c in range(2)]
        u = (silu(3 * a) - S[0] * k[0] - S[1] * k[1]) / (1 + math.exp(-b))
        S = [S[c] + k[c] * u for c in range(2)]
        o = S[0] * q[0] + S[1] * q[1]
        assert got[t].item() == pytest.approx(2 * o / math.sqrt(o * o + 1e-2) / (1 + math.exp(-0.7 * a)))


def test_the_short_convolution_by_hand():
    x = torch.tensor([[1.0], [10.0], [100.0]])
    assert plain_nogosun.short_convolution(x, torch.tensor([[3.0, 2.0]])).flatten().tolist() == [2.0, 23.0, 230.0]


def test_the_experts_by_hand():
    """Scores over all experts, not made to sum to one among the chosen."""
    h = torch.tensor([[1.0, 0.0], [0.0, 2.0]], dtype=torch.float64)
    e = torch.eye(2, dtype=torch.float64)
    w = {"x.router": torch.tensor([[2.0, 0.0], [0.0, 1.0], [1.0, 0.5]]).double()}
    for k in range(3):
        w[f"x.e{k}.up"], w[f"x.e{k}.down"] = e, (k + 1) * e
    got = plain_nogosun.experts(h, w, "x.", {"router": {"experts": 3, "top": 2}})
    gelu = 0.5 * (1 + math.erf(1 / math.sqrt(2)))
    s = [math.exp(z) / (math.exp(2) + 1 + math.exp(1)) for z in (2.0, 0.0, 1.0)]
    assert got[0].tolist() == pytest.approx([(s[0] + 3 * s[2]) * gelu, 0.0])
    gelu = 0.5 * 2 * (1 + math.erf(2 / math.sqrt(2)))
    s = [math.exp(z) / (1 + math.exp(2) + math.exp(1)) for z in (0.0, 2.0, 1.0)]
    assert got[1].tolist() == pytest.approx([0.0, (2 * s[1] + 3 * s[2]) * gelu])


# ------------------------------------------------------------------ the engine's host logic
@pytest.mark.parametrize("key", ["A", "B", "C"])
@pytest.mark.parametrize("family", ["whole", "tail", "chunked", "mixed"])
def test_step_function_matches_plain(monkeypatch, key, family):
    reference_ops.install(monkeypatch)
    cfg, page, seed = nc.ALL[key]
    weights = weights_for(cfg, seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, LENGTHS[key], seed)
    steps = {"whole": traces.whole, "tail": traces.tail_decode, "chunked": traces.chunked,
             "mixed": traces.mixed}[family](prompts)
    blocks = traces.max_live_tokens(steps, page) // page
    runner = make_runner(cfg, weights, page, blocks, "float32", "cpu")
    compare(replay(runner, steps), cfg, weights, prompts, 3e-5, plain_logits(cfg, weights, prompts))
    assert not runner.cache.requests
    for g in runner.cache.groups:
        assert g.pool.num_free() == blocks


def test_stream_after_every_layer(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg, page, seed = nc.ALL["A"]
    weights = weights_for(cfg, seed)
    ids = prompts_for({"vocab_size": cfg["vocab"]}, [19], seed)["r0"]
    _, want = plain_nogosun.forward(cfg, plain_weights(weights), ids, keep_layers=True)
    runner = make_runner(cfg, weights, page, 8, "float32", "cpu")
    seen = []
    for layer in runner.model.layers:
        block, inner = layer.block, layer.block.forward

        def spy(stream, site, inner=inner):
            inner(stream, site)
            seen.append((stream.h.double() + ops.value(stream.pending).double()).clone())
        block.forward = spy
    runner.step([StepEntry("r", ids[:7], [])])
    runner.step([StepEntry("r", ids[7:], [len(ids) - 8])])
    assert len(seen) == 2 * len(want)
    for k, ref in enumerate(want):
        got = torch.cat([seen[k], seen[len(want) + k]], dim=0)
        assert float((got - ref).abs().max()) < 1e-5 * float(ref.abs().max())


def test_every_learned_number_moves_the_logits():
    """Each tensor matters at the size the tests give it."""
    for key in ("A", "B"):
        cfg, _, seed = nc.ALL[key]
        weights = plain_weights(weights_for(cfg, seed))
        ids = prompts_for({"vocab_size": cfg["vocab"]}, [17], seed)["r0"]
        base = plain_nogosun.forward(cfg, weights, ids)
        spread = float((base - base.mean(-1, keepdim=True)).pow(2).mean().sqrt())
        for name in weights:
            if ".mlp.e" in name:
                continue                # an expert may not be chosen
            other = dict(weights)
            other[name] = weights[name] * 0.5 + 0.1
            moved = float((plain_nogosun.forward(cfg, other, ids) - base).pow(2).mean().sqrt()) / spread
            assert moved > 1e-4, f"{name} moves the logits by {moved:.1e}"


def test_a_slot_that_is_used_again_starts_from_zeros(monkeypatch):
    """With one slot, the second request finds the first one's states and inputs there."""
    reference_ops.install(monkeypatch)
    cfg, page, seed = nc.ALL["A"]
    weights = weights_for(cfg, seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [25, 14], seed)
    runner = make_runner(cfg, weights, page, 8, "float32", "cpu", max_seqs=1)
    got = replay(runner, traces.chunked(prompts, sizes=(9, 2, 13)))
    compare(got, cfg, weights, prompts, 3e-5, plain_logits(cfg, weights, prompts))


def test_greedy_generation_through_the_scheduler(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg, page, seed = nc.ALL["A"]
    weights = weights_for(cfg, seed, std=0.15)
    arch = architecture_for(cfg)
    config = arch.read_config(cfg)
    model = _build(arch.model_spec(config), DictSource(weights), "float32", "cpu")
    engine = LLMEngine(model, config, EngineConfig(dtype="float32", block_size=page, max_blocks=40, max_seqs=3,
                                                   max_tokens_per_step=9, device="cpu", run_ahead=False))
    prompts = list(prompts_for({"vocab_size": cfg["vocab"]}, [4, 13, 27], seed + 1).values())
    got = engine.generate(prompts, SamplingParams(max_new_tokens=5))
    assert got == [greedy(cfg, weights, p, 5) for p in prompts]
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


@pytest.mark.parametrize("seed", range(8))
def test_random_configurations_on_the_host(monkeypatch, seed):
    reference_ops.install(monkeypatch)
    cfg, page = nc.random_configuration(seed)
    weights = weights_for(cfg, 100 + seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [3, 35, 18], seed)
    steps = traces.mixed(prompts, seed=seed)
    runner = make_runner(cfg, weights, page, traces.max_live_tokens(steps, page) // page, "float32", "cpu")
    compare(replay(runner, steps), cfg, weights, prompts, 3e-5, plain_logits(cfg, weights, prompts))
