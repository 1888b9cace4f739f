"""The Vasanex design on the CPU: its configuration and what is refused, its tensors, what its layers need of the
cache, the plain implementation's mechanisms against hand-made cases, and the engine's host logic (step function,
cache, state slots, values that pass from layer to layer, batches) with the plain torch versions of the kernels put
in their place, against the plain whole-sequence implementation."""
import copy
import math

import pytest
import torch

import plain_vasanex
import reference_ops
import traces
import vasanex_configs
from helpers import compare, make_runner, prompts_for, random_weights, replay
from lucciola_amd import models  # noqa: F401  (registers the architectures)
from lucciola_amd.cache.specs import FixedStates, PagedRows
from lucciola_amd.config.engine_config import EngineConfig
from lucciola_amd.config.model_config import ConfigError
from lucciola_amd.config.registry import architecture_for
from lucciola_amd.config.vasanex_config import VasanexConfig
from lucciola_amd.engine.batch import StepEntry
from lucciola_amd.engine.llm_engine import LLMEngine
from lucciola_amd.engine.loading import _build
from lucciola_amd.kernels import ops
from lucciola_amd.models.causal_lm import declared_tensors
from lucciola_amd.models.vasanex import vasanex_model_spec
from lucciola_amd.parts.feed_forward import GatedMLP
from lucciola_amd.parts.masked_attention import MaskedAttention
from lucciola_amd.config.specs import PartSpec
from lucciola_amd.sampling.sampler import SamplingParams
from lucciola_amd.weights.loader import DictSource

LENGTHS = {"A": [1, 12, 45], "B": [2, 40, 21], "C": [30, 9]}


def weights_for(cfg, seed, std=vasanex_configs.STD):
    return vasanex_configs.telling_weights(random_weights(cfg, seed, std=std), seed)


def plain_weights(weights):
    return {k: v.to(torch.float64) for k, v in weights.items()}


def plain_logits(cfg, weights, prompts):
    w = plain_weights(weights)
    return {n: plain_vasanex.forward(cfg, w, ids) for n, ids in prompts.items()}


def greedy(cfg, weights, prompt, count):
    w = plain_weights(weights)
    ids = list(prompt)
    for _ in range(count):
        ids.append(int(torch.argmax(plain_vasanex.forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]


# ------------------------------------------------------------------ configuration, tensors, cache
def test_configuration_is_read_layer_by_layer():
    cfg = VasanexConfig.from_dict(vasanex_configs.V_B)
    assert (cfg.vocab, cfg.width, cfg.norm_eps, cfg.embedding_scale) == (131, 50, 3e-6, 0.7)
    assert [l.type for l in cfg.layers] == ["mlstm", "attention", "attention", "attention", "mlstm"]
    m = cfg.layers[0].mixer
    assert (m.heads, m.dim, m.vdim, m.gate_cap) == (3, 7, 5, 2.5)
    a, b, c = (cfg.layers[i].mixer for i in (1, 2, 3))
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.v_mix) == (3, 3, 10, 7, 0.31, None, True)
    assert (a.rot.dims, a.rot.base) == (6, 77.0) and b.window == 1 and c.rot is None and c.window == 6
    assert cfg.layers[0].mlp is None and (cfg.layers[2].mlp.ff, cfg.layers[2].mlp.limit) == (22, 3.0)
    without = {k: v for k, v in vasanex_configs.V_B.items() if k != "embedding"}
    assert VasanexConfig.from_dict(without).embedding_scale == 1.0
    assert architecture_for(vasanex_configs.V_B).name == "Vasanex"


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="lightning"), "not a mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"].update(gate_cap=0.0), "positive"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=2), "multiple"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=5), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=12), "at most"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(v_mix=1), "true or false"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=9), "mixes values"),
    (lambda c: c["layers"][2]["mixer"]["mask"].update(size=0), "at least 1"),
    (lambda c: c["layers"][2]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][2]["mlp"].update(limit=-1.0), "positive"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "not a feed-forward"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c.update(layers=[]), "at least one"),
])
def test_configuration_refuses(change, message):
    cfg = copy.deepcopy(vasanex_configs.V_B)
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        VasanexConfig.from_dict(cfg)


def test_tensors_blocks_and_whose_values_are_mixed():
    spec = vasanex_model_spec(VasanexConfig.from_dict(vasanex_configs.V_B))
    assert [e.layer for e in spec.run_order] == [0, 1, 2, 3, 4]
    assert [l.block for l in spec.layers] == ["prenorm_mixer", "prenorm_residual", "prenorm_residual", "prenorm_mixer",
                                              "prenorm_residual"]
    assert [l.parts["mixer"].params.get("values") for l in spec.layers] == [None, "keep", "mix", "mix", None]
    names = declared_tensors(spec)
    shapes = {n: d.shape for n, d in names.items()}
    assert shapes["embed"] == (131, 50) and "head" not in shapes and shapes["final.norm"] == (50,)
    assert shapes["l0.mix.q"] == (21, 50) and shapes["l0.mix.v"] == (15, 50) and shapes["l0.mix.g"] == (15, 50)
    assert shapes["l0.mix.i"] == (3, 50) and shapes["l0.mix.f.b"] == (3,) and shapes["l0.mix.norm"] == (15,)
    assert shapes["l0.mix.o"] == (50, 15) and "l0.norm2" not in shapes and "l0.mlp.up" not in shapes
    assert shapes["l1.mix.q.b"] == (30,) and shapes["l1.mix.k.norm"] == (30,) and shapes["l1.mix.o.b"] == (50,)
    assert shapes["l2.mix.q"] == (84, 50) and shapes["l2.mix.k.b"] == (42,) and shapes["l2.mix.q.norm"] == (84,)
    assert shapes["l1.mix.vmix"] == () and shapes["l3.mix.vmix"] == () and shapes["l3.mix.sink"] == (9,)
    assert shapes["l4.mlp.gate"] == (34, 50) and shapes["l4.mlp.down"] == (50, 34) and shapes["l4.norm2"] == (50,)
    first = vasanex_model_spec(VasanexConfig.from_dict(vasanex_configs.V_A))
    assert [l.parts["mixer"].params.get("values") for l in first.layers] == [None, None, "keep", None, "mix"]
    assert "l0.mix.vmix" not in declared_tensors(first)


def test_what_the_layers_keep(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg, page, seed = vasanex_configs.ALL["B"]
    runner = make_runner(cfg, weights_for(cfg, seed), page, 8, "float32", "cpu", max_seqs=3)
    assert runner.model.site_needs() == [
        FixedStates(((3, 6, 7), (3,))), PagedRows(30, 21, None), PagedRows(42, 21, 1), PagedRows(18, 21, 6),
        FixedStates(((1, 10, 11), (1,)))]
    assert len(runner.cache.groups) == 3 and runner.cache.has_fixed_state


def test_parts_refuse_what_no_kernel_has():
    sizes = dict(hidden_size=8, num_heads=2, num_kv_heads=1, head_dim=4, value_dim=4, scale=1.0, eps=1e-6)
    with pytest.raises(ValueError, match="neither 'keep' nor 'mix'"):
        MaskedAttention(**sizes, values="other")
    for more in (dict(conv_taps=2, bias=True), dict(unit_qk=True, row_norm=True), dict(conv_taps=3, values="mix")):
        with pytest.raises(ValueError, match="no prologue kernel has both"):
            MaskedAttention(**sizes, **more)
    half = PartSpec("rotary", {"rotary_dim": 6, "theta": 10.0, "pairing": "half"})
    with pytest.raises(ValueError, match="rotated entries"):
        MaskedAttention(**sizes, position=half)
    with pytest.raises(ValueError, match="go with 'silu'"):
        GatedMLP(8, 8, activation="gelu_tanh", limit=1.0)
    assert GatedMLP(8, 8).form is ops.SILU_GATE


# ------------------------------------------------------------------ the plain implementation by hand
def test_the_whole_row_norm_by_hand():
    """Two heads of two entries normed together: one large head takes the other one's share away."""
    w = {"x.q": torch.eye(4), "x.q.b": torch.tensor([0.0, 0, 0, 1.0]), "x.q.norm": torch.tensor([1.0, 2, 3, 4])}
    w = {k: v.double() for k, v in w.items()}
    h = torch.tensor([[3.0, 1.0, 0.0, 1.0]], dtype=torch.float64)
    got = plain_vasanex.divided_by_rms(plain_vasanex.biased(h, w, "x.q"), 0.0) * w["x.q.norm"]
    root = math.sqrt((9 + 1 + 0 + 4) / 4)
    assert got[0].tolist() == pytest.approx([3 / root, 2 / root, 0.0, 8 / root])


def test_the_rotation_by_hand():
    x = torch.arange(1.0, 7.0, dtype=torch.float64).view(1, 1, 6)
    got = plain_vasanex.rotate_halves(x, torch.tensor([2]), 4, 100.0)[0, 0].tolist()
    a, b = 2.0, 2.0 * 100.0 ** -0.5
    assert got == pytest.approx([1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b),
                                 3 * math.cos(a) + 1 * math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 5.0, 6.0])


def test_the_window_and_the_sink_by_hand():
    mask = plain_vasanex.visible(5, 3)
    for i in range(5):
        assert mask[i].tolist() == [0 <= i - j < 3 for j in range(5)]
    assert plain_vasanex.visible(4, None).tolist() == [[j <= i for j in range(4)] for i in range(4)]
    weights = plain_vasanex.softmax_with_sink(torch.zeros(5, 5, dtype=torch.float64), mask,
                                              torch.tensor(math.log(2.0), dtype=torch.float64))
    assert weights[0, 0].item() == pytest.approx(1 / 3) and weights[4, 2].item() == pytest.approx(1 / 5)
    assert weights[4, 1].item() == 0.0


def test_the_matrix_memory_by_hand():
    """One head of one key and two value entries over three tokens, the reference point written out: the sums
    with gates i_t and f_t do not depend on it, but for the bound of the denominator."""
    cap = 4.0
    raw_i, raw_f = [1.0, -3.0, 0.5], [0.3, -0.7, 2.0]
    h = torch.tensor([[raw_i[t], raw_f[t], t + 1.0] for t in range(3)], dtype=torch.float64)
    e = torch.eye(3, dtype=torch.float64)
    w = {"q": e[2:], "k": e[2:], "v": torch.stack([e[2], -e[2]]), "i": e[:1], "f": e[1:2], "i.b": torch.zeros(1),
         "f.b": torch.ones(1), "g": torch.zeros(2, 3), "norm": torch.tensor([1.0, 3.0]), "o": torch.eye(2)}
    w = {"x." + k: v.double() for k, v in w.items()}
    m = {"heads": 1, "dim": 1, "vdim": 2, "gate_cap": cap}
    out = plain_vasanex.matrix_memory(h, w, "x.", m, 1e-3)
    log_i = [cap * math.tanh(v / cap) for v in raw_i]
    log_f = [-math.log1p(math.exp(-cap * math.tanh((v + 1.0) / cap))) for v in raw_f]
    top = 0.0
    for t in range(3):
        top = max(log_f[t] + top, log_i[t])
        gates = [math.exp(log_i[s] + sum(log_f[s + 1:t + 1])) for s in range(t + 1)]
        S = sum(g * (s + 1) * (s + 1) for s, g in enumerate(gates))
        n = sum(g * (s + 1) for s, g in enumerate(gates))
        o = S * (t + 1) / (max(abs(n * (t + 1)), 1.0) + 1e-6 * math.exp(top))
        rms = math.sqrt(o * o + 1e-3)
        assert out[t].tolist() == pytest.approx([0.5 * o / rms, -1.5 * o / rms], rel=1e-9)


def test_the_clamped_gate_by_hand():
    w = {"x.gate": torch.eye(3), "x.up": torch.eye(3).flip(0), "x.down": torch.eye(3)}
    w = {k: v.double() for k, v in w.items()}
    got = plain_vasanex.clamped_gated_mlp(torch.tensor([[5.0, -0.5, -9.0]], dtype=torch.float64), w, "x.", 2.0)
    want = []
    for g, u in ((2.0, -2.0), (-0.5, -0.5), (-9.0, 2.0)):         # the gate is held below the limit only
        want.append(g / (1 + math.exp(-1.702 * g)) * (u + 1))
    assert got[0].tolist() == pytest.approx(want)


# ------------------------------------------------------------------ the engine's host logic
@pytest.mark.parametrize("key", ["A", "B", "C"])
@pytest.mark.parametrize("family", ["whole", "tail", "chunked", "mixed"])
def test_step_function_matches_plain(monkeypatch, key, family):
    reference_ops.install(monkeypatch)
    cfg, page, seed = vasanex_configs.ALL[key]
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
    cfg, page, seed = vasanex_configs.ALL["A"]
    weights = weights_for(cfg, seed)
    ids = prompts_for({"vocab_size": cfg["vocab"]}, [19], seed)["r0"]
    _, want = plain_vasanex.forward(cfg, plain_weights(weights), ids, keep_layers=True)
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
    """Each tensor but the first mixing layer's number matters at the size the tests give it."""
    cfg, _, seed = vasanex_configs.ALL["B"]
    weights = plain_weights(weights_for(cfg, seed))
    ids = prompts_for({"vocab_size": cfg["vocab"]}, [17], seed)["r0"]
    base = plain_vasanex.forward(cfg, weights, ids)
    spread = float((base - base.mean(-1, keepdim=True)).pow(2).mean().sqrt())
    for name in weights:
        other = dict(weights)
        other[name] = weights[name] * 0.5 + 0.1
        moved = float((plain_vasanex.forward(cfg, other, ids) - base).pow(2).mean().sqrt()) / spread
        if name == "l1.mix.vmix":
            assert moved == 0.0
        else:
            assert moved > 1e-3, f"{name} moves the logits by {moved:.1e}"


def test_nothing_is_passed_on_between_steps(monkeypatch):
    """What a layer leaves for later layers is gone when the step is over."""
    reference_ops.install(monkeypatch)
    cfg, page, seed = vasanex_configs.ALL["A"]
    runner = make_runner(cfg, weights_for(cfg, seed), page, 8, "float32", "cpu")
    batches = []
    inner = runner.model.forward

    def spy(batch, sites):
        batches.append(batch)
        return inner(batch, sites)
    monkeypatch.setattr(runner.model, "forward", spy)
    runner.step([StepEntry("r", [1, 2, 3], [2])])
    assert batches[-1].passing == {}


def test_a_mixing_layer_without_an_earlier_one(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg = copy.deepcopy(vasanex_configs.V_B)
    arch = architecture_for(cfg)
    spec = arch.model_spec(arch.read_config(cfg))
    spec.layers[1].parts["mixer"].params["values"] = "mix"
    model = _build(spec, DictSource(weights_for(cfg, 3)), "float32", "cpu")
    from lucciola_amd.engine.runner import ModelRunner
    runner = ModelRunner(model, EngineConfig(dtype="float32", block_size=8, max_blocks=8, max_seqs=2, device="cpu"))
    with pytest.raises(ValueError, match="no earlier layer"):
        runner.step([StepEntry("r", [1, 2], [1])])
    assert not runner.cache.requests


def test_a_slot_that_is_used_again_starts_from_zeros(monkeypatch):
    """With one slot, the second request finds the first one's memory and reference points there."""
    reference_ops.install(monkeypatch)
    cfg, page, seed = vasanex_configs.ALL["B"]
    weights = weights_for(cfg, seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [25, 14], seed)
    runner = make_runner(cfg, weights, page, 8, "float32", "cpu", max_seqs=1)
    got = replay(runner, traces.chunked(prompts, sizes=(9, 2, 30)))
    compare(got, cfg, weights, prompts, 3e-5, plain_logits(cfg, weights, prompts))


def test_greedy_generation_through_the_scheduler(monkeypatch):
    reference_ops.install(monkeypatch)
    cfg, page, seed = vasanex_configs.ALL["A"]
    weights = weights_for(cfg, seed, std=0.2)
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


@pytest.mark.parametrize("seed", [0, 1, 2, 3, 4, 5, 6, 7])
def test_random_configurations_on_the_host(monkeypatch, seed):
    reference_ops.install(monkeypatch)
    cfg, page = vasanex_configs.random_configuration(seed)
    weights = weights_for(cfg, 100 + seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [3, 35, 18], seed)
    steps = traces.mixed(prompts, seed=seed)
    runner = make_runner(cfg, weights, page, traces.max_live_tokens(steps, page) // page, "float32", "cpu")
    compare(replay(runner, steps), cfg, weights, prompts, 3e-5, plain_logits(cfg, weights, prompts))
