"""The Vasanex design on the GPU: every kernel it brought against the plain torch version of the same operation, and the
engine against the plain whole-sequence implementation (``plain_vasanex``) in the four families of traces, in float32
and in bfloat16."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_vasanex
import reference_ops
import traces
import vasanex_configs as vc
from helpers import make_runner, prompts_for, random_weights, replay
from lucciola_amd.config.engine_config import EngineConfig
from lucciola_amd.config.registry import architecture_for
from lucciola_amd.engine.batch import Plan, StepEntry
from lucciola_amd.engine.llm_engine import LLMEngine
from lucciola_amd.engine.loading import _build
from lucciola_amd.kernels import ops
from lucciola_amd.parts import BuildContext, ResidualStream
from lucciola_amd.parts.norm import RMSNorm
from lucciola_amd.sampling.sampler import SamplingParams
from lucciola_amd.weights.loader import DictSource

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
# A row's error: root mean square of the difference of the logits, means taken off, over that of the plain logits.
TOL = {"float32": 4e-5, "bfloat16": 6e-2}
LENGTHS = {"A": [5, 1, 47, 90, 130], "B": [2, 61, 33, 100], "C": [150, 9, 230, 70]}
_cache = {}


def weights_for(cfg, seed, std=vc.STD):
    return vc.telling_weights(random_weights(cfg, seed, std=std), seed)


def plain_logits(cfg, weights, prompts):
    w = {k: v.to(torch.float64) for k, v in weights.items()}
    return {n: plain_vasanex.forward(cfg, w, ids) for n, ids in prompts.items()}


def case(key):
    if key not in _cache:
        cfg, page, seed = vc.ALL[key]
        weights = weights_for(cfg, seed)
        prompts = prompts_for({"vocab_size": cfg["vocab"]}, LENGTHS[key], seed)
        _cache[key] = (cfg, page, weights, prompts, plain_logits(cfg, weights, prompts))
    return _cache[key]


def row_error(row, ref):
    diff = row - ref
    return float((diff - diff.mean()).pow(2).mean().sqrt() / (ref - ref.mean()).pow(2).mean().sqrt())


def check_rows(got, prompts, refs, dtype, every=True):
    errors = []
    for name, ids in prompts.items():
        for pos in range(len(ids)):
            if (name, pos) not in got:
                assert not every, f"{name} position {pos}: no logits"
                continue
            row, ref = got[(name, pos)], refs[name][pos]
            assert torch.isfinite(row).all(), f"{name} position {pos}: logits are not finite"
            errors.append((row_error(row, ref), name, pos))
    tol = TOL[str(dtype).replace("torch.", "")]
    over = sorted(e for e in errors if e[0] > tol)
    worst = max(errors)
    assert worst[0] <= 3 * tol, f"request {worst[1]} position {worst[2]}: error {worst[0]:.3e} (bound {tol:.1e})"
    assert len(over) <= max(1, len(errors) // 50), (
        f"{len(over)} of {len(errors)} rows over {tol:.1e}; first: request {over[0][1]} position {over[0][2]} "
        f"({over[0][0]:.3e})")
    return worst[0]


def close(got, want, dtype, what, scale=1.0):
    tol = (4e-6 if dtype == torch.float32 else 1.2e-2) * scale
    err = float((got.double() - want.double()).abs().max() / want.double().abs().max().clamp_min(1e-9))
    assert err < tol, f"{what}: relative error {err:.3e}"


def request_lists(lengths, slots):
    q_offsets = torch.tensor([sum(lengths[:i]) for i in range(len(lengths) + 1)], dtype=torch.int32)
    return q_offsets, torch.tensor(slots, dtype=torch.int32)


# ------------------------------------------------------------------ kernels alone
ROWS_CASES = [
    # q heads, k heads, v heads, d, dv, page, tokens, rot, half, bias, norm, values
    (8, 2, 2, 32, 48, 16, 37, 16, True, True, True, "keep"),
    (8, 2, 2, 32, 48, 16, 1, 32, True, True, True, "mix"),
    (9, 3, 3, 10, 7, 4, 5, 6, True, True, True, "mix"),
    (3, 3, 3, 7, 9, 8, 70, 0, True, True, True, None),
    (16, 4, 4, 128, 128, 16, 300, 64, True, True, True, "mix"),
    (32, 8, 8, 128, 64, 32, 3, 128, True, True, True, "keep"),
    (4, 1, 1, 64, 16, 16, 9, 10, False, True, False, None),
    (6, 2, 2, 12, 20, 8, 33, 12, False, False, True, "mix"),
    (2, 1, 1, 256, 256, 16, 2, 2, True, False, False, "keep"),
    (5, 1, 1, 24, 12, 4, 6, 12, False, True, True, "mix"),
    (8, 4, 4, 80, 36, 16, 40, 40, True, True, True, "keep"),
]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case_", ROWS_CASES)
@pytest.mark.parametrize("extra", [5, 8])       # columns behind the heads: with 5, rows begin at odd places
def test_attention_rows(case_, dtype, extra):
    """q, the cache rows (and every row that is not a token's: untouched) and the kept values."""
    nq, nk, nv, d, dv, page, T, rot, half, bias, norm, values = case_
    g = torch.Generator().manual_seed(nq * 100 + d)
    C = (nq + nk) * d + nv * dv
    proj = torch.randn(T, C + extra, generator=g) * 2
    pages = T // page + 4
    places = torch.randperm(pages * page, generator=g)[:T].to(torch.int32)
    places[T // 2] = -1 if T > 2 else places[T // 2]
    positions = torch.randint(0, 3000, (T,), generator=g).to(torch.int32)
    table = None
    if rot:
        angle = torch.arange(3000, dtype=torch.float64)[:, None] * (300.0 ** (-torch.arange(rot // 2, dtype=torch.float64) * 2 / rot))[None, :]
        table = torch.cat([torch.cos(angle), torch.sin(angle)], dim=1).float()
    tensors = dict(bias=torch.randn(C, generator=g) if bias else None,
                   q_weight=1 + 0.3 * torch.randn(nq * d, generator=g) if norm else None,
                   k_weight=1 + 0.3 * torch.randn(nk * d, generator=g) if norm else None, table=table, positions=positions,
                   mix_from=torch.randn(T, nv * dv, generator=g) if values == "mix" else None)
    outs = []
    for o, where in ((reference_ops, "cpu"), (ops, DEV)):
        def on(t):
            return None if t is None else t.clone().to(where)
        kc = torch.full((pages, page, nk * d), 7.0, dtype=dtype, device=where)
        vc_ = torch.full((pages, nv * dv, page), 7.0, dtype=dtype, device=where)
        q, own = o.attention_rows(on(proj), nq, nk, nv, d, dv, dtype, kc, vc_, on(places), eps=1e-5, rot=rot, half=half,
                                  mix=0.37, keep_values=values == "keep", **{k: on(v) for k, v in tensors.items()})
        outs.append([t.cpu() if t is not None else None for t in (q, kc, vc_, own)])
    for got, want, what in zip(outs[1], outs[0], ("q", "key rows", "value rows", "kept values")):
        assert (got is None) == (want is None)
        if want is not None:
            close(got, want, torch.float32 if what == "kept values" else dtype, what)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_rows_bits_do_not_depend_on_the_step(dtype):
    """A token alone (its entries over several workgroups) and the same token among many."""
    g = torch.Generator().manual_seed(1)
    nq, nk, nv, d, dv, page, T = 16, 4, 4, 64, 64, 16, 400
    C = (nq + nk) * d + nv * dv
    proj = torch.randn(T, C, generator=g).to(DEV)
    common = dict(bias=torch.randn(C, generator=g).to(DEV), q_weight=torch.randn(nq * d, generator=g).to(DEV),
                  k_weight=torch.randn(nk * d, generator=g).to(DEV), eps=1e-6)
    caches = [(torch.zeros(30, page, nk * d, dtype=dtype, device=DEV), torch.zeros(30, nv * dv, page, dtype=dtype, device=DEV))
              for _ in range(2)]
    rows = torch.arange(T, dtype=torch.int32, device=DEV)
    q, _ = ops.attention_rows(proj, nq, nk, nv, d, dv, dtype, *caches[0], rows, **common)
    for t in (0, 17, 399):
        alone, _ = ops.attention_rows(proj[t:t + 1].contiguous(), nq, nk, nv, d, dv, dtype, *caches[1], rows[t:t + 1], **common)
        assert torch.equal(alone[0], q[t])
        assert torch.equal(caches[1][0].view(-1, nk * d)[t], caches[0][0].view(-1, nk * d)[t])
        assert torch.equal(caches[1][1][t // page, :, t % page], caches[0][1][t // page, :, t % page])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 48, 100, 129])
def test_one_key_carries_the_weight_at_a_windows_edges(dtype, window):
    """Among hundreds of keys one has a score that stands out and a value of its own, beside a sink: a query sees it
    exactly when fewer than ``window`` tokens lie between them and it is not ahead, in prompts, in portions that
    begin anywhere and in lone tokens, at page borders and at a sequence's start, on both attention kernels."""
    heads, kv, d, dv, page, length = 4, 2, 32, 16, 16, 260
    g = torch.Generator().manual_seed(window)
    table = torch.randperm(length // page + 3, generator=g)[:length // page + 1].to(torch.int32).view(1, -1)
    places = torch.tensor([int(table[0, p // page]) * page + p % page for p in range(length)], device=DEV)
    k_cache = torch.zeros(length // page + 3, page, kv * d, dtype=dtype, device=DEV)
    v_cache = torch.zeros(length // page + 3, kv * dv, page, dtype=dtype, device=DEV)
    q = torch.ones(length, heads * d, dtype=dtype, device=DEV)
    sink = torch.tensor([0.0, 1.0, -1.0, 2.0], device=DEV)
    for marked in (0, 1, 15, 16, 31, 100, 111, 112, 144, 200):
        k = torch.zeros(length, kv * d, dtype=dtype, device=DEV)
        v = torch.full((length, kv * dv), -1.0, dtype=dtype, device=DEV)
        k[marked], v[marked] = 1.0, 5.0
        k_cache.view(-1, kv * d)[places], v_cache[places // page, :, places % page] = k, v
        edge = marked + window
        lone_rows = sorted({p for p in (marked - 1, marked, marked + 1, edge - 1, edge, edge + 1, length - 1) if 0 <= p < length})
        for lone in (False, True):
            rows = lone_rows if lone else list(range(length))
            plans = [None]
            if ops.masked_attention_on_matrix_cores(dtype, d, dv, page, 1):
                for cut in ((1,) if lone else (16, 7, 2)):      # tiles of so many tokens
                    tiles = [[i, min(cut, len(rows) - i), 0, rows[i]] for i in range(0, len(rows), cut)]
                    plans.append(Plan({"tiles": torch.tensor(tiles, dtype=torch.int32, device=DEV)},
                                      {"any_portion": not lone, "any_lone": any(t[1] == 1 for t in tiles)}))
            for plan in plans:
                out = ops.masked_attention(q[:len(rows)].contiguous(), k_cache, v_cache,
                                           torch.zeros(len(rows), dtype=torch.int32, device=DEV),
                                           torch.tensor(rows, dtype=torch.int32, device=DEV), table.to(DEV), page, heads, kv,
                                           1, d, dv, 1.0, window=window, sink=sink, plan=plan).float().cpu()
                for at, p in enumerate(rows):
                    seen = min(p + 1, window)
                    sees = p - window < marked <= p
                    for h in (0, 3):
                        top, others = (float(np.exp(32.0)) if sees else 0.0), seen - int(sees)
                        want = (5.0 * top - others) / (top + others + float(np.exp(float(sink[h]))))
                        got = float(out[at, h * dv])
                        assert abs(got - want) < 2e-2 * max(1.0, abs(want)), (
                            f"key {marked}, query {p}, head {h} ({'lone' if lone else 'prompt'}, "
                            f"{'general' if plan is None else 'matrix cores'}): {got:.3f}, expected {want:.3f}")


MEMORY_CASES = [
    # heads, dk, dv, cap, lengths of two steps
    (4, 32, 40, 11.0, [70, 1, 129, 2]),
    (3, 7, 5, 2.5, [3, 200, 1, 64]),
    (1, 128, 128, 15.0, [65, 600, 1, 193]),
    (2, 16, 16, 6.0, [1, 1, 1, 1]),
    (5, 64, 31, 0.7, [191, 192, 2, 385]),
    (2, 256, 8, 9.0, [1, 1, 40, 1]),
]


@pytest.mark.parametrize("case_", MEMORY_CASES)
def test_matrix_memory_kernels(case_):
    """Three steps in a row over the same slots (the last one of lone tokens): the scan's inputs, the reference points,
    the scan and the read-out against their plain versions, and the slots of other requests untouched."""
    heads, dk, dv, cap, lengths = case_
    g = torch.Generator().manual_seed(dk)
    n = heads * dv
    gate_column = heads * (2 * dk + dv)
    cols = gate_column + n + 2 * heads + 3
    i_bias, f_bias = torch.randn(heads, generator=g) * 2, torch.randn(heads, generator=g) * 2 + 1
    weight = 1 + 0.3 * torch.randn(n, generator=g)
    slots = [4, 0, 5, 2]
    states = {where: (torch.zeros(7, heads, dv + 1, dk, device=where), torch.zeros(7, heads, device=where))
              for where in ("cpu", DEV)}
    for step, new in enumerate((lengths, lengths[::-1], [1, 1, 1, 1])):
        q_offsets, slot_ids = request_lists(new, slots)
        proj = torch.randn(sum(new), cols, generator=g)
        proj[:, gate_column + n:] *= 4
        outs = []
        for o, where in ((reference_ops, "cpu"), (ops, DEV)):
            state, reference = states[where]
            pj, qo, si = proj.to(where), q_offsets.to(where), slot_ids.to(where)
            coef, v, bottoms = o.mlstm_prepare(pj, heads, dk, dv, gate_column + n, gate_column + n + heads, i_bias.to(where),
                                               f_bias.to(where), cap, dk ** -0.5, reference, qo, si, len(new))
            y = o.delta_scan(coef, v, state, qo, si, len(new), heads, dk, dv + 1)
            got = [o.mlstm_readout(y, bottoms, 1e-6, pj, gate_column, weight.to(where), 1e-5, heads, dv, dtype)
                   for dtype in (torch.float32, torch.bfloat16)]
            outs.append([t.cpu() for t in (coef[0], coef[1], coef[2], v, bottoms, reference, y, state, *got)])
        for got, want, what in zip(outs[1], outs[0], ("decay", "write", "read", "values", "bottoms", "reference points",
                                                      "scan", "state", "read-out", "read-out in bfloat16")):
            close(got, want, torch.bfloat16 if "bfloat16" in what else torch.float32, f"step {step}: {what}",
                  10.0 if "read-out" in what else 6.0)
        for slot in (1, 3, 6):
            assert float(states[DEV][0][slot].abs().max()) == 0.0 and float(states[DEV][1][slot].abs().max()) == 0.0


def test_reference_points_have_the_same_bits_for_every_cut():
    """450 tokens whole, in portions and one by one (the kernel of lone tokens): gates, reads and reference points."""
    heads, dk, dv, T = 3, 8, 8, 450
    g = torch.Generator().manual_seed(5)
    cols = heads * (2 * dk + dv) + 2 * heads
    proj = (torch.randn(T, cols, generator=g) * 3).to(DEV)
    i_bias, f_bias = torch.randn(heads, generator=g).to(DEV), torch.randn(heads, generator=g).to(DEV)

    def run(cut):
        reference, parts = torch.zeros(1, heads, device=DEV), []
        for t0 in range(0, T, cut):
            part = proj[t0:t0 + cut].contiguous()
            offsets = torch.tensor([0, part.shape[0]], dtype=torch.int32, device=DEV)
            parts.append(ops.mlstm_prepare(part, heads, dk, dv, cols - 2 * heads, cols - heads, i_bias, f_bias, 6.7, 0.5,
                                           reference, offsets, torch.zeros(1, dtype=torch.int32, device=DEV), 1))
        return [torch.cat([p[0] for p in parts], dim=1), torch.cat([p[1] for p in parts]),
                torch.cat([p[2] for p in parts]), reference]
    whole = run(T)
    for cut in (1, 2, 15, 63, 100, 191, 192, 193, 385):
        for a, b in zip(whole, run(cut)):
            assert torch.equal(a, b), f"portions of {cut}: the bits differ"


@pytest.mark.parametrize("limit,slope,shift", [(1.5, 1.702, 1.0), (0.4, 1.0, 0.0), (7.0, 0.6, -0.25), (float("inf"), 1.0, 0.0)])
@pytest.mark.parametrize("M,I,K", [(1, 64, 128), (5, 256, 512), (16, 192, 1024), (40, 384, 256), (130, 128, 2048),
                                   (300, 512, 128), (600, 1536, 640), (2048, 1024, 256)])
def test_gated_products_in_every_form(M, I, K, limit, slope, shift):
    """The product with the gate in its epilogue (few rows, tiles, tiles cut along K) and the kernel behind a plain
    product, against the formula."""
    g = torch.Generator().manual_seed(M + I)
    form = ops.GateForm(limit, slope, shift)
    x = torch.randn(M, K, generator=g).to(torch.bfloat16)
    gate, up = ((torch.randn(I, K, generator=g) * 1.5 / K ** 0.5).to(torch.bfloat16) for _ in range(2))
    want = reference_ops.gated_activation(torch.cat([x.double() @ gate.double().T, x.double() @ up.double().T], dim=1), "silu", form)
    got = ops.gemm_swiglu(x.to(DEV), ops.interleave_gate_up(gate, up).to(DEV), form)
    close(got.cpu(), want, torch.bfloat16, "in the product's epilogue")
    if limit == float("inf"):
        plain = ops.gemm_swiglu(x.to(DEV), ops.interleave_gate_up(gate, up).to(DEV))
        assert torch.equal(got, plain)
    both = ops.gemm(x.to(DEV), torch.cat([gate, up]).to(DEV), torch.float32)
    close(ops.gated_activation(both, "silu", form).cpu(), want, torch.float32, "behind a plain product", 4.0)


@pytest.mark.parametrize("form", [ops.GateForm(1.1, 1.702, 1.0), ops.SILU_GATE])
@pytest.mark.parametrize("T", [1, 3, 16])
def test_few_rows_norm_and_gate_in_the_products(T, form):
    """The fused steps of a decode step: a branch's product with a bias goes to the stream inside its kernel, the norm's
    factor is applied by the gated product that follows."""
    g = torch.Generator().manual_seed(T)
    n, K, I = 256, 384, 320
    h = torch.randn(T, n, generator=g) * 2
    x = torch.randn(T, K, generator=g).to(torch.bfloat16)
    w = (torch.randn(n, K, generator=g) * 0.05).to(torch.bfloat16)
    bias, weight = torch.randn(n, generator=g), 1 + 0.2 * torch.randn(n, generator=g)
    gate, up = ((torch.randn(I, n, generator=g) * 0.1).to(torch.bfloat16) for _ in range(2))
    v = h.double() + x.double() @ w.double().T + bias.double()
    normed = v / torch.sqrt((v * v).mean(-1, keepdim=True) + 1e-6) * weight.double()
    want = reference_ops.gated_activation(torch.cat([normed @ gate.double().T, normed @ up.double().T], dim=1), "silu",
                                          form)
    stream = h.to(DEV)
    pending = ops.gemm(x.to(DEV), w.to(DEV), torch.bfloat16, defer=True)
    assert isinstance(pending, ops.PendingProduct)
    rows = ops.rmsnorm(stream, ops.BiasedBranch(pending, bias.to(DEV)), weight.to(DEV), 1e-6, torch.bfloat16, scaled=True)
    assert isinstance(rows, ops.ScaledRows)
    close(stream.cpu(), v, torch.float32, "stream", 4.0)
    got = ops.gemm_swiglu(rows, ops.interleave_gate_up(gate, up).to(DEV), form)
    close(got.cpu(), want, torch.bfloat16, "gated", 2.0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,n,K", [(7, 50, 30), (3, 640, 128), (200, 1024, 4096), (70, 4096, 256), (33, 128, 2048)])
def test_a_branchs_bias_joins_the_stream(dtype, T, n, K):
    """A branch with a bias through the norm (as a tensor, as a product cut along K, at picked rows) and as a value."""
    g = torch.Generator().manual_seed(n)
    h, bias = torch.randn(T, n, generator=g), torch.randn(n, generator=g)
    weight = 0.2 * torch.randn(n, generator=g)
    x = torch.randn(T, K, generator=g).to(dtype)
    w = (torch.randn(n, K, generator=g) / K ** 0.5).to(dtype)
    v = h.double() + x.double() @ w.double().T + bias.double()
    want = v / torch.sqrt((v * v).mean(-1, keepdim=True) + 1e-5) * (1 + weight.double())
    norm = RMSNorm(size=n, eps=1e-5, one_plus=True)
    norm.bind({"weight": weight.to(DEV)}, BuildContext(dtype=dtype, device=torch.device(DEV)))
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32)
    for picked in (None, rows):
        for deferred in (False, True):
            stream = ResidualStream(h.clone().to(DEV))
            stream.pending = ops.BiasedBranch(ops.gemm(x.to(DEV), w.to(DEV), dtype, defer=deferred), bias.to(DEV))
            if picked is None:
                close(norm.add_norm(stream).cpu(), want, dtype, f"normed (deferred {deferred})")
                close(stream.h.cpu(), v, dtype, "stream")
                assert stream.pending is None
            else:
                close(norm.add_norm_rows(stream, picked.to(DEV)).cpu(), want[picked.long()], dtype, "picked rows")
                assert torch.equal(stream.h.cpu(), h)
    branch = ops.gemm(x.to(DEV), w.to(DEV), dtype)
    close(ops.value(ops.BiasedBranch(branch, bias.to(DEV))).cpu(), branch.cpu().double() + bias.double(), dtype, "value")


# ------------------------------------------------------------------ the engine
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("key", ["A", "B", "C"])
@pytest.mark.parametrize("family", ["whole", "tail", "chunked", "mixed"])
def test_replay_families(dtype, key, family):
    cfg, page, weights, prompts, refs = case(key)
    steps = {"whole": traces.whole, "tail": traces.tail_decode, "chunked": traces.chunked,
             "mixed": traces.mixed}[family](prompts)
    blocks = traces.max_live_tokens(steps, page) // page
    runner = make_runner(cfg, weights, page, blocks, dtype, DEV)
    check_rows(replay(runner, steps), prompts, refs, dtype)
    assert not runner.cache.requests
    for g in runner.cache.groups:
        assert g.pool.num_free() == blocks


MECHANISMS = {
    "attention alone": [vc.layer(vc.attention(4, 2, 16, 12, 0.3))],
    "attention in a window": [vc.layer(vc.attention(2, 2, 8, 8, 0.3, 13))],
    "a window of one token": [vc.layer(vc.attention(3, 1, 8, 16, 0.3, 1, rot_dims=8))],
    "rotation of some entries": [vc.layer(vc.attention(2, 1, 16, 8, 0.3, rot_dims=6, base=50.0))],
    "rotation of all entries": [vc.layer(vc.attention(2, 1, 16, 16, 0.3, 30, rot_dims=16, base=9000.0))],
    "values of the first layer, then of the third": [
        vc.layer(vc.attention(2, 2, 8, 6, 0.3, 20, v_mix=True)), vc.layer(vc.attention(2, 1, 8, 8, 0.3, 9)),
        vc.layer(vc.attention(4, 2, 12, 6, 0.3, 7, v_mix=True)), vc.layer(vc.attention(6, 2, 4, 6, 0.3, v_mix=True))],
    "one layer that says it mixes": [vc.layer(vc.attention(2, 2, 8, 8, 0.3, 5, v_mix=True))],
    "memory alone": [vc.layer(vc.mlstm(4, 16, 8, 6.0))],
    "memory with a small cap": [vc.layer(vc.mlstm(2, 8, 24, 0.5))],
    "two memories": [vc.layer(vc.mlstm(1, 32, 32, 15.0)), vc.layer(vc.mlstm(3, 5, 7, 3.0))],
    "feed-forward behind a memory": [vc.layer(vc.mlstm(1, 4, 4, 6.0), 40, 0.3)],
    "feed-forward with a wide limit": [vc.layer(vc.attention(1, 1, 4, 4, 0.3, 3), 24, 50.0)],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_each_mechanism(name, dtype):
    cfg = {"architecture": "Vasanex", "vocab": 90, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
           "layers": MECHANISMS[name]}
    weights = weights_for(cfg, 5, std=0.08)
    prompts = prompts_for({"vocab_size": 90}, [37, 4, 60], 2)
    refs = plain_logits(cfg, weights, prompts)
    steps = traces.chunked(prompts, sizes=(7, 2, 16, 1, 1, 3, 30))
    runner = make_runner(cfg, weights, 8, traces.max_live_tokens(steps, 8) // 8, dtype, DEV)
    check_rows(replay(runner, steps), prompts, refs, dtype)


def test_float32_logits_do_not_depend_on_the_cut():
    """The same bits whole, in portions and token by token: every sum's order follows from the token alone."""
    for key in ("A", "B"):
        cfg, page, weights, _, _ = case(key)
        prompts = prompts_for({"vocab_size": cfg["vocab"]}, [75, 40], 3)
        runs = []
        for steps in (traces.whole(prompts), traces.chunked(prompts), traces.tail_decode(prompts, tail=30),
                      traces.mixed(prompts)):
            runs.append(replay(make_runner(cfg, weights, page, 80, "float32", DEV), steps))
        for other in runs[1:]:
            for at, row in runs[0].items():
                same = torch.equal(row, other[at])
                assert same, f"{key} {at}: the bits differ between two cuts"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("key", ["A", "B", "C"])
def test_a_batch_of_unequal_requests_against_each_alone(key, dtype):
    cfg, page, weights, prompts, refs = case(key)
    names = list(prompts)[:4]
    alone = {}
    for n in names:
        alone.update(replay(make_runner(cfg, weights, page, 64, dtype, DEV), traces.whole({n: prompts[n]})))
    runner = make_runner(cfg, weights, page, 160, dtype, DEV)
    cut = {n: max(1, len(prompts[n]) - 3) for n in names}
    rest = {n: prompts[n][cut[n]:] for n in names}
    steps = [([(n, prompts[n][:cut[n]], list(range(cut[n]))) for n in names], [n for n in names if not rest[n]])]
    for k in range(max(len(r) for r in rest.values())):
        steps.append(([(n, [rest[n][k]], [0]) for n in names if k < len(rest[n])],
                      [n for n in names if k == len(rest[n]) - 1]))
    together = replay(runner, steps)
    assert sorted(together) == sorted(alone)
    for at, row in alone.items():
        if dtype == "float32":
            same = torch.equal(row, together[at])
            assert same, f"{at}: the bits differ between alone and in a batch"
        else:
            assert row_error(together[at], row) < 6e-2, at


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(seed, dtype):
    """Configurations drawn at random, requests in mixed steps with so few pages and slots that they are used
    again, against the plain implementation."""
    cfg, page = vc.random_configuration(seed)
    weights = weights_for(cfg, 100 + seed)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [3, 120, 41, 77, 1, 150], seed)
    refs = plain_logits(cfg, weights, prompts)
    steps = traces.mixed(prompts, seed=seed)
    runner = make_runner(cfg, weights, page, traces.max_live_tokens(steps, page) // page, dtype, DEV)
    check_rows(replay(runner, steps), prompts, refs, dtype)
    assert not runner.cache.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("key", ["A", "C"])
def test_long_decoding_past_windows_with_used_pages_and_slots(dtype, key):
    """Two slots and few pages: a request decodes token by token until its windows have passed over what it decoded,
    while others come and go in the pages and slots that earlier ones gave back."""
    cfg, page, weights, _, _ = case(key)
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [150, 30, 26, 41], 9)
    refs = plain_logits(cfg, weights, prompts)
    names = list(prompts)
    long_ids = prompts[names[0]]
    steps = [([(names[1], prompts[names[1]], [29])], [names[1]]), ([(names[0], long_ids[:20], list(range(20)))], [])]
    others = [names[2], names[3]]
    fed = {n: 0 for n in others}
    for i in range(20, 150):
        entries, end = [(names[0], [long_ids[i]], [0])], []
        live = next((n for n in others if fed[n] < len(prompts[n])), None)
        if live is not None and i % 2:
            n = min(5, len(prompts[live]) - fed[live])
            entries.append((live, prompts[live][fed[live]:fed[live] + n], list(range(n))))
            fed[live] += n
            if fed[live] == len(prompts[live]):
                end.append(live)
        if i == 149:
            end.append(names[0])
        steps.append((entries, end))
    runner = make_runner(cfg, weights, page, traces.max_live_tokens(steps, page) // page, dtype, DEV, max_seqs=2)
    check_rows(replay(runner, steps), prompts, refs, dtype, every=False)
    assert not runner.cache.requests


def test_replayed_decode_steps_equal_eager_ones():
    """Steps of single tokens replayed from a HIP graph (values handed from layer to layer inside it, states updated in
    place), with eager portions in between, against a runner that launches every step's kernels."""
    cfg, page, weights, prompts, _ = case("C")
    names = list(prompts)[:3]
    runs = []
    for graphs in (True, False):
        runner = make_runner(cfg, weights, page, 80, "bfloat16", DEV)
        assert runner.use_graphs
        runner.use_graphs = graphs
        out = []
        for n in names:
            out.append(runner.step([StepEntry(n, prompts[n][:9], [8])]).cpu())
        for k in range(9, 40):
            live = [n for n in names if k < len(prompts[n])]
            out.append(runner.step([StepEntry(n, [prompts[n][k]], [0]) for n in live]).cpu())
            if k == 20:
                runner.step([StepEntry("other", prompts[names[0]][:30], [29])])
                runner.finish("other")
        assert (runner.graph_replays > 20) == graphs
        runs.append(out)
    for a, b in zip(*runs):
        assert torch.equal(a, b)


@pytest.mark.parametrize("key", ["A", "B", "C"])
def test_greedy_generation_through_the_engine(key):
    cfg, page, seed = vc.ALL[key]
    weights = weights_for(cfg, seed, std=0.2)
    arch = architecture_for(cfg)
    config = arch.read_config(cfg)
    w64 = {k: v.to(torch.float64) for k, v in weights.items()}
    model = _build(arch.model_spec(config), DictSource(weights), "float32", DEV)
    engine = LLMEngine(model, config, EngineConfig(dtype="float32", block_size=page, max_blocks=60, max_seqs=3,
                                                   max_tokens_per_step=24, device=DEV))
    prompts = list(prompts_for({"vocab_size": cfg["vocab"]}, [4, 33, 57, 9], seed + 1).values())
    got = engine.generate(prompts, SamplingParams(max_new_tokens=8))
    for p, tokens in zip(prompts, got):
        assert len(tokens) == 8
        ids = list(p)
        for t in tokens:        # every generated token is the plain form's argmax, or a near tie with it
            logits = plain_vasanex.forward(cfg, w64, ids)[-1]
            best = int(torch.argmax(logits))
            assert t == best or float(logits[best] - logits[t]) < 1e-4 * float(logits.abs().max()), (ids, t, best)
            ids.append(t)
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(tmp_path, dtype):
    """A model folder made from a configuration and a seed, replayed by ``bin/trace_run``: the architecture is found by
    config.json alone, and the pool is as small as the live requests allow."""
    from lucciola_amd.weights.random_init import write_model_folder
    from lucciola_amd.weights.safetensors_io import SafetensorsFile
    cfg, page, seed = vc.ALL["B"]
    folder = write_model_folder(str(tmp_path / "model"), dict(cfg, initializer_range=vc.STD), seed)
    with SafetensorsFile(os.path.join(folder, "model.safetensors")) as f:
        weights = {n: f.get(n).clone() for n in f.names()}
    prompts = prompts_for({"vocab_size": cfg["vocab"]}, [70, 33, 50, 3, 61], seed)
    steps = traces.mixed(prompts, seed=3)
    lines, index, fed = [], {}, {}
    for i, (entries, end) in enumerate(steps):
        lines.append(json.dumps({"step": i, "end": end, "entries": [{"id": n, "tokens": t, "want": w} for n, t, w in entries]}))
        rows = []
        for n, t, w in entries:
            rows += [(n, fed.get(n, 0) + k) for k in w]
            fed[n] = fed.get(n, 0) + len(t)
        index[i] = rows
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype,
                           "--out", str(out), "--max-tokens", str(traces.max_live_tokens(steps, 64))],
                          input="\n".join(lines) + "\n", text=True, capture_output=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert proc.stdout.split() == [x for i in range(len(steps)) for x in ("done", str(i))]
    got = {}
    for i, rows in index.items():
        data = np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"])
        for r, key in enumerate(rows):
            got[key] = torch.from_numpy(data[r].astype("float64"))
    check_rows(got, prompts, plain_logits(cfg, weights, prompts), dtype)
