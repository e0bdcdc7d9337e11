"""Mepolix on the CPU: configuration, spec and tensor names, the torch stand-ins of its kernels against the plain
implementation mechanism by mechanism (each mixer in pieces on scattered pages and on a slot, inputs made so that one far
key, the sink or a remembered token decides), and the engine's host side (cache and state manager, step function, layers
that use another layer's tensors with a memory of their own, slots and pages used again) against the plain model under
every cut."""
import copy
import math

import pytest
import torch

from tests import trace_tools as tt
from tests.mepolix_cases import (CASES, MEPO_A, MEPO_B, attention_tensors, build_attention, build_delta, build_parallel,
                                 build_recurrence, deciding_rows, delta_tensors, make_folder, random_case,
                                 recurrence_tensors, run_in_pieces, runtime)
from tests.plain import mepolix_plain as plain
from tests.torch_ops import TorchOps

RANDOM_SEEDS = [401, 402, 403, 404, 405, 406]
F64 = torch.float64


def d64(w):
    return {k: v.double() for k, v in w.items()}


@pytest.fixture(scope="module", params=sorted(CASES) + RANDOM_SEEDS, ids=str)
def model(request, tmp_path_factory):
    folder = make_folder(tmp_path_factory, request.param)
    cfg, w = plain.read_folder(folder)
    return folder, cfg, w


def runner_for(folder, max_tokens, page=16, max_live=4, **kw):
    from return_amd.config import EngineConfig
    from return_amd.engine import ModelRunner
    ec = EngineConfig(dtype="float32", device="cpu", page_size=page, max_token=max_tokens, max_reside=max_live,
                      max_step_tokens=max(max_tokens, 4), prefill_chunk=max_tokens, use_graphs=False,
                      tune_products=False, **kw)
    return ModelRunner(folder, engine_config=ec, ops=TorchOps("cpu"))


# ------------------------------------------------------------------ configuration and spec
def test_config_reads_every_layer_and_refuses_what_it_cannot_run():
    from return_amd.config.base import ConfigError
    from return_amd.config.mepolix import MepolixConfig
    cfg = MepolixConfig.from_dict(MEPO_A)
    assert [layer["type"] for layer in cfg.layers] == ["delta", "parallel", "parallel", "parallel", "delta"]
    assert [cfg.owner(i) for i in range(5)] == [0, 1, 2, 1, 0]
    assert [MepolixConfig.from_dict(MEPO_B).owner(i) for i in range(4)] == [2, 1, 2, 3]
    assert MepolixConfig.from_dict(cfg.to_dict()) == cfg
    for change in (lambda c: c["layers"][0].update(type="attention"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
                   lambda c: c["layers"][0]["mixer"].pop("vdim"),
                   lambda c: c["layers"][0]["mixer"].update(conv=0),
                   lambda c: c["layers"][0]["mlp"].update(kind="moe"),
                   lambda c: c["layers"][0].update(mlp={"kind": "dense", "ff": 0}),
                   lambda c: c["layers"][2]["mixer"].pop("right"),
                   lambda c: c["layers"][2]["mixer"]["right"].update(blocks=3),
                   lambda c: c["layers"][2]["mixer"]["left"].pop("scale"),
                   lambda c: c["layers"][2]["mixer"]["left"].update(kv_heads=2),
                   lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(dims=12),
                   lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(dims=5),
                   lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(scaling={"factor": 2.0}),
                   lambda c: c["layers"][2]["mixer"].update(left_scale="1"),
                   lambda c: c["layers"][3].update(weights_of=9),
                   lambda c: c["layers"][3].update(weights_of=3),
                   lambda c: c["layers"][3].update(weights_of=2),
                   lambda c: (c["layers"][0].update(weights_of=4),),
                   lambda c: c.update(layers=[]),
                   lambda c: c.update(logit_softcap=-1.0),
                   lambda c: c.pop("norm")):
        bad = copy.deepcopy(MEPO_A)
        change(bad)
        with pytest.raises(ConfigError):
            MepolixConfig.from_dict(bad)


def test_spec_names_the_tensors_and_gives_every_layer_its_own_memory(model):
    from return_amd.config import load_config, lookup_architecture
    folder, cfg, w = model
    config = load_config(folder)
    spec = lookup_architecture(config.architecture)[1](config)
    assert set(spec.expected_tensors()) == set(w)
    own = [i for i, layer in enumerate(cfg["layers"]) if layer.get("weights_of") is None]
    assert len(spec.blocks) == len(own)
    kept = []
    for i, (layer, call) in enumerate(zip(cfg["layers"], spec.schedule)):
        assert call.block == own.index(config.owner(i)) and call.writes_cache
        assert any(n.startswith(f"l{i}.") for n in w) == (i in own)
        kept += list(call.cache) if layer["type"] == "parallel" else [call.cache]
        if i in own:
            assert (f"l{i}.norm2" in w) == (layer["mlp"] is not None)
    assert kept == list(range(len(kept)))                # no two layers share a memory, also where they share tensors


# ------------------------------------------------------------------ the stand-ins, mechanism by mechanism
def test_stretched_rotary_tables_are_the_rule_in_64_bit():
    from return_amd.parts.position import RotaryPosition
    rt = runtime(TorchOps("cpu"), positions=300)
    for base, dims, stretch in ((1000.0, 6, (4.0, 32, 8.0, 1.0)), (50.0, 10, None), (1e6, 64, (8.0, 100, 32.0, 1.0)),
                                (20000.0, 32, (2.0, 64, 16.0, 2.0)), (10.0, 2, (3.0, 8, 2.0, 0.5)), (1e4, 16, (1.0, 64, 32.0, 1.0))):
        rot = {"base": base, "dims": dims}
        if stretch:
            rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), stretch))
        part = RotaryPosition({"head_dim": dims + 2, "rotary_dim": dims, "theta": base, "max_position": None,
                               "exact_tables": True, "scaling": rot.get("scaling")}, {}, rt)
        cos, sin, n = part.tables()
        f, factor = plain.stretched_frequencies(rot)
        a = torch.arange(300, dtype=F64)[:, None] * f[None, :]
        assert n == dims and cos.shape == (300, dims // 2)
        torch.testing.assert_close(cos.double(), a.cos() * factor, atol=2e-6, rtol=0)
        torch.testing.assert_close(sin.double(), a.sin() * factor, atol=2e-6, rtol=0)


ATTENTIONS = [
    dict(heads=4, kv_heads=2, dim=8, vdim=12, scale=0.7, rot={"base": 500.0, "dims": 6, "scaling": {"factor": 4.0, "original": 16, "fast": 4.0, "slow": 0.5}}),
    dict(heads=3, kv_heads=3, dim=10, vdim=4, scale=0.5, rot={"base": 1000.0, "dims": 10}),
    dict(heads=2, kv_heads=1, dim=16, vdim=16, scale=1.0),
]
PIECES = lambda T: ([T], [1] * T, [2, 1, 9, 2, T - 14])


@pytest.mark.parametrize("m", ATTENTIONS, ids=["grouped_wide_values", "narrow_values_all_rotated", "no_rotation"])
def test_attention_with_norms_and_sinks_in_pieces_equals_the_plain_function(m):
    g = torch.Generator().manual_seed(m["heads"])
    W, T, eps = 24, 37, 1e-5
    w = attention_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    want = plain.sink_attention(x.double(), d64(w), m, eps)
    low = dict(w, sink=torch.full_like(w["sink"], -40.0))
    assert (want - plain.sink_attention(x.double(), d64(low), m, eps)).abs().max() > 1e-2      # the sinks do something
    for pieces in PIECES(T):
        rt = runtime(TorchOps("cpu"))
        got, = run_in_pieces([build_attention(rt, W, m, w, eps)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)


@pytest.mark.parametrize("key_at", [0, 3, 15, 16, 31])
def test_a_far_key_decides(key_at):
    """One key's score stands far above all others of one query: the output is that key's value, whole, decoded, and cut
    right behind the key; a sink as far above it takes the value away."""
    m = dict(heads=2, kv_heads=1, dim=8, vdim=6, scale=1.0)
    g = torch.Generator().manual_seed(7)
    W, T, q_at, eps = 16, 50, 45, 1e-5
    w = attention_tensors(g, W, m)
    x, m["scale"] = deciding_rows(T, W, q_at, key_at, w, m, seed=2)
    for sink, stays in ((-30.0, True), (40.0, False)):
        w["sink"] = torch.full((2,), sink)
        want = plain.sink_attention(x.double(), d64(w), m, eps)
        alone = (x[key_at].double() @ d64(w)["v"].T).repeat(2) @ d64(w)["o"].T
        assert ((want[q_at] - alone).abs().max() < 1e-4) == stays
        for pieces in ([T], [q_at] + [1] * (T - q_at), [key_at + 1, 3, T - key_at - 4]):
            rt = runtime(TorchOps("cpu"))
            got, = run_in_pieces([build_attention(rt, W, m, w, eps)], [x], pieces)
            torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)


RECURRENCES = [dict(width=24, blocks=3, conv=4), dict(width=35, blocks=5, conv=1), dict(width=16, blocks=1, conv=8)]


@pytest.mark.parametrize("m", RECURRENCES, ids=["blocks", "one_tap", "one_block_long_filter"])
def test_channel_recurrence_in_pieces_equals_the_plain_function(m):
    g = torch.Generator().manual_seed(m["conv"])
    W, T = 20, 37
    w = recurrence_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    want, _, _ = plain.gated_recurrence(x.double(), d64(w), m)
    for pieces in PIECES(T):
        rt = runtime(TorchOps("cpu"))
        got, = run_in_pieces([build_recurrence(rt, W, m, w)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)


def test_channel_recurrence_keeps_what_it_should_and_forgets_what_it_should():
    """lam far below zero: a decay of one, what the first tokens wrote is there 150 tokens later; lam far above: only the
    newest input is left. The zeros before the start are zeros, not biased inputs: the first row's filter sees one input."""
    m = dict(width=6, blocks=2, conv=3)
    g = torch.Generator().manual_seed(3)
    W, T = 12, 150
    w = recurrence_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    other = x.clone()
    other[:3] += 2.0
    for lam, keeps in ((-16.0, True), (6.0, False)):
        w["lam"] = torch.full((6,), lam)
        want, S, _ = plain.gated_recurrence(x.double(), d64(w), m)
        _, S_other, _ = plain.gated_recurrence(other.double(), d64(w), m)
        assert ((S - S_other).abs().max() > 1e-5) == keeps
        rt = runtime(TorchOps("cpu"))
        got, = run_in_pieces([build_recurrence(rt, W, m, w)], [x], [100, 1, 1, 48], pages=tuple(range(12)))
        torch.testing.assert_close(got.double(), want, atol=5e-5, rtol=1e-4)
    u, _ = plain.causal_filter(x[:1].double() @ w["x"].double().T + w["x.b"].double(), w["conv"].double(), w["conv.b"].double())
    first = (x[:1].double() @ w["x"].double().T + w["x.b"].double()) * w["conv"].double()[:, -1] + w["conv.b"].double()
    torch.testing.assert_close(u, first)


DELTAS = [dict(heads=4, kv_heads=2, dim=6, vdim=10, conv=3), dict(heads=3, kv_heads=1, dim=12, vdim=5, conv=1),
          dict(heads=2, kv_heads=2, dim=8, vdim=8, conv=5)]


@pytest.mark.parametrize("m", DELTAS, ids=["grouped", "one_tap", "long_filter"])
def test_delta_mixer_in_pieces_equals_the_plain_function(m):
    g = torch.Generator().manual_seed(m["heads"])
    W, T, eps = 24, 37, 1e-5
    w = delta_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    want, _, _ = plain.delta(x.double(), d64(w), m, eps)
    for pieces in PIECES(T):
        rt = runtime(TorchOps("cpu"))
        got, = run_in_pieces([build_delta(rt, W, m, w, eps)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)


def test_delta_rule_writes_before_it_reads_and_overwrites_the_same_key():
    """With beta one and no decay a key's second value replaces its first; the read-out sees the token's own write."""
    k = torch.zeros(3, 1, 4, dtype=F64)
    k[:, 0, 0] = 1.0
    v = torch.tensor([[[1.0, 2.0]], [[5.0, -1.0]], [[7.0, 0.5]]], dtype=F64)
    ones = torch.ones(3, 1, dtype=F64)
    o, S = plain.delta_rule(k, k, v, ones, ones)
    torch.testing.assert_close(o[:, 0], v[:, 0])
    torch.testing.assert_close(S[0, 0], v[2, 0])


@pytest.mark.parametrize("right", [dict(width=24, blocks=3, conv=4), dict(width=27, blocks=3, conv=2)], ids=["aligned", "filled_up"])
def test_mixers_side_by_side_in_pieces_equal_the_plain_function(right):
    g = torch.Generator().manual_seed(5)
    W, T, eps = 20, 37, 1e-5
    m = {"left": dict(heads=3, kv_heads=1, dim=6, vdim=5, scale=0.6, rot={"base": 100.0, "dims": 4}), "right": right,
         "left_scale": 0.3, "right_scale": -1.7}
    wl, wr = attention_tensors(g, W, m["left"]), recurrence_tensors(g, W, m["right"])
    x = torch.randn(T, W, generator=g)
    w = {**{"left." + k: v for k, v in wl.items()}, **{"right." + k: v for k, v in wr.items()}}
    want = plain.parallel(x.double(), w, m, eps)
    for pieces in PIECES(T):
        rt = runtime(TorchOps("cpu"))
        got, = run_in_pieces([build_parallel(rt, W, m, wl, wr, eps)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)
        assert len(rt.products) == 2                     # one product in front and one behind for both sides


def test_layer_norm_has_a_mean_and_the_soft_cap_is_one():
    from return_amd.parts.embedding import LinearHead
    from return_amd.parts.norm import LayerNorm
    rt = runtime(TorchOps("cpu"))
    g = torch.Generator().manual_seed(4)
    x, w = torch.randn(7, 20, generator=g) + 3.0, 1 + 0.2 * torch.randn(20, generator=g)
    part = LayerNorm({"size": 20, "eps": 1e-5}, {"weight": w}, rt)
    torch.testing.assert_close(part.forward(x.clone()).double(), plain.layer_norm(x.double(), w.double(), 1e-5), atol=1e-5, rtol=1e-5)
    rows = torch.tensor([5, 0], dtype=torch.int32)
    torch.testing.assert_close(part.forward(x.clone(), None, rows).double(), plain.layer_norm(x.double(), w.double(), 1e-5)[[5, 0]],
                               atol=1e-5, rtol=1e-5)
    head = LinearHead({"vocab_size": 9, "hidden_size": 20, "softcap": 4.0}, {"weight": 3.0 * torch.randn(9, 20, generator=g)}, rt)
    z = x.double() @ head.weight.double().T
    torch.testing.assert_close(head.forward(x).double(), 4.0 * torch.tanh(z / 4.0), atol=1e-5, rtol=1e-5)
    assert z.abs().max() > 4.0


def test_the_stream_after_every_layer_is_the_plain_one(model):
    folder, cfg, w = model
    runner = runner_for(folder, 64)
    toks = tt.random_tokens(cfg["vocab"], 21, seed=9)
    want = []
    plain.forward(cfg, w, toks, want)
    seen = []
    for block in runner.model.blocks:
        def wrapped(h, pending, step, cache, write_cache=True, _f=block.forward):
            h, out = _f(h, pending, step, cache, write_cache)
            seen.append(h.clone())
            return h, out
        block.forward = wrapped
    tt.run_in_process(runner, tt.whole({"r": toks}))
    assert len(seen) == len(want)
    for got, ref in zip(seen, want):
        torch.testing.assert_close(got.double(), ref, atol=3e-4, rtol=1e-4)


# ------------------------------------------------------------------ the engine's host side under every cut
def _requests(cfg, seed):
    return {f"r{i}": tt.random_tokens(cfg["vocab"], n, seed=seed + i) for i, n in enumerate([50, 1, 23, 2, 34])}


def _check(got, cfg, w, requests, atol=3e-4):
    for rid, toks in requests.items():
        want = plain.logits(cfg, w, toks)
        rows = torch.stack([got[(rid, p)] for p in range(len(toks))]).double()
        torch.testing.assert_close(rows, want, atol=atol, rtol=1e-4)


def test_engine_equals_plain_under_every_cut(model):
    folder, cfg, w = model
    requests = _requests(cfg, 11)
    for name, steps in (("whole", tt.whole(requests)), ("tail", tt.tail_decoded(requests, tail=20)),
                        ("portions", tt.portions(requests)), ("mixed", tt.mixed(requests, seed=3))):
        runner = runner_for(folder, tt.peak_tokens(steps, 16) + 16, page=16)
        _check(tt.run_in_process(runner, steps), cfg, w, requests)


def test_pages_of_four_and_slots_used_again(tmp_path_factory):
    folder = make_folder(tmp_path_factory, "a")
    cfg, w = plain.read_folder(folder)
    requests = {f"r{i}": tt.random_tokens(cfg["vocab"], n, seed=40 + i) for i, n in enumerate([30, 9, 45, 3, 26, 12])}
    steps = tt.mixed(requests, seed=5, max_live=3, decode_tail=5, sizes=(6, 2, 13, 3))
    runner = runner_for(folder, tt.peak_tokens(steps, 4) + 8, page=4, max_live=3)
    _check(tt.run_in_process(runner, steps), cfg, w, requests)


def test_a_batch_of_unequal_requests_equals_each_alone(tmp_path_factory):
    folder = make_folder(tmp_path_factory, "b")
    cfg, w = plain.read_folder(folder)
    requests = {f"r{i}": tt.random_tokens(cfg["vocab"], n, seed=60 + i) for i, n in enumerate([37, 2, 18, 5])}
    together = [{"step": 0, "entries": [{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in requests.items()],
                 "end": list(requests)}]
    got = tt.run_in_process(runner_for(folder, 128), together)
    alone = tt.run_in_process(runner_for(folder, 128), tt.whole(requests))
    for key in alone:
        torch.testing.assert_close(got[key], alone[key], atol=1e-5, rtol=1e-5)
    _check(got, cfg, w, requests)


def test_greedy_generation_through_the_engine_equals_plain(tmp_path_factory):
    from return_amd.config import EngineConfig
    from return_amd.engine import Engine, ModelRunner
    from return_amd.sampling import SamplingParams
    folder = make_folder(tmp_path_factory, "a")
    cfg, w = plain.read_folder(folder)
    ec = EngineConfig(dtype="float32", device="cpu", page_size=16, max_token=256, max_reside=4, max_step_tokens=32,
                      prefill_chunk=16, use_graphs=False, tune_products=False, check_invariants=True)
    eng = Engine(runner=ModelRunner(folder, engine_config=ec, ops=TorchOps("cpu")))
    prompts = [tt.random_tokens(cfg["vocab"], n, seed=80 + n) for n in (5, 29, 1, 14, 40)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=7))
    for prompt, out in zip(prompts, outs):
        assert list(out.output_ids) == plain.greedy(cfg, w, prompt, 7)
