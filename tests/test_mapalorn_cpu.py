"""Mapalorn on the CPU: configuration, spec and tensor names, the torch stand-ins of its kernels against the plain
implementation mechanism by mechanism (each mixer in pieces on scattered pages, inputs made so that one far key, by either
part of its score, or the sink decides; both feed-forwards), sums of experts left to the norm that follows, and the engine's
host side (cache manager, step function, runs of layers gone through several times with a cache per pass, pages used again)
against the plain model under every cut."""
import copy
import math

import pytest
import torch

from tests import trace_tools as tt
from tests.mapalorn_cases import (CASES, MAPA_A, MAPA_B, MAPA_C, attention_tensors, build_ff, build_mixer,
                                  deciding_attention_rows, deciding_latent_rows, deciding_rotated_rows, ff_tensors,
                                  latent_tensors, make_folder, run_in_pieces, runtime)
from tests.plain import mapalorn_plain as plain
from tests.torch_ops import TorchOps

RANDOM_SEEDS = [601, 602, 603, 604, 605, 606]
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
    from return_amd.config.mapalorn import MapalornConfig
    cfg = MapalornConfig.from_dict(MAPA_A)
    assert [layer["type"] for layer in cfg.layers] == ["attention", "latent_attention", "attention", "latent_attention", "latent_attention"]
    assert cfg.run_order() == [0, 1, 2, 3, 1, 2, 3, 4] == plain.run_order(MAPA_A)
    assert MapalornConfig.from_dict(MAPA_B).run_order() == [0, 1, 2, 3]
    assert MapalornConfig.from_dict(MAPA_C).run_order() == [0, 0, 0, 0, 1, 2, 3, 4]
    assert MapalornConfig.from_dict(cfg.to_dict()) == cfg
    for change in (lambda c: c["layers"][0].update(type="delta"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
                   lambda c: c["layers"][0]["mixer"].pop("scale"),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5),
                   lambda c: c["layers"][0]["mixer"].update(vdim=0),
                   lambda c: c["layers"][0]["mlp"]["router"].update(top=6),
                   lambda c: c["layers"][0]["mlp"].pop("expert"),
                   lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"),
                   lambda c: c["layers"][0]["mlp"].update(kind="sparse"),
                   lambda c: c["layers"][1]["mixer"].pop("kv_rank"),
                   lambda c: c["layers"][1]["mixer"].pop("rot"),
                   lambda c: c["layers"][1]["mixer"].update(rot_dim=8),
                   lambda c: c["layers"][1]["mlp"].pop("limit"),
                   lambda c: c["layers"][1]["mlp"].update(limit=0.0),
                   lambda c: c["loop"].update(stop=6),
                   lambda c: c["loop"].update(start=4),
                   lambda c: c["loop"].update(times=0),
                   lambda c: c.update(layers=[]),
                   lambda c: c.pop("norm")):
        bad = copy.deepcopy(MAPA_A)
        change(bad)
        with pytest.raises(ConfigError):
            MapalornConfig.from_dict(bad)


def test_spec_names_the_tensors_and_gives_every_run_its_own_cache(model):
    from return_amd.config import load_config, lookup_architecture
    folder, cfg, w = model
    config = load_config(folder)
    spec = lookup_architecture(config.architecture)[1](config)
    assert set(spec.expected_tensors()) == set(w) and len(spec.blocks) == len(cfg["layers"])
    assert [call.block for call in spec.schedule] == plain.run_order(cfg)
    assert [call.cache for call in spec.schedule] == list(range(len(spec.schedule)))
    for i, layer in enumerate(cfg["layers"]):
        assert f"l{i}.norm1.b" in w and f"l{i}.norm2" not in w
        assert any(n.startswith(f"l{i}.mlp.") for n in w) == (layer["mlp"] is not None)


# ------------------------------------------------------------------ the stand-ins, mechanism by mechanism
LATENTS = [dict(heads=3, dim=5, rot_dim=6, vdim=7, kv_rank=10, scale=0.6, rot={"base": 100.0, "dims": 6}),
           dict(heads=1, dim=8, rot_dim=2, vdim=4, kv_rank=24, scale=0.4, rot={"base": 1e6, "dims": 2}),
           dict(heads=4, dim=3, rot_dim=16, vdim=12, kv_rank=6, scale=0.3, rot={"base": 10.0, "dims": 16})]
ATTENTIONS = [dict(heads=4, kv_heads=2, dim=8, vdim=12, scale=0.7, rot={"base": 500.0, "dims": 6}),
              dict(heads=3, kv_heads=3, dim=10, vdim=4, scale=0.5, rot={"base": 1000.0, "dims": 10}),
              dict(heads=4, kv_heads=1, dim=16, scale=0.3)]
PIECES = lambda T: ([T], [1] * T, [2, 1, 9, 2, T - 14])


@pytest.mark.parametrize("m", LATENTS, ids=["small", "one_head_one_pair", "mostly_rotated"])
def test_latent_attention_in_pieces_equals_the_plain_function(m):
    g = torch.Generator().manual_seed(m["heads"])
    W, T, eps = 24, 37, 1e-5
    w = latent_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    want = plain.latent_attention(x.double(), d64(w), m, eps)
    low = dict(w, sink=torch.full_like(w["sink"], -40.0))
    assert (want - plain.latent_attention(x.double(), d64(low), m, eps)).abs().max() > 1e-2      # the sinks do something
    for pieces in PIECES(T):
        got, = run_in_pieces([build_mixer(runtime(TorchOps("cpu")), W, "latent_attention", m, w, eps)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=3e-5, rtol=1e-5)


@pytest.mark.parametrize("m", ATTENTIONS, ids=["grouped_wide_values", "narrow_values_all_rotated", "no_rotation"])
def test_gated_attention_in_pieces_equals_the_plain_function(m):
    g = torch.Generator().manual_seed(m["heads"])
    W, T, eps = 24, 37, 1e-5
    w = attention_tensors(g, W, m)
    x = torch.randn(T, W, generator=g)
    want = plain.gated_attention(x.double(), d64(w), m, eps)
    for pieces in PIECES(T):
        got, = run_in_pieces([build_mixer(runtime(TorchOps("cpu")), W, "attention", m, w, eps)], [x], pieces)
        torch.testing.assert_close(got.double(), want, atol=2e-5, rtol=1e-5)


def test_norms_run_over_the_whole_projection():
    """One head of a query row a hundred times the others: the row's root mean square is nearly that head's alone."""
    x = torch.ones(1, 12, dtype=F64)
    x[0, :4] = 100.0
    y = plain.rms_norm(x, torch.ones(12, dtype=F64), 0.0)
    torch.testing.assert_close(y[0, 0], torch.tensor(100.0 / math.sqrt((4 * 1e4 + 8) / 12), dtype=F64))
    ops = TorchOps("cpu")
    q = torch.empty(1, 2, 4)
    ops.qkv_rows_prepare(torch.cat([x.float(), torch.ones(1, 4)], dim=1), 2, 1, 4, torch.ones(8), torch.ones(4), 8, 4, 0.0,
                         torch.zeros(1, dtype=torch.int32), None, None, 0, q, None, None, None)
    want = plain.rms_norm(x[:, :8], torch.ones(8, dtype=F64), 0.0).float()
    torch.testing.assert_close(q.view(1, 8), want)


@pytest.mark.parametrize("key_at", [0, 3, 15, 16, 31])
@pytest.mark.parametrize("which", ["attention", "latent", "rotated"])
def test_a_far_key_decides(which, key_at):
    """One key's score stands far above all others of one query: the output is that key's value, whole, decoded, and cut
    right behind the key; in the latent attention a sink as far above it takes the value away."""
    g = torch.Generator().manual_seed(7)
    W, T, q_at, eps = 16, 50, 45, 1e-5
    if which == "attention":
        m = dict(heads=4, kv_heads=2, dim=8, vdim=6, scale=1.0)
        w = attention_tensors(g, W, m)
        x, m["scale"] = deciding_attention_rows(T, W, q_at, key_at, w, m, seed=2)
        v = (d64(w)["v"] @ x[key_at].double()).view(2, 6).repeat_interleave(2, 0).reshape(-1)
        alone = (v * torch.sigmoid(d64(w)["g"] @ x[q_at].double())) @ d64(w)["o"].T
        kind, function, sinks = "attention", plain.gated_attention, [None]
    else:
        m = dict(heads=2, dim=8, rot_dim=12, vdim=6, kv_rank=10, scale=1.0, rot={"base": 30.0, "dims": 12})
        w = latent_tensors(g, W, m)
        x, m["scale"] = (deciding_latent_rows if which == "latent" else deciding_rotated_rows)(T, W, q_at, key_at, w, m, seed=2)
        c = plain.rms_norm(d64(w)["dkv"][:10] @ x[key_at].double(), d64(w)["dkv.norm"], eps)
        alone = (d64(w)["uv"] @ c) @ d64(w)["o"].T
        kind, function, sinks = "latent_attention", plain.latent_attention, [-60.0, 150.0]
    for sink in sinks:
        if sink is not None:
            w["sink"] = torch.full((2,), sink)
        want = function(x.double(), d64(w), m, eps)
        assert ((want[q_at] - alone).abs().max() < 2e-3) == (sink is None or sink < 0)
        for pieces in ([T], [q_at] + [1] * (T - q_at), [key_at + 1, 3, T - key_at - 4]):
            got, = run_in_pieces([build_mixer(runtime(TorchOps("cpu")), W, kind, m, w, eps)], [x], pieces)
            torch.testing.assert_close(got.double(), want, atol=1e-4, rtol=1e-5)


def test_the_one_in_the_denominator_is_a_key_of_score_zero():
    """With scores far below zero the output goes to nothing, with scores far above it is that of a plain softmax."""
    s = torch.full((1, 1, 5), -30.0, dtype=F64)
    assert plain.causal_weights(s, torch.zeros(1, dtype=F64)).sum() < 1e-10
    torch.testing.assert_close(plain.causal_weights(s + 60.0, torch.zeros(1, dtype=F64)).sum(), torch.tensor(1.0, dtype=F64))
    torch.testing.assert_close(plain.causal_weights(s + 30.0, torch.zeros(1, dtype=F64))[0, 0], torch.full((5,), 1.0 / 6.0, dtype=F64))


FEED_FORWARDS = [dict(kind="dense", ff=20, limit=0.7),
                 dict(kind="moe", expert=dict(ff=12), router=dict(experts=5, top=1), shared=dict(ff=20)),
                 dict(kind="moe", expert=dict(ff=7), router=dict(experts=4, top=3), shared=dict(ff=5)),
                 dict(kind="moe", expert=dict(ff=9), router=dict(experts=3, top=3))]
FF_IDS = ["dense", "top1", "top3", "all_without_shared"]


def _ff_plain(x, w, mlp):
    return plain.clamped_ff(x, w, mlp["limit"]) if mlp["kind"] == "dense" else plain.experts_ff(x, w, mlp)


@pytest.mark.parametrize("mlp", FEED_FORWARDS, ids=FF_IDS)
def test_feed_forwards_equal_the_plain_functions(mlp):
    from return_amd.parts.runtime import RowSums
    g = torch.Generator().manual_seed(3)
    W = 22
    w = ff_tensors(g, W, mlp)
    x = 1.5 * torch.randn(19, W, generator=g)
    want = _ff_plain(x.double(), d64(w), mlp)
    rt = runtime(TorchOps("cpu"))
    part = build_ff(rt, W, mlp, w)
    torch.testing.assert_close(part.forward(x).double(), want, atol=2e-5, rtol=1e-5)
    if mlp["kind"] == "moe":
        sums = part.forward(x, combine=False)
        assert isinstance(sums, RowSums) and sums.weights is None and tuple(sums.shape) == (19, W)
        torch.testing.assert_close(rt.ops.row_sums(sums).double(), want, atol=2e-5, rtol=1e-5)


def test_a_score_in_front_of_an_expert_is_not_one_behind_it():
    """SiLU and the product of the halves are not linear: the two places of the weight give different results, and the
    scores are not divided by their sum."""
    g = torch.Generator().manual_seed(4)
    mlp = dict(kind="moe", expert=dict(ff=8), router=dict(experts=4, top=2))
    w = d64(ff_tensors(g, 10, mlp))
    x = 1.5 * torch.randn(6, 10, generator=g).double()
    ids, s = plain.route(x, w["router"], 2)
    want = plain.experts_ff(x, w, mlp)
    behind, renormed = torch.zeros_like(x), torch.zeros_like(x)
    for t in range(6):
        for k in range(2):
            e = f"e{int(ids[t, k])}."
            behind[t] += s[t, k] * plain.expert(x[t], w[e + "gate"], w[e + "up"], w[e + "down"])
            renormed[t] += plain.expert(x[t] * s[t, k] / s[t].sum(), w[e + "gate"], w[e + "up"], w[e + "down"])
    assert (want - behind).abs().max() > 1e-2 and (want - renormed).abs().max() > 1e-2
    assert (s[:, 0] >= s[:, 1]).all() and (s.sum(-1) - 1).abs().max() > 1e-2


def test_layer_norm_takes_every_form_of_what_is_pending():
    from return_amd.parts.norm import LayerNorm
    from return_amd.parts.runtime import Pair, RowSums, Scaled, enter_stream
    rt = runtime(TorchOps("cpu"))
    g = torch.Generator().manual_seed(4)
    r = lambda *s: torch.randn(*s, generator=g)
    x, w, b = r(7, 20) + 3.0, 1 + 0.2 * r(20), r(20)
    part = LayerNorm({"size": 20, "eps": 1e-5, "bias": True}, {"weight": w, "bias": b}, rt)
    a, y, extra, logits, factors = r(7, 20), r(21, 20), r(7, 20), r(7, 1), r(7, 3)
    sums = RowSums(y, 3, factors, extra, logits)
    total = (y.view(7, 3, 20) * factors[:, :, None]).sum(1) + extra * torch.sigmoid(logits)
    for pending, added in ((None, 0.0), (a, a), (Scaled(a, -0.5), -0.5 * a), (Pair(a, extra), a + extra), (sums, total),
                           (Pair(a, sums), a + total), (RowSums(a, 1), a)):
        want = plain.layer_norm((x + added).double(), w.double(), b.double(), 1e-5)
        h = x.clone()
        torch.testing.assert_close(part.forward(h, pending).double(), want, atol=1e-5, rtol=1e-5)
        torch.testing.assert_close(h, x + added)
        rows = torch.tensor([5, 0], dtype=torch.int32)
        torch.testing.assert_close(part.forward(x.clone(), pending, rows).double(), want[[5, 0]], atol=1e-5, rtol=1e-5)
        h = x.clone()
        enter_stream(rt.ops, h, pending)
        torch.testing.assert_close(h, x + added)


def test_the_stream_after_every_layer_run_is_the_plain_one(model):
    from return_amd.parts.runtime import enter_stream
    folder, cfg, w = model
    runner = runner_for(folder, 64)
    toks = tt.random_tokens(cfg["vocab"], 21, seed=9)
    want = []
    plain.forward(cfg, w, toks, want)
    seen = []
    for block in runner.model.blocks:
        def wrapped(h, pending, step, cache, write_cache=True, after=None, _f=block.forward):
            h, out = _f(h, pending, step, cache, write_cache, after=after)
            total = h.clone()
            enter_stream(runner.rt.ops, total, out)
            seen.append(total)
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


def test_pages_of_four_used_again(tmp_path_factory):
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
        torch.testing.assert_close(got[key], alone[key], atol=2e-5, rtol=1e-5)
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
