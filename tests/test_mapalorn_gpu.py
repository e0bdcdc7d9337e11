"""Mapalorn on the GPU: every new kernel alone against its torch stand-in; both attentions with inputs made so that one far
key, by either part of its score, or the sink decides (a page's first and last row, the first places, far back; as a
prompt's portion and decoded), on the plain and the matrix-core kernels; mixers and feed-forwards of the package in pieces
against the plain functions; the engine against the plain model whole, with a decoded tail, in portions down to two tokens
and in mixed batches with pages used again, in both precisions and on configurations drawn from seeds; long decoding; greedy
generation through Engine.generate with and without graphs; the command line; the trace program."""
import os

import pytest
import torch

from tests import trace_tools as tt
from tests.mapalorn_cases import (CASES, attention_tensors, build_ff, build_mixer, deciding_attention_rows,
                                  deciding_latent_rows, deciding_rotated_rows, ff_tensors, latent_tensors, make_folder,
                                  run_in_pieces, runtime)
from tests.plain import mapalorn_plain as plain
from tests.test_fefulorn_gpu import i32, rnd, row_error, tol
from tests.torch_ops import TorchOps

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]
RANDOM_SEEDS = [701, 702, 703, 704, 705, 706, 707, 708, 709, 710]


@pytest.fixture(scope="module")
def ops():
    from return_amd.kernels.hip_ops import HipOps
    return HipOps(DEV)


@pytest.fixture(scope="module")
def ref():
    return TorchOps(DEV)


def d64(w):
    return {k: v.double() for k, v in w.items()}


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H", [(1, 64), (7, 76), (33, 210), (300, 4096), (2, 5000), (3, 9000), (5, 9), (2, 20000)])
def test_layer_norm_adds_what_is_pending(ops, ref, dtype, T, H):
    from return_amd.parts.runtime import RowSums
    w, bias = 1 + rnd(H, seed=4, scale=0.2), rnd(H, seed=5)
    a, y, extra = rnd(T, H, dtype=dtype, seed=2), rnd(3 * T, H, dtype=dtype, seed=3), rnd(T, H, dtype=dtype, seed=6)
    wide, factors = rnd(T, 11, seed=7), rnd(T, 3, seed=8)
    rows = i32([T - 1, 0, T // 2])
    for kw in (dict(), dict(first=a), dict(second=extra), dict(first=a, second=extra), dict(second=RowSums(y, 3, factors)),
               dict(first=a, second=RowSums(y, 3)), dict(first=a, second=RowSums(y, 3, None, extra, wide[:, 4:5])),
               dict(second=RowSums(a, 1, None, extra, wide[:, :1]))):
        for some in (False, True):
            for b in (bias, None):
                ha = rnd(T, H, seed=1, scale=2.0) + 5.0            # (a mean far from zero)
                hb = ha.clone()
                xa, xb = (torch.zeros(3 if some else T, H, dtype=dtype, device=DEV) for _ in range(2))
                ops.layer_norm(ha, w, 1e-5, xa, rows if some else None, bias=b, **kw)
                ref.layer_norm(hb, w, 1e-5, xb, rows if some else None, bias=b, **kw)
                torch.testing.assert_close(ha, hb, atol=1e-5, rtol=1e-5)
                torch.testing.assert_close(xa.float(), xb.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("Hq,Hkv,D,d,R,P,T", [(4, 2, 16, 12, 8, 16, 37), (3, 3, 10, 10, 10, 4, 5), (8, 1, 64, 32, 32, 16, 70),
                                              (2, 2, 12, 5, 0, 8, 1), (5, 5, 128, 128, 64, 16, 19), (6, 2, 80, 66, 2, 32, 33),
                                              (4, 2, 64, 64, 64, 16, 300), (1, 1, 4, 3, 2, 8, 9), (32, 8, 128, 128, 128, 16, 3),
                                              (6, 2, 256, 200, 192, 4, 9), (17, 1, 31, 31, 30, 16, 5)])
def test_preparation_with_norms_over_whole_projections(ops, ref, dtype, Hq, Hkv, D, d, R, P, T):
    """Rows are columns of wider rows; what a head has beyond its true width is zero and does not count."""
    n = (Hq + 2 * Hkv) * D
    wide = rnd(T, n + 40, dtype=dtype, seed=1)
    heads = wide[:, 8:8 + n].unflatten(1, (Hq + 2 * Hkv, D))
    heads[:, :Hq + Hkv, d:] = 0
    heads[:, 0] *= 4.0                                       # (one head's rows longer than the others': the norm is not per head)
    wq, wk = 1 + rnd(Hq * D, seed=2, scale=0.3), 1 + rnd(Hkv * D, seed=9, scale=0.3)
    positions = i32([(7 * t) % 90 for t in range(T)])
    cos, sin = rnd(90, max(R // 2, 1), seed=3), rnd(90, max(R // 2, 1), seed=4)
    pages = -(-T // P) + 2
    slots = torch.randperm(pages * P, generator=torch.Generator().manual_seed(6))[:T].tolist()
    for write in (True, False):
        outs = []
        for k in (ops, ref):
            q = torch.zeros(T, Hq, D, dtype=dtype, device=DEV)
            kp, vp = (torch.zeros(pages, Hkv, P, D, dtype=dtype, device=DEV) for _ in range(2))
            k.qkv_rows_prepare(wide[:, 8:8 + n], Hq, Hkv, D, wq, wk, Hq * d, Hkv * d, 1e-5, positions, cos if R else None,
                               sin if R else None, R, q, kp if write else None, vp if write else None, i32(slots))
            outs.append((q, kp, vp))
        for x, y in zip(*outs):
            torch.testing.assert_close(x.float(), y.float(), **tol(dtype))
        assert bool((outs[0][1] != 0).any()) == write


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,N", [(1, 64), (9, 77), (300, 512), (4, 4098)])
def test_gates_on_rows_and_halves_that_meet(ops, ref, dtype, T, N):
    wide, gates = rnd(T, N + 24, dtype=dtype, seed=1), rnd(T, N + 40, dtype=dtype, seed=2, scale=3.0)
    a, b = wide.clone(), wide.clone()
    ops.gate_rows(a[:, 8:8 + N], gates[:, 16:16 + N])
    ref.gate_rows(b[:, 8:8 + N], gates[:, 16:16 + N])
    torch.testing.assert_close(a.float(), b.float(), **tol(dtype))
    assert torch.equal(a[:, :8], wide[:, :8]) and torch.equal(a[:, 8 + N:], wide[:, 8 + N:])
    for source in {dtype, torch.float32}:
        gu = rnd(T, 2 * N + 20, dtype=source, seed=3, scale=2.0)[:, 4:]
        for act, limit in (("silu", 0.0), ("clamped", 0.7)):
            o, p = (torch.empty(T, N, dtype=dtype, device=DEV) for _ in range(2))
            ops.gated_rows(gu, o, act, limit)
            ref.gated_rows(gu, p, act, limit)
            torch.testing.assert_close(o.float(), p.float(), **tol(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("Hn,D,R,rot,C,P,T", [(3, 5, 6, 6, 10, 4, 9), (8, 32, 16, 16, 64, 16, 33), (1, 8, 2, 2, 300, 8, 1),
                                              (16, 64, 64, 64, 512, 16, 70), (2, 3, 8, 4, 7, 16, 12)])
def test_latent_preparation_without_a_query_latent(ops, ref, dtype, Hn, D, R, rot, C, P, T):
    at = Hn * (D + R)
    wide = rnd(T, at + C + R + 13, dtype=dtype, seed=1)
    w = 1 + rnd(C, seed=2, scale=0.3)
    positions = i32([(11 * t) % 70 for t in range(T)])
    cos, sin = rnd(70, rot // 2, seed=3), rnd(70, rot // 2, seed=4)
    pages = -(-T // P) + 2
    slots = i32(torch.randperm(pages * P, generator=torch.Generator().manual_seed(6))[:T].tolist())
    outs = []
    for k in (ops, ref):
        kp, vp = torch.zeros(pages, 1, P, R, dtype=dtype, device=DEV), torch.zeros(pages, 1, P, C, dtype=dtype, device=DEV)
        qq = torch.full((T, Hn, C + R), 3.0, dtype=dtype, device=DEV)
        k.latent_kv_prepare(wide[:, at:at + C + R], 0, C, R, None, w, 1e-5, positions, cos, sin, rot, None, kp, vp, slots,
                            q=wide[:, :at], qq_out=qq)
        outs.append((kp, vp, qq))
    for x, y in zip(*outs):
        torch.testing.assert_close(x.float(), y.float(), **tol(dtype))
    assert bool((outs[0][2][:, :, :C] == 3.0).all())         # the product's place stays as it was


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B,M,K,N,wide", [(3, 5, 6, 7, 2), (8, 1, 64, 128, 32), (16, 33, 32, 64, 16), (2, 64, 128, 256, 0), (4, 40, 24, 48, 8)])
def test_batched_products_into_columns(ops, dtype, B, M, K, N, wide):
    """Left operand a transposed view of rows, result into the heads' places side by side: the bits of the result as it
    comes alone, and nothing beside the places."""
    a = rnd(M, B * (K + 8), dtype=dtype, seed=1).unflatten(1, (B, K + 8))[:, :, :K].transpose(0, 1)
    b = rnd(B, K, N, dtype=dtype, seed=2, scale=K ** -0.5)
    out = torch.full((M, B, N + wide), 5.0, dtype=dtype, device=DEV)
    ops.batched_product(a, b, out=out.transpose(0, 1)[:, :, :N])
    want = torch.stack([a[i].double() @ b[i].double() for i in range(B)])
    torch.testing.assert_close(out[:, :, :N].transpose(0, 1).double(), want, atol=2e-5 if dtype == torch.float32 else 2e-2,
                               rtol=2e-5 if dtype == torch.float32 else 2e-2)
    assert bool((out[:, :, N:] == 5.0).all())


@pytest.mark.parametrize("T,E,top,groups,keep", [(1, 4, 1, 1, 1), (9, 8, 8, 1, 1), (70, 33, 5, 1, 1), (6, 12, 3, 4, 2), (5, 300, 20, 1, 1)])
def test_router_with_raw_sigmoid_scores(ops, ref, T, E, top, groups, keep):
    z = rnd(T, E + 9, seed=1, scale=2.0)[:, 5:5 + E]         # (columns of wider rows)
    for bias in (None, rnd(E, seed=2, scale=0.1)):
        ia, wa = ops.moe_route(z, bias, top, groups, keep, 0.0, law="sigmoid_raw")
        ib, wb = ref.moe_route(z, bias, top, groups, keep, 0.0, law="sigmoid_raw")
        assert torch.equal(ia, ib)
        torch.testing.assert_close(wa, wb, atol=1e-6, rtol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,I,E,top", [(1, 24, 16, 4, 1), (9, 40, 24, 3, 3), (37, 22, 10, 5, 2), (400, 64, 48, 4, 2), (130, 72, 64, 2, 1)])
def test_experts_that_read_the_token_times_its_weight(ops, ref, dtype, T, H, I, E, top):
    """All three forms of the experts' product (pairs an expert few, some and many), sums formed and left."""
    x = rnd(T, H, dtype=dtype, seed=1, scale=1.5)
    ids, w = ref.moe_route(rnd(T, E, seed=2, scale=2.0), None, top, 1, 1, 0.0, law="sigmoid_raw")
    gu, down = rnd(E, 2 * I, H, dtype=dtype, seed=3, scale=1.5 * H ** -0.5), rnd(E, H, I, dtype=dtype, seed=4, scale=I ** -0.5)
    extra, logits = rnd(T, H, dtype=dtype, seed=5), rnd(T, 6, seed=6)
    for kw in (dict(), dict(extra=extra, extra_logits=logits[:, 2:3])):
        want = ref.moe_experts(x, ids, w, gu, down, weigh="input", **kw)
        got = ops.moe_experts(x, ids, w, gu, down, weigh="input", **kw)
        torch.testing.assert_close(got.float(), want.float(), **tol(dtype))
        sums = ops.moe_experts(x, ids, w, gu, down, weigh="input", combine=False, **kw)
        assert sums.weights is None and sums.count == top
        assert torch.equal(ops.row_sums(sums), got)
    other = ops.moe_experts(x, ids, w, gu, down)
    assert (other.float() - ref.moe_experts(x, ids, w, gu, down, weigh="input").float()).abs().max() > 1e-2


# ------------------------------------------------------------------ one far key decides
LATENT_SIZES = [dict(heads=3, dim=10, rot_dim=12, vdim=6, kv_rank=14), dict(heads=4, dim=32, rot_dim=32, vdim=48, kv_rank=64),
                dict(heads=20, dim=16, rot_dim=64, vdim=16, kv_rank=96)]
ATTN_SIZES = [dict(heads=3, kv_heads=1, dim=10, vdim=6), dict(heads=4, kv_heads=2, dim=64, vdim=48),
              dict(heads=2, kv_heads=2, dim=32, vdim=80)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size", [0, 1, 2])
@pytest.mark.parametrize("which", ["attention", "latent", "rotated"])
@pytest.mark.parametrize("key_at", [0, 3, 15, 16, 333])
def test_a_far_key_decides(ops, dtype, which, size, key_at):
    W, query_at, eps = 32, 610, 1e-5
    T = query_at + 3
    store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    g = torch.Generator().manual_seed(9)
    if which == "attention":
        m = dict(ATTN_SIZES[size], scale=1.0)
        w = attention_tensors(g, W, m, store)
        x, m["scale"] = deciding_attention_rows(T, W, query_at, key_at, w, m, seed=4)
        kind, function, sinks = "attention", plain.gated_attention, [None]
    else:
        m = dict(LATENT_SIZES[size], scale=1.0)
        m["rot"] = {"base": 30.0, "dims": m["rot_dim"]}
        w = latent_tensors(g, W, m, store)
        x, m["scale"] = (deciding_latent_rows if which == "latent" else deciding_rotated_rows)(T, W, query_at, key_at, w, m, seed=4)
        kind, function, sinks = "latent_attention", plain.latent_attention, [-60.0, 150.0]
    if dtype == "bfloat16":
        x = x.bfloat16().float()
    H, V = m["heads"], m["vdim"]
    for sink in sinks:
        if sink is not None:
            w["sink"] = torch.full((H,), sink)
        want = function(x.double(), d64(w), m, eps)
        if which == "attention":
            v = (d64(w)["v"] @ x[key_at].double()).view(m["kv_heads"], V).repeat_interleave(H // m["kv_heads"], 0).reshape(-1)
            alone = (v * torch.sigmoid(d64(w)["g"] @ x[query_at].double())) @ d64(w)["o"].T
        else:
            c = plain.rms_norm(d64(w)["dkv"][:m["kv_rank"]] @ x[key_at].double(), d64(w)["dkv.norm"], eps)
            alone = (d64(w)["uv"] @ c) @ d64(w)["o"].T
        assert ((want[query_at] - alone).abs().max() < 2e-2 * alone.abs().max()) == (sink is None or sink < 0)
        for pieces in ([T], [query_at] + [1] * 3, [key_at + 1, T - key_at - 1]):
            rt = runtime(ops, dtype, DEV, positions=1024)
            got, = run_in_pieces([build_mixer(rt, W, kind, m, w, eps)], [x], pieces, pages=tuple(reversed(range(-(-T // 16)))))
            err = (got.double() - want)[query_at].abs().max() / alone.abs().max()
            assert err < (2e-4 if dtype == "float32" else 5e-2), f"{pieces}: {err}"


# ------------------------------------------------------------------ parts of the package in pieces
PIECES = ([150], [100] + [1] * 50, [5, 2, 1, 17, 64, 61])


@pytest.mark.parametrize("kind,m", [
    ("latent_attention", dict(heads=3, dim=5, rot_dim=6, vdim=7, kv_rank=10, scale=0.5, rot={"base": 100.0, "dims": 6})),
    ("latent_attention", dict(heads=4, dim=48, rot_dim=16, vdim=24, kv_rank=64, scale=0.15, rot={"base": 5000.0, "dims": 16})),
    ("latent_attention", dict(heads=40, dim=16, rot_dim=64, vdim=32, kv_rank=160, scale=0.12, rot={"base": 1e5, "dims": 64})),
    ("attention", dict(heads=4, kv_heads=2, dim=8, vdim=12, scale=0.7, rot={"base": 500.0, "dims": 6})),
    ("attention", dict(heads=8, kv_heads=2, dim=64, vdim=48, scale=0.2, rot={"base": 5000.0, "dims": 16})),
    ("attention", dict(heads=4, kv_heads=4, dim=96, vdim=96, scale=0.1))],
    ids=["latent_odd", "latent_16", "latent_64", "attention_odd", "attention_cores", "attention_no_rotation"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixers_in_pieces(ops, dtype, kind, m):
    g = torch.Generator().manual_seed(3)
    W, eps = 40, 1e-5
    store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    w = (latent_tensors if kind == "latent_attention" else attention_tensors)(g, W, m, store)
    x = torch.randn(150, W, generator=g).to(store).float()
    want = (plain.latent_attention if kind == "latent_attention" else plain.gated_attention)(x.double(), d64(w), m, eps)
    for pieces in PIECES:
        got, = run_in_pieces([build_mixer(runtime(ops, dtype, DEV), W, kind, m, w, eps)], [x], pieces, pages=tuple(reversed(range(10))))
        if dtype == "float32":
            torch.testing.assert_close(got.double(), want, atol=2e-4, rtol=1e-4)
        else:
            assert (got.double() - want).pow(2).mean().sqrt() < 0.03 * want.pow(2).mean().sqrt()


@pytest.mark.parametrize("mlp", [dict(kind="dense", ff=40, limit=0.7),
                                 dict(kind="moe", expert=dict(ff=24), router=dict(experts=5, top=1), shared=dict(ff=40)),
                                 dict(kind="moe", expert=dict(ff=11), router=dict(experts=4, top=3), shared=dict(ff=5)),
                                 dict(kind="moe", expert=dict(ff=16), router=dict(experts=3, top=3))],
                         ids=["dense", "top1", "top3_odd", "all_without_shared"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [1, 19, 260])
def test_feed_forwards(ops, dtype, mlp, T):
    g = torch.Generator().manual_seed(3)
    W = 48
    store = torch.bfloat16 if dtype == "bfloat16" else torch.float32
    w = ff_tensors(g, W, mlp, store)
    x = (1.5 * torch.randn(T, W, generator=g)).to(store)
    want = plain.clamped_ff(x.double(), d64(w), mlp["limit"]) if mlp["kind"] == "dense" else plain.experts_ff(x.double(), d64(w), mlp)
    rt = runtime(ops, dtype, DEV)
    got = build_ff(rt, W, mlp, w).forward(x.to(rt.dtype).to(DEV)).double().cpu()
    if dtype == "float32":
        torch.testing.assert_close(got, want, atol=5e-5, rtol=1e-4)
    else:
        apart = (got - want).pow(2).mean(-1).sqrt() > 0.05 * want.pow(2).mean().sqrt()
        assert int(apart.sum()) <= T // 50, "rows whose error is more than rounding (a close call of the router may be one)"


# ------------------------------------------------------------------ the engine against the plain model
LENGTHS = {"a": 5, "b": 17, "c": 33, "d": 100, "e": 64, "f": 150, "g": 1, "h": 47}
# A row's error: the root mean square over the vocabulary of the difference of the logits, its mean taken off, over the
# root mean square of the plain logits. In bfloat16 a router may decide a close call the other way: such rows are held to
# the looser bound, at most one in twenty of them.
ROW_ERROR = {"float32": (2e-4, 5e-5), "bfloat16": (1.0, 0.1)}
ROW_ERROR_16_MEAN = 0.04


def make_runner(folder, dtype, max_tokens, page=16, **kw):
    from return_amd.config import EngineConfig
    from return_amd.engine import ModelRunner
    ec = EngineConfig(dtype=dtype, page_size=page, max_token=max_tokens, max_reside=4, max_step_tokens=max(max_tokens, 4),
                      prefill_chunk=max_tokens, tune_products=False, check_invariants=True, **kw)
    return ModelRunner(folder, engine_config=ec)


@pytest.fixture(scope="module", params=sorted(CASES))
def model(request, tmp_path_factory):
    folder = make_folder(tmp_path_factory, request.param)
    cfg, w = plain.read_folder(folder)
    reqs = {rid: tt.random_tokens(cfg["vocab"], n, seed=ord(rid)) for rid, n in LENGTHS.items()}
    want = {rid: plain.logits(cfg, w, toks) for rid, toks in reqs.items()}
    return folder, cfg, reqs, want


def compare(got, want, reqs, dtype):
    errs, apart = [], []
    most, usual = ROW_ERROR[dtype]
    for rid, toks in reqs.items():
        for p in range(len(toks)):
            e = row_error(got[(rid, p)], want[rid][p])
            errs.append(e)
            assert e <= most, f"request {rid} position {p} (first wrong place): row error {e:.3e}"
            if e > usual:
                apart.append((rid, p, f"{e:.1e}"))
    assert len(apart) <= max(2, len(errs) // 20), f"rows far from the plain logits: {apart[:8]}"
    if dtype == "bfloat16":
        assert sum(errs) / len(errs) <= ROW_ERROR_16_MEAN, f"mean row error {sum(errs) / len(errs):.3e}"
    return max(errs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut", ["whole", "tail_decoded", "portions", "mixed"])
def test_engine_matches_plain(model, dtype, cut):
    folder, cfg, reqs, want = model
    steps = {"whole": tt.whole, "tail_decoded": tt.tail_decoded, "portions": tt.portions, "mixed": tt.mixed}[cut](reqs)
    runner = make_runner(folder, dtype, tt.peak_tokens(steps))
    got = tt.run_in_process(runner, steps)
    print(f"mapalorn {dtype} {cut}: largest row error {compare(got, want, reqs, dtype):.2e}")
    assert not runner.cache.live and all(g.pages.in_use() == 0 for g in runner.cache.groups)


@pytest.mark.parametrize("seed", RANDOM_SEEDS)
def test_configurations_drawn_at_random(tmp_path_factory, seed):
    folder = make_folder(tmp_path_factory, seed)
    cfg, w = plain.read_folder(folder)
    lens = {"a": 1 + seed % 3, "b": 20 + seed % 50, "c": 100 + 7 * (seed % 30), "d": 2 + seed % 60}
    reqs = {rid: tt.random_tokens(cfg["vocab"], n, seed=seed + ord(rid)) for rid, n in lens.items()}
    want = {rid: plain.logits(cfg, w, toks) for rid, toks in reqs.items()}
    steps = tt.mixed(reqs, seed=seed)
    got = tt.run_in_process(make_runner(folder, "float32", tt.peak_tokens(steps), page=(4, 16, 64)[seed % 3]), steps)
    compare(got, want, reqs, "float32")
    got = tt.run_in_process(make_runner(folder, "bfloat16", tt.peak_tokens(steps)), steps)
    # (several experts a token and weights as they are: close calls of a router spread through later layers, in an engine
    # of torch operations at the same rounding too; most rows have none)
    rows = sorted(row_error(got[(rid, p)], want[rid][p]) for rid, toks in reqs.items() for p in range(len(toks)))
    assert rows[len(rows) // 2] < 0.06 and sum(rows) / len(rows) < 0.12, f"mean row error {sum(rows) / len(rows):.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["a", "c"])
def test_long_decoding(tmp_path_factory, dtype, name):
    """A short prompt and 380 tokens one by one."""
    folder = make_folder(tmp_path_factory, name)
    cfg, w = plain.read_folder(folder)
    toks = tt.random_tokens(cfg["vocab"], 400, seed=4)
    got = tt.run_in_process(make_runner(folder, dtype, 448), tt.tail_decoded({"r": toks}, tail=380))
    want = {"r": plain.logits(cfg, w, toks)}
    print(f"mapalorn {name} {dtype} long decoding: largest row error {compare(got, want, {'r': toks}, dtype):.2e}")


def test_batches_of_unequal_requests_equal_each_alone(tmp_path_factory):
    folder = make_folder(tmp_path_factory, "b")
    cfg, _ = plain.read_folder(folder)
    reqs = {rid: tt.random_tokens(cfg["vocab"], n, seed=ord(rid)) for rid, n in (("a", 70), ("b", 3), ("c", 41), ("d", 1))}
    sizes = {"a": [30, 1, 1, 38], "b": [1, 2], "c": [2, 39], "d": [1]}
    alone = {}
    for rid, toks in reqs.items():
        r = make_runner(folder, "float32", 256)
        alone.update(tt.run_in_process(r, tt.portions({rid: toks}, sizes=tuple(sizes[rid]))))
    steps, at = [], {rid: 0 for rid in reqs}
    for k in range(4):
        entries, end = [], []
        for rid, toks in reqs.items():
            if k < len(sizes[rid]):
                n = sizes[rid][k]
                entries.append({"id": rid, "tokens": toks[at[rid]:at[rid] + n], "want": list(range(n))})
                at[rid] += n
                if at[rid] == len(toks):
                    end.append(rid)
        steps.append({"step": k, "entries": entries, "end": end})
    together = tt.run_in_process(make_runner(folder, "float32", 256), steps)
    for key, row in alone.items():
        assert row_error(together[key], row) < 2e-5


# ------------------------------------------------------------------ generation and the programs
def test_greedy_generation_through_the_engine(tmp_path_factory):
    from return_amd import SamplingParams
    from return_amd.engine import Engine
    for name in ("a", "c"):
        folder = make_folder(tmp_path_factory, name)
        cfg, w = plain.read_folder(folder)
        prompts = [tt.random_tokens(cfg["vocab"], n, seed=n) for n in (1, 8, 31, 64, 90)]
        want = [plain.greedy(cfg, w, p, 10) for p in prompts]
        for graphs in (False, True):
            eng = Engine(folder, dtype="float32", page_size=16, max_token=1024, max_reside=4, max_step_tokens=64,
                         prefill_chunk=24, use_graphs=graphs, check_invariants=True)
            got = eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=10))
            assert [r.output_ids for r in got] == want, f"model {name}, graphs {graphs}"
            assert not eng.runner.cache.live


def test_bf16_generation_from_graphs_equals_eager(tmp_path_factory):
    from return_amd import SamplingParams
    from return_amd.engine import Engine
    folder = make_folder(tmp_path_factory, "c")
    cfg, _ = plain.read_folder(folder)
    prompts = [tt.random_tokens(cfg["vocab"], n, seed=n) for n in (3, 40, 77)]
    outs = []
    for graphs in (False, True):
        eng = Engine(folder, dtype="bfloat16", page_size=16, max_token=1024, max_reside=4, use_graphs=graphs)
        outs.append([r.output_ids for r in eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=24))])
    assert outs[0] == outs[1]


def test_command_line_makes_a_model_and_generates(tmp_path):
    """random-model writes a folder from a config.json alone; generate answers greedy requests as the plain model would
    and a sampled one with a token among the plain model's first five."""
    import json
    import subprocess
    import sys
    from tests.mapalorn_cases import MAPA_A
    cfg_path = tmp_path / "config.json"
    cfg_path.write_text(json.dumps(MAPA_A))
    folder = str(tmp_path / "model")
    made = subprocess.run([sys.executable, "-m", "return_amd.cli", "random-model", "--config", str(cfg_path), "--out", folder,
                           "--seed", "5", "--std", "0.15", "--embedding-std", "0.5"], cwd=tt.ROOT, capture_output=True, text=True,
                          timeout=300)
    assert made.returncode == 0, made.stderr
    cfg, w = plain.read_folder(folder)
    reqs = [{"session_id": "s0", "prompt_ids": tt.random_tokens(cfg["vocab"], 9, seed=1), "max_new_tokens": 5, "temperature": 0.0},
            {"session_id": "s1", "prompt_ids": tt.random_tokens(cfg["vocab"], 40, seed=2), "max_new_tokens": 4, "temperature": 0.0},
            {"session_id": "s2", "prompt_ids": tt.random_tokens(cfg["vocab"], 3, seed=3), "max_new_tokens": 6, "temperature": 0.8,
             "top_k": 5, "top_p": 0.9}]
    f = tmp_path / "reqs.jsonl"
    f.write_text("\n".join(json.dumps(r) for r in reqs))
    out = subprocess.run([sys.executable, "-m", "return_amd.cli", "generate", "--model", folder, "--dtype", "float32",
                          "--max-reside", "4", "--max-token", "1024", "--requests", str(f)],
                         cwd=tt.ROOT, capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr
    lines = [json.loads(l) for l in out.stdout.strip().splitlines()]
    assert [l["session_id"] for l in lines] == ["s0", "s1", "s2"]
    for l, r in zip(lines[:2], reqs[:2]):
        assert l["output_ids"] == plain.greedy(cfg, w, r["prompt_ids"], r["max_new_tokens"])
    toks = reqs[2]["prompt_ids"] + lines[2]["output_ids"]
    lg = plain.logits(cfg, w, toks)
    for i, tok in enumerate(lines[2]["output_ids"]):
        assert tok in lg[len(reqs[2]["prompt_ids"]) - 1 + i].topk(5).indices.tolist()


def test_trace_program_on_a_model_folder(tmp_path_factory, tmp_path):
    folder = make_folder(tmp_path_factory, "a")
    cfg, w = plain.read_folder(folder)
    reqs = {rid: tt.random_tokens(cfg["vocab"], n, seed=ord(rid)) for rid, n in (("a", 40), ("b", 7), ("c", 90))}
    steps = tt.mixed(reqs, seed=3, max_live=3)
    got = tt.run_program(folder, "float32", steps, str(tmp_path), tt.peak_tokens(steps), cfg["vocab"],
                         env=dict(os.environ))
    compare(got, {rid: plain.logits(cfg, w, t) for rid, t in reqs.items()}, reqs, "float32")
