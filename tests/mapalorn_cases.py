"""Small Mapalorn configurations for the tests, each with random weights of its own, and helpers that build one mixer of
the package. The configurations differ from one another in every size and option: which mixer comes first, runs of one
layer, of several and of all layers gone through one to four times, grouped and ungrouped heads, one head, values narrower
than, as wide as and wider than keys, rotation over all of a head, part of it and none, latents narrower and wider than a
head, dense feed-forwards, mixtures of experts with top 1, several and all, with and without the shared expert (narrower
and wider than the others), layers without feed-forward behind either mixer, widths that are no multiple of 8."""
from __future__ import annotations

import torch

from tests.fefulorn_cases import run_in_pieces, runtime  # noqa: F401  (used by the tests through this file)


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim}}}


def _attn(heads, kv_heads, dim, scale, vdim=None, rot=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "scale": scale}
    if vdim:
        m["vdim"] = vdim
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def _dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


# begins with the attention; values wider than keys, part of a head turns; a run of three layers gone through twice, in
# whose middle there is a layer without feed-forward; top 2 of 5
MAPA_A = {
    "architecture": "Mapalorn", "vocab": 203, "width": 56, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 4, "times": 2},
    "layers": [
        _attn(4, 2, 8, 0.6, 12, (1000.0, 6), _moe(24, 5, 2, 20)),
        _latent(3, 10, 6, 14, 20, 0.4, 500.0, _dense(40, 0.8)),
        _attn(6, 3, 10, 0.5, 4, (50.0, 10), None),
        _latent(4, 6, 4, 8, 12, 0.5, 10000.0, _moe(16, 6, 1, 36)),
        _latent(2, 7, 2, 5, 9, 0.6, 20.0, None),
    ]}
MAPA_A_INIT = dict(seed=61, std=0.14, embedding_std=0.6, norm_jitter=0.1)

# begins with the latent attention; a width that is no multiple of 8, one head, no rotation in the attention, no shared
# expert, every expert chosen; no loop
MAPA_B = {
    "architecture": "Mapalorn", "vocab": 91, "width": 44, "norm": {"eps": 4e-6},
    "layers": [
        _latent(1, 9, 8, 11, 18, 0.35, 300.0, _moe(10, 4, 4)),
        _attn(5, 1, 6, 0.7, None, None, _dense(28, 2.5)),
        _attn(3, 3, 14, 0.3, 14, (700.0, 14), _moe(12, 3, 2, 6)),
        _latent(5, 4, 10, 6, 7, 0.5, 1000.0, _moe(22, 2, 1)),
    ]}
MAPA_B_INIT = dict(seed=62, std=0.18, embedding_std=0.8, norm_jitter=0.2)

# sizes in multiples of 16 throughout (what the matrix-core kernels take); the first layer gone through four times
MAPA_C = {
    "architecture": "Mapalorn", "vocab": 160, "width": 96, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 1, "times": 4},
    "layers": [
        _latent(4, 32, 16, 48, 64, 0.16, 20000.0, _moe(32, 8, 3, 48)),
        _attn(4, 2, 32, 0.2, 32, (20000.0, 32), _dense(64, 1.2)),
        _latent(16, 16, 32, 16, 32, 0.14, 10000.0, _moe(48, 4, 1, 16)),
        _attn(6, 1, 64, 0.125, 48, (10000.0, 32), _moe(16, 16, 5, 32)),
        _latent(6, 48, 64, 32, 96, 0.1, 500000.0, None),
    ]}
MAPA_C_INIT = dict(seed=63, std=0.1, embedding_std=0.5, norm_jitter=0.05)

CASES = {"a": (MAPA_A, MAPA_A_INIT), "b": (MAPA_B, MAPA_B_INIT), "c": (MAPA_C, MAPA_C_INIT)}


def random_case(seed):
    """A configuration drawn from a seed: one to five layers, every size and option drawn on its own."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.choice([1, 2, 3, 4, 5])):
        mlp = None
        kind = rng.choice(["dense", "moe", "moe", "moe", None])
        if kind == "dense":
            mlp = _dense(rng.choice([8, 20, 48, 72]), rng.choice([0.4, 1.0, 7.0]))
        elif kind == "moe":
            experts = rng.choice([1, 2, 3, 4, 7, 12])
            mlp = _moe(rng.choice([4, 8, 24, 40]), experts, rng.randint(1, min(experts, 5)), rng.choice([None, 4, 13, 32]))
        if rng.random() < 0.6:
            dim, rot_dim = rng.choice([2, 5, 8, 16, 48]), rng.choice([2, 4, 6, 16, 32, 64])
            layers.append(_latent(rng.choice([1, 2, 3, 6, 9, 16]), dim, rot_dim, rng.choice([3, 8, 16, 40]),
                                  rng.choice([4, 7, 16, 32, 48, 64, 96, 128]), rng.choice([(dim + rot_dim) ** -0.5, 0.2, 0.5]),
                                  rng.choice([10.0, 10000.0, 500000.0]), mlp))
        else:
            dim, kv = rng.choice([4, 6, 16, 32, 48, 64, 80]), rng.choice([1, 2, 3])
            rot = (rng.choice([10.0, 10000.0, 500000.0]), rng.choice(range(2, dim + 1, 2))) if rng.random() < 0.85 else None
            layers.append(_attn(kv * rng.choice([1, 2, 4, 17]), kv, dim, rng.choice([dim ** -0.5, 0.2, 0.6]),
                                rng.choice([None, 3, 16, 24, 96]), rot, mlp))
    raw = {"architecture": "Mapalorn", "vocab": rng.choice([50, 97, 256]), "width": rng.choice([16, 24, 44, 64, 96, 200]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}, "layers": layers}
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        raw["loop"] = {"start": start, "stop": rng.randint(start + 1, len(layers)), "times": rng.choice([1, 2, 3])}
    return raw, dict(seed=seed, std=0.15, embedding_std=0.5, norm_jitter=0.1)


def make_folder(tmp_path_factory, name, dtype="bfloat16"):
    from tests.conftest import make_folder as make
    raw, init = random_case(name) if isinstance(name, int) else CASES[name]
    return make(tmp_path_factory, "mapalorn_" + str(name), dict(raw, architectures=[raw["architecture"]]), init, dtype)


# ------------------------------------------------------------------ one mixer of the package
def _r(g, dtype):
    return lambda *shape, s=1.0: (s * torch.randn(*shape, generator=g)).to(dtype)


def latent_tensors(g, W, m, dtype=torch.float32):
    H, D, R, V, C = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    r = _r(g, dtype)
    return {"q": r(H * (D + R), W, s=2 * W ** -0.5), "dkv": r(C + R, W, s=2 * W ** -0.5), "dkv.norm": (1 + 0.2 * r(C)).to(dtype),
            "uk": r(H * D, C, s=2 * C ** -0.5), "uv": r(H * V, C, s=C ** -0.5), "sink": r(H), "o": r(W, H * V, s=(H * V) ** -0.5)}


def attention_tensors(g, W, m, dtype=torch.float32):
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    V = m.get("vdim") or D
    r = _r(g, dtype)
    return {"q": r(H * D, W, s=W ** -0.5), "k": r(G * D, W, s=W ** -0.5), "v": r(G * V, W, s=W ** -0.5),
            "q.norm": (1 + 0.3 * r(H * D)).to(dtype), "k.norm": (1 + 0.3 * r(G * D)).to(dtype), "g": r(H * V, W, s=W ** -0.5),
            "o": r(W, H * V, s=(H * V) ** -0.5)}


def ff_tensors(g, W, mlp, dtype=torch.float32):
    r = _r(g, dtype)
    three = lambda p, n: {p + "gate": r(n, W, s=1.5 * W ** -0.5), p + "up": r(n, W, s=1.5 * W ** -0.5), p + "down": r(W, n, s=n ** -0.5)}
    if mlp["kind"] == "dense":
        return three("", mlp["ff"])
    w = {"router": r(mlp["router"]["experts"], W, s=2 * W ** -0.5)}
    for e in range(mlp["router"]["experts"]):
        w.update(three(f"e{e}.", mlp["expert"]["ff"]))
    if mlp.get("shared"):
        w.update(three("shared.", mlp["shared"]["ff"]))
        w["shared.sg"] = r(1, W, s=W ** -0.5)
    return w


def _one_layer(rt, W, layer, w, eps, prefix):
    """The PartSpec that the model's builder makes of one layer's mixer or feed-forward, its shared parts, and its tensors."""
    from return_amd.config.mapalorn import MapalornConfig
    from return_amd.models.mapalorn import build_spec
    from return_amd.parts.registry import part_class
    cfg = MapalornConfig.from_dict({"architecture": "Mapalorn", "vocab": 8, "width": W, "norm": {"eps": eps}, "layers": [layer]})
    spec = build_spec(cfg)
    name, category = ("mixer", "mixer") if prefix == "l0.mix." else ("feed_forward", "feed_forward")
    ps = spec.blocks[0].part(name)
    shared = {k: part_class("position", p.kind)(p.params, {}, rt) for k, p in spec.positions.items()}
    tensors = {role: w[t[len(prefix):]].to(rt.dtype).to(rt.device) for role, t in ps.tensors.items()}
    cls = part_class(category, ps.kind)
    assert {k: tuple(v.shape) for k, v in tensors.items()} == {k: tuple(v) for k, v in cls.tensor_shapes(ps.params).items()}
    return cls(ps.params, tensors, rt, shared)


def build_mixer(rt, W, kind, m, w, eps):
    return _one_layer(rt, W, {"type": kind, "mixer": m, "mlp": None}, w, eps, "l0.mix.")


def build_ff(rt, W, mlp, w):
    layer = _latent(1, 2, 2, 2, 2, 1.0, 10.0, mlp)
    return _one_layer(rt, W, layer, w, 1e-5, "l0.mlp.")


# ------------------------------------------------------------------ inputs of which one key decides
def deciding_attention_rows(T, W, query_at, key_at, w, m, seed):
    """(rows [T, W], the scale) such that one key decides for the row at query_at in every head: all rows lie near one
    direction d and the query's map is minus the key's map, so every score is far below zero but that of the key at key_at,
    whose row is -d. The scale sets the scores about 40 apart. Changes w: q becomes minus k's map, the norms' weights agree
    (the whole query row then has the key row's root mean square, the group's heads being copies)."""
    D, G, H = m["dim"], m["kv_heads"], m["heads"]
    g = torch.Generator().manual_seed(seed)
    w["q"] = -w["k"].view(G, D, W).repeat_interleave(H // G, 0).reshape(-1, W).contiguous()
    w["q.norm"] = w["k.norm"].view(G, D).repeat_interleave(H // G, 0).reshape(-1).contiguous()
    d = torch.randn(W, generator=g)
    x = d[None, :] + 0.02 * torch.randn(T, W, generator=g)
    x[query_at], x[key_at] = d, -d
    kn = w["k"].double() @ d.double()
    kn = (kn / torch.sqrt((kn * kn).mean()) * w["k.norm"].double()).view(G, D)
    return x, float(20.0 / (kn * kn).sum(-1).min())


def deciding_latent_rows(T, W, query_at, key_at, w, m, seed):
    """The same for the latent attention's unrotated part: W_q of a head becomes minus W_uk times the latent's map (without
    its root mean square), its rotated rows are made small."""
    H, D, R, C = (m[k] for k in ("heads", "dim", "rot_dim", "kv_rank"))
    g = torch.Generator().manual_seed(seed)
    d = torch.randn(W, generator=g)
    c = w["dkv"][:C].double() @ d.double()
    q = w["q"].view(H, D + R, W).clone()
    q[:, :D] = -torch.einsum("hdc,cw->hdw", w["uk"].double().view(H, D, C) * w["dkv.norm"].double(),
                             w["dkv"][:C].double() / torch.sqrt((c * c).mean())).to(q.dtype)
    q[:, D:] *= 0.02
    w["q"] = q.reshape(H * (D + R), W)
    x = d[None, :] + 0.02 * torch.randn(T, W, generator=g)
    x[query_at], x[key_at] = d, -d
    k = torch.einsum("hdc,c->hd", w["uk"].double().view(H, D, C), c / torch.sqrt((c * c).mean()) * w["dkv.norm"].double())
    return x, float(20.0 / (k * k).sum(-1).min())


def deciding_rotated_rows(T, W, query_at, key_at, w, m, seed):
    """(rows, the scale) such that the rotated part decides: of the rows in front of the query only the one at key_at has
    anything in the first coordinate, the only one that the shared key part reads; every head's rotated query is the key's
    part turned (neighbours 2i, 2i + 1) by the distance between the two, so that exactly that distance fits."""
    H, D, R, C = (m[k] for k in ("heads", "dim", "rot_dim", "kv_rank"))
    g = torch.Generator().manual_seed(seed)
    a = torch.randn(R, generator=g).double()
    f = float(m["rot"]["base"]) ** (-2.0 * torch.arange(R // 2).double() / R)
    t = (key_at - query_at) * f
    turned = torch.stack([a[0::2] * t.cos() - a[1::2] * t.sin(), a[1::2] * t.cos() + a[0::2] * t.sin()], dim=1).reshape(R)
    dkv, q = w["dkv"].clone(), w["q"].view(H, D + R, W).clone()
    dkv[C:] = 0
    dkv[C:, 0] = a.to(dkv.dtype)
    q[:, :D] *= 0.01
    q[:, D:] = 0
    q[:, D:, 0] = turned.to(q.dtype)
    w["dkv"], w["q"] = dkv, q.reshape(H * (D + R), W)
    x = torch.randn(T, W, generator=g)
    x[:, 0] = 0.0
    x[query_at, 0] = x[key_at, 0] = 2.0
    apart = float((a * a).sum() - (a * turned).sum())       # (the query's own key is the only rival)
    assert apart > 0.15 * float((a * a).sum()), "the distance's turn leaves the key part where it was: other sizes"
    return x, float(12.0 / apart)
