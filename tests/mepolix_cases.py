"""Small Mepolix configurations for the tests, each with random weights of its own, and helpers that build one mixer
of the package. The configurations differ from one another in every size and option: which mixer comes first, layers
that use an earlier (or a later) layer's tensors, grouped and ungrouped heads, values narrower than, as wide as and
wider than keys, rotation over all of a head, part of it and none, stretched and unstretched, recurrences narrower and
wider than the stream, one block and several, blocks that are no multiple of eight, filters of one to eight taps, layers
with and without feed-forward behind either mixer, with and without a soft cap, widths that are no multiple of 8."""
from __future__ import annotations

import torch

from tests.fefulorn_cases import run_in_pieces, runtime  # noqa: F401  (used by the tests through this file)


def _left(heads, kv_heads, dim, scale, vdim=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "scale": scale}
    if vdim:
        m["vdim"] = vdim
    if rot:
        base, dims, stretch = rot
        m["rot"] = {"base": base, "dims": dims}
        if stretch:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), stretch))
    return m


def _parallel(left, right, scales, ff=None):
    width, blocks, conv = right
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left, "right": {"width": width, "blocks": blocks, "conv": conv},
                      "left_scale": scales[0], "right_scale": scales[1]}}


def _delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "delta", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def _again(layers, j):
    layers.append(dict(layers[j], weights_of=j))
    return layers


# begins with the delta rule; values wider than keys; part of a head turns; both mixers with and without feed-forward;
# layers 3 and 4 use the tensors of layers 1 and 0
MEPO_A = {
    "architecture": "Mepolix", "vocab": 203, "width": 56, "norm": {"eps": 1e-5}, "logit_softcap": 6.0,
    "layers": _again(_again([
        _delta(4, 2, 6, 10, 3, 40),
        _parallel(_left(4, 2, 8, 0.5, 12, (1000.0, 6, (4.0, 32, 8.0, 1.0))), (48, 3, 4), (0.7, 1.3), 24),
        _parallel(_left(3, 3, 10, 0.3, 4, (50.0, 10, None)), (40, 5, 2), (1.0, 0.4)),
    ], 1), 0)}
MEPO_A_INIT = dict(seed=51, std=0.15, embedding_std=0.6, norm_jitter=0.1)

# a width that is no multiple of 8, one head, one block, filters of one and eight taps, no rotation, no soft cap; the
# first layer uses the tensors of a later one
MEPO_B = {
    "architecture": "Mepolix", "vocab": 91, "width": 44, "norm": {"eps": 4e-6},
    "layers": [
        dict(_delta(3, 1, 12, 7, 5), weights_of=2),
        _parallel(_left(2, 1, 6, 0.4), (36, 1, 1), (-0.5, 2.0), 12),
        _delta(3, 1, 12, 7, 5),
        _parallel(_left(1, 1, 14, 0.25, None, (700.0, 14, (3.0, 20, 4.0, 0.5))), (27, 3, 8), (2.0, 0.25)),
    ]}
MEPO_B_INIT = dict(seed=52, std=0.2, embedding_std=0.8, norm_jitter=0.2)

# sizes in multiples of 16 throughout (what the matrix-core kernels take), heads of 32 and 64
MEPO_C = {
    "architecture": "Mepolix", "vocab": 160, "width": 96, "norm": {"eps": 1e-6}, "logit_softcap": 20.0,
    "layers": _again([
        _parallel(_left(4, 2, 32, 0.2, 32, (20000.0, 32, (2.0, 64, 16.0, 2.0))), (112, 7, 4), (0.8, 1.5), 64),
        _delta(4, 4, 16, 16, 4),
        _parallel(_left(6, 1, 64, 0.125, 48, (10000.0, 32, None)), (64, 2, 3), (1.2, 0.9)),
        _delta(2, 1, 32, 48, 2, 48),
    ], 2)}
MEPO_C_INIT = dict(seed=53, std=0.12, embedding_std=0.5, norm_jitter=0.05)

CASES = {"a": (MEPO_A, MEPO_A_INIT), "b": (MEPO_B, MEPO_B_INIT), "c": (MEPO_C, MEPO_C_INIT)}


def random_case(seed):
    """A configuration drawn from a seed: one to six layers, every size and option drawn on its own."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.choice([1, 2, 3, 4, 5, 6])):
        own = [j for j, layer in enumerate(layers) if "weights_of" not in layer]
        if own and rng.random() < 0.25:
            _again(layers, rng.choice(own))
            continue
        ff = rng.choice([None, 8, 20, 48, 72])
        kv = rng.choice([1, 2, 3])
        if rng.random() < 0.5:
            dim = rng.choice([4, 6, 16, 32, 48, 64, 80])
            rot = None
            if rng.random() < 0.8:
                stretch = None
                if rng.random() < 0.7:
                    stretch = (rng.choice([1.0, 2.0, 8.0]), rng.choice([8, 50, 400]), rng.choice([4.0, 32.0]), rng.choice([0.5, 1.0]))
                rot = (rng.choice([10.0, 10000.0, 500000.0]), rng.choice(range(2, dim + 1, 2)), stretch)
            blocks = rng.choice([1, 2, 3, 4])
            left = _left(kv * rng.choice([1, 2, 4, 17]), kv, dim, rng.choice([dim ** -0.5, 0.2, 0.6]), rng.choice([None, 3, 16, 24, 96]), rot)
            layers.append(_parallel(left, (blocks * rng.choice([3, 8, 16, 20, 40, 72]), blocks, rng.choice([1, 2, 3, 4, 8])),
                                    (rng.choice([1.0, 0.3, 1.7]), rng.choice([1.0, 0.6, -1.2])), ff))
        else:
            layers.append(_delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([3, 4, 8, 16, 33, 64]),
                                 rng.choice([4, 7, 12, 16, 32, 130]), rng.choice([1, 2, 3, 4, 7]), ff))
    raw = {"architecture": "Mepolix", "vocab": rng.choice([50, 97, 256]), "width": rng.choice([16, 24, 44, 64, 96, 200]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}, "layers": layers}
    cap = rng.choice([None, 3.0, 30.0])
    if cap:
        raw["logit_softcap"] = cap
    return raw, dict(seed=seed, std=0.15, embedding_std=0.5, norm_jitter=0.1)


def make_folder(tmp_path_factory, name, dtype="bfloat16"):
    from tests.conftest import make_folder as make
    raw, init = random_case(name) if isinstance(name, int) else CASES[name]
    return make(tmp_path_factory, "mepolix_" + str(name), dict(raw, architectures=[raw["architecture"]]), init, dtype)


# ------------------------------------------------------------------ one mixer of the package
def _r(g, dtype):
    return lambda *shape, s=1.0: (s * torch.randn(*shape, generator=g)).to(dtype)


def attention_tensors(g, W, m, dtype=torch.float32):
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    Dv = m.get("vdim") or D
    r = _r(g, dtype)
    return {"q": r(H * D, W, s=W ** -0.5), "k": r(G * D, W, s=W ** -0.5), "v": r(G * Dv, W, s=W ** -0.5),
            "q.norm": (1 + 0.2 * r(D)).to(dtype), "k.norm": (1 + 0.2 * r(D)).to(dtype), "sink": r(H),
            "o": r(W, H * Dv, s=(H * Dv) ** -0.5)}


def recurrence_tensors(g, W, m, dtype=torch.float32):
    C, B, K = m["width"], m["blocks"], m["conv"]
    bw = C // B
    r = _r(g, dtype)
    return {"y": r(C, W, s=W ** -0.5), "y.b": r(C, s=0.3), "x": r(C, W, s=W ** -0.5), "x.b": r(C, s=0.3),
            "conv": r(C, K, s=0.5), "conv.b": r(C, s=0.2), "ra": r(B, bw, bw, s=bw ** -0.5), "ra.b": r(B, bw, s=0.5),
            "ri": r(B, bw, bw, s=bw ** -0.5), "ri.b": r(B, bw, s=0.5), "lam": (r(C) - 3.0).to(dtype), "o": r(W, C, s=C ** -0.5)}


def delta_tensors(g, W, m, dtype=torch.float32):
    H, G, D, V, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    r = _r(g, dtype)
    return {"q": r(G * D, W, s=W ** -0.5), "k": r(G * D, W, s=W ** -0.5), "v": r(H * V, W, s=W ** -0.5),
            "q.conv": r(G * D, K, s=0.5), "k.conv": r(G * D, K, s=0.5), "v.conv": r(H * V, K, s=0.5),
            "b": r(H, W, s=W ** -0.5), "a": r(H, W, s=W ** -0.5), "A_log": r(H, s=0.5), "dt_bias": (r(H) - 1.5).to(dtype),
            "norm": (1 + 0.2 * r(V)).to(dtype), "g": r(H * V, W, s=W ** -0.5), "o": r(W, H * V, s=(H * V) ** -0.5)}


ATTENTION_ROLES = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink",
                   "o_proj": "o"}
RECURRENCE_ROLES = {"y_proj": "y", "y_bias": "y.b", "x_proj": "x", "x_bias": "x.b", "conv": "conv", "conv_bias": "conv.b",
                    "r_gate": "ra", "r_bias": "ra.b", "i_gate": "ri", "i_bias": "ri.b", "lam": "lam", "o_proj": "o"}


def _on(rt, w, roles):
    return {role: w[name].to(rt.dtype).to(rt.device) for role, name in roles.items()}


def _attention_params(rt, W, m, eps):
    from return_amd.parts.position import RotaryPosition
    shared, rot = {}, m.get("rot")
    if rot:
        shared["p"] = RotaryPosition({"head_dim": m["dim"], "rotary_dim": rot["dims"], "theta": rot["base"],
                                      "max_position": None, "exact_tables": True, "scaling": rot.get("scaling")}, {}, rt)
    return {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m.get("vdim") or m["dim"], "scale": m["scale"], "bias": False, "qk_norm_eps": eps, "sink": True,
            "fine_weights": True, "window": None, "position": "p" if rot else None}, shared


def _recurrence_params(W, m):
    return {"hidden_size": W, "width": m["width"], "blocks": m["blocks"], "conv_taps": m["conv"]}


def build_attention(rt, W, m, w, eps):
    from return_amd.parts.attention import BlendAttention
    params, shared = _attention_params(rt, W, m, eps)
    return BlendAttention(params, _on(rt, w, ATTENTION_ROLES), rt, shared)


def build_recurrence(rt, W, m, w):
    from return_amd.parts.channel import GatedChannelRecurrence
    return GatedChannelRecurrence(_recurrence_params(W, m), _on(rt, w, RECURRENCE_ROLES), rt)


def build_parallel(rt, W, m, w_left, w_right, eps):
    from return_amd.parts.side_by_side import SideBySideMixer
    left, shared = _attention_params(rt, W, m["left"], eps)
    params = {"hidden_size": W, "sides": [
        {"name": "left", "kind": "blend_attention", "params": left, "scale": m["left_scale"]},
        {"name": "right", "kind": "gated_channel_recurrence", "params": _recurrence_params(W, m["right"]), "scale": m["right_scale"]}]}
    tensors = {"left." + k: v for k, v in _on(rt, w_left, ATTENTION_ROLES).items()}
    tensors.update({"right." + k: v for k, v in _on(rt, w_right, RECURRENCE_ROLES).items()})
    assert {k: tuple(v.shape) for k, v in tensors.items()} == SideBySideMixer.tensor_shapes(params)
    return SideBySideMixer(params, tensors, rt, shared)


def build_delta(rt, W, m, w, eps):
    from return_amd.parts.delta import HeadDeltaMixer
    params = {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
              "value_dim": m["vdim"], "conv_taps": m["conv"], "eps": eps}
    roles = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv",
             "b_proj": "b", "a_proj": "a", "A_log": "A_log", "dt_bias": "dt_bias", "o_norm": "norm", "g_proj": "g", "o_proj": "o"}
    return HeadDeltaMixer(params, _on(rt, w, roles), rt)


def deciding_rows(T, W, query_at, key_at, w, m, seed):
    """(rows [T, W], the scale) such that one key decides for the row at query_at: every head of q and k is made a unit
    vector times a weight, so a row far out would not stand out by its length; here all rows are near one direction d and
    the query's map is minus the key's map, so every score is far below zero but that of the key at key_at, whose row is
    the opposite, -d. The scale sets the scores about 20 apart. Changes w: q becomes minus k's map, the norms' weights
    agree, the sink is far below."""
    D, G, H = m["dim"], m["kv_heads"], m["heads"]
    g = torch.Generator().manual_seed(seed)
    w["q"] = -w["k"].view(G, D, W).repeat_interleave(H // G, 0).reshape(-1, W).contiguous()
    w["q.norm"] = w["k.norm"].clone()
    d = torch.randn(W, generator=g)
    x = d[None, :] + 0.02 * torch.randn(T, W, generator=g)
    x[query_at], x[key_at] = d, -d
    kn = (w["k"].double() @ d.double()).view(G, D)
    kn = kn / torch.sqrt((kn * kn).mean(-1, keepdim=True)) * w["k.norm"].double()
    return x, float(10.0 / (kn * kn).sum(-1).min())
