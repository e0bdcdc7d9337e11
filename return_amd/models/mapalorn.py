"""Mapalorn as a ModelSpec: a decoder whose layers are described one by one in config.json.

A layer has one layer norm (weight and bias) and two sublayers side by side that both read it: h += mixer(norm(h)) +
ff(norm(h)), the feed-forward optional. The mixer is an attention over a latent row per token (queries straight from the
stream, a rotated key part of neighbouring pairs shared by all heads, a learned sink per head) or a grouped attention with
norms over the whole query and key projections, a one in the softmax's denominator and a gate on every element of its
output. The feed-forward is dense with clamped halves, or a mixture of experts that read the token times its raw sigmoid
score beside a shared expert behind a gate. A run of layers may be gone through several times in a row. Tensor names:
"embed", "final.norm", "head", and "l<i>." + norm1, mix.*, mlp.*; a norm's bias is its name + ".b".
"""
from __future__ import annotations

from ..config.base import register_architecture
from ..config.mapalorn import MapalornConfig
from ..parts.moe import GroupedRoutedExperts
from ..parts.spec import BlockSpec, LayerCall, ModelSpec, PartSpec


def _rotary(positions, head_dim, rot, pairing):
    """The name of the shared rotary part of these constants."""
    name = f"rotary_{pairing}_{head_dim}_{int(rot['dims'])}_{float(rot['base'])!r}"
    positions.setdefault(name, PartSpec("rotary", {
        "head_dim": head_dim, "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]), "max_position": None,
        "exact_tables": True, "pairing": pairing}))
    return name


def _latent_attention(cfg, i, m, positions):
    p = f"l{i}.mix."
    params = {"hidden_size": cfg.width, "num_heads": int(m["heads"]), "head_dim": int(m["dim"]), "rot_dim": int(m["rot_dim"]),
              "value_dim": int(m["vdim"]), "direct_q": True, "kv_rank": int(m["kv_rank"]), "scale": float(m["scale"]),
              "eps": float(cfg.norm["eps"]), "position": _rotary(positions, int(m["rot_dim"]), m["rot"], "interleaved"),
              "sink": True, "gate": False, "window": None}
    names = {"q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "sink": "sink", "o": "o"}
    return PartSpec("latent_attention", params, {role: p + name for role, name in names.items()})


def _attention(cfg, i, m, positions):
    p = f"l{i}.mix."
    dim = int(m["dim"])
    params = {"hidden_size": cfg.width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": dim,
              "value_dim": int(m.get("vdim") or dim), "scale": float(m["scale"]), "bias": False,
              "row_norm_eps": float(cfg.norm["eps"]), "sink_one": True, "gate": True, "fine_weights": True, "window": None,
              "position": _rotary(positions, dim, m["rot"], "half") if m.get("rot") else None}
    names = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "q_norm": "q.norm", "k_norm": "k.norm", "g_proj": "g", "o_proj": "o"}
    return PartSpec("blend_attention", params, {role: p + name for role, name in names.items()})


def _feed_forward(cfg, i, mlp):
    p = f"l{i}.mlp."
    if mlp["kind"] == "dense":
        return PartSpec("clamped_glu", {"hidden_size": cfg.width, "intermediate_size": int(mlp["ff"]),
                                        "limit": float(mlp["limit"]), "slope": 1.702},
                        {"gate_proj": p + "gate", "up_proj": p + "up", "down_proj": p + "down"})
    experts = int(mlp["router"]["experts"])
    params = {"hidden_size": cfg.width, "expert_size": int(mlp["expert"]["ff"]), "experts": experts,
              "top": int(mlp["router"]["top"]), "router": "sigmoid_raw", "activation": "silu", "weigh": "input"}
    tensors = GroupedRoutedExperts.tensor_names(p, experts)
    del tensors["correction"]
    if mlp.get("shared") is not None:
        params.update({"shared": {"size": int(mlp["shared"]["ff"])}, "joint_router": True})
        tensors.update({"shared_gate": p + "shared.gate", "shared_up": p + "shared.up", "shared_down": p + "shared.down",
                        "shared_weight": p + "shared.sg"})
    return PartSpec("routed_experts", params, tensors)


def build_spec(cfg: MapalornConfig) -> ModelSpec:
    W, eps = cfg.width, float(cfg.norm["eps"])
    norm = lambda name: PartSpec("layer_norm", {"size": W, "eps": eps, "bias": True}, {"weight": name, "bias": name + ".b"})
    positions, blocks = {}, []
    for i, layer in enumerate(cfg.layers):
        mixer = _latent_attention if layer["type"] == "latent_attention" else _attention
        parts = {"mixer_norm": ("norm", norm(f"l{i}.norm1")), "mixer": ("mixer", mixer(cfg, i, layer["mixer"], positions))}
        if layer.get("mlp") is not None:
            parts["feed_forward"] = ("feed_forward", _feed_forward(cfg, i, layer["mlp"]))
        blocks.append(BlockSpec(parts, "parallel_pre_norm"))
    # every run of a layer has a cache layer of its own
    schedule = [LayerCall(block=i, cache=run, writes_cache=True) for run, i in enumerate(cfg.run_order())]
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=W, vocab_size=cfg.vocab, max_position=None,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": W}, {"weight": "embed"}),
        positions=positions, blocks=blocks, schedule=schedule, final_norm=norm("final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": W}, {"weight": "head"}))


register_architecture("Mapalorn", MapalornConfig, build_spec)
