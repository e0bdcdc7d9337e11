"""Mepolix as a ModelSpec: a decoder whose layers are described one by one in config.json.

A sublayer reads the stream as it is and enters it through a layer norm of its output: h += norm1(mixer(h)), then
h += norm2(ff(h)), the feed-forward optional. The mixer is a gated delta rule with one decay per head and token, or two
mixers side by side on the same input, each times a factor: a grouped attention (norms on queries and keys, a rotation
stretched for long contexts, a learned sink per head) and a gated linear recurrence per channel behind a short filter.
The feed-forward is a dense gated one. A layer may use another layer's tensors (it is one more call of that layer's
block, with a cache and state of its own). The logits pass a soft cap. Tensor names: "embed", "final.norm", "head", and
"l<i>." + norm1, norm2, mix.*, mlp.*.
"""
from __future__ import annotations

from ..config.base import register_architecture
from ..config.mepolix import MepolixConfig
from ..parts.spec import BlockSpec, LayerCall, ModelSpec, PartSpec


def _parallel(cfg, i, m, positions):
    p = f"l{i}.mix."
    left, right = m["left"], m["right"]
    dim, rot = int(left["dim"]), left.get("rot")
    position = None
    if rot is not None:
        stretch = rot.get("scaling")
        stretch = {k: float(stretch[k]) for k in ("factor", "original", "fast", "slow")} if stretch else None
        position = f"rotary_{dim}_{int(rot['dims'])}_{float(rot['base'])!r}" + \
            ("_" + "_".join(repr(v) for v in stretch.values()) if stretch else "")
        positions.setdefault(position, PartSpec("rotary", {
            "head_dim": dim, "rotary_dim": int(rot["dims"]), "theta": float(rot["base"]), "max_position": None,
            "exact_tables": True, "scaling": stretch}))
    attention = {"hidden_size": cfg.width, "num_heads": int(left["heads"]), "num_kv_heads": int(left["kv_heads"]),
                 "head_dim": dim, "value_dim": int(left.get("vdim") or dim), "scale": float(left["scale"]), "bias": False,
                 "qk_norm_eps": float(cfg.norm["eps"]), "sink": True, "fine_weights": True, "window": None,
                 "position": position}
    recurrence = {"hidden_size": cfg.width, "width": int(right["width"]), "blocks": int(right["blocks"]),
                  "conv_taps": int(right["conv"])}
    scale = lambda key: float(m[key]) if m.get(key) is not None else 1.0
    params = {"hidden_size": cfg.width, "sides": [
        {"name": "left", "kind": "blend_attention", "params": attention, "scale": scale("left_scale")},
        {"name": "right", "kind": "gated_channel_recurrence", "params": recurrence, "scale": scale("right_scale")}]}
    names = {"left.q_proj": "left.q", "left.k_proj": "left.k", "left.v_proj": "left.v", "left.q_norm": "left.q.norm",
             "left.k_norm": "left.k.norm", "left.sink": "left.sink", "left.o_proj": "left.o", "right.y_proj": "right.y",
             "right.y_bias": "right.y.b", "right.x_proj": "right.x", "right.x_bias": "right.x.b", "right.conv": "right.conv",
             "right.conv_bias": "right.conv.b", "right.r_gate": "right.ra", "right.r_bias": "right.ra.b",
             "right.i_gate": "right.ri", "right.i_bias": "right.ri.b", "right.lam": "right.lam", "right.o_proj": "right.o"}
    return PartSpec("side_by_side", params, {role: p + name for role, name in names.items()})


def _delta(cfg, i, m):
    p = f"l{i}.mix."
    params = {"hidden_size": cfg.width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]),
              "head_dim": int(m["dim"]), "value_dim": int(m["vdim"]), "conv_taps": int(m["conv"]),
              "eps": float(cfg.norm["eps"])}
    names = {"q_proj": "q", "k_proj": "k", "v_proj": "v", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv",
             "b_proj": "b", "a_proj": "a", "A_log": "A_log", "dt_bias": "dt_bias", "o_norm": "norm", "g_proj": "g",
             "o_proj": "o"}
    return PartSpec("head_delta", params, {role: p + name for role, name in names.items()})


def build_spec(cfg: MepolixConfig) -> ModelSpec:
    W, eps = cfg.width, float(cfg.norm["eps"])
    norm = lambda name: PartSpec("layer_norm", {"size": W, "eps": eps}, {"weight": name})
    positions, blocks, ignorable, block_of = {}, [], [], {}
    for i, layer in enumerate(cfg.layers):
        if cfg.owner(i) != i:
            continue
        p = f"l{i}."
        mixer = _parallel(cfg, i, layer["mixer"], positions) if layer["type"] == "parallel" else _delta(cfg, i, layer["mixer"])
        parts = {"mixer": ("mixer", mixer), "mixer_post_norm": ("norm", norm(p + "norm1"))}
        if layer.get("mlp") is not None:
            parts["feed_forward"] = ("feed_forward", PartSpec(
                "swiglu", {"hidden_size": W, "intermediate_size": int(layer["mlp"]["ff"])},
                {"gate_proj": p + "mlp.gate", "up_proj": p + "mlp.up", "down_proj": p + "mlp.down"}))
            parts["feed_forward_post_norm"] = ("norm", norm(p + "norm2"))
        else:
            ignorable.append(p + "norm2")                 # a layer without feed-forward has no use for a second norm
        block_of[i] = len(blocks)
        blocks.append(BlockSpec(parts, "post_norm"))
    # every layer has cache layers of its own, also one that uses another's tensors: the attention's pages and the
    # recurrence's state, or the delta rule's state
    schedule, at = [], 0
    for i, layer in enumerate(cfg.layers):
        kept = 2 if layer["type"] == "parallel" else 1
        schedule.append(LayerCall(block=block_of[cfg.owner(i)], cache=at if kept == 1 else tuple(range(at, at + kept)),
                                  writes_cache=True))
        at += kept
    return ModelSpec(
        architecture=cfg.architecture, hidden_size=W, vocab_size=cfg.vocab, max_position=None,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": W}, {"weight": "embed"}),
        positions=positions, blocks=blocks, schedule=schedule, final_norm=norm("final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": W, "softcap": float(cfg.logit_softcap or 0.0)},
                      {"weight": "head"}),
        ignorable=ignorable)


register_architecture("Mepolix", MepolixConfig, build_spec)
