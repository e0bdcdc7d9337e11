"""Plain implementation of the Mapalorn design: whole sequences, no cache, 64-bit, one function per mechanism.

A decoder whose config.json lists its layers one by one. A layer has one layer norm (weight and bias), and both of its
sublayers read what it makes: x <- x + mixer(norm(x)) + ff(norm(x)), the feed-forward optional. The mixer is an attention
over a latent row per token (a rotated key part shared by all heads, a learned sink per head) or a grouped attention with
norms over the whole query and key rows, a term of one in the softmax's denominator and a gate on every element of its
output. The feed-forward is dense with clamped halves, or a mixture of experts that are fed the token times its score,
beside a gated expert that every token uses. A run of layers may be gone through several times. This file shares nothing
with the package; tests hold the engine against it.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


# ------------------------------------------------------------------ norms
def layer_norm(x, w, b, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ------------------------------------------------------------------ rotations
def angles(positions, base, dims):
    """(cos, sin) [T, 1, dims/2]: pair i turns by position * base^(-2i/dims)."""
    f = float(base) ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    a = positions.to(F64)[:, None] * f[None, :]
    return a.cos()[:, None, :], a.sin()[:, None, :]


def rotate_neighbours(x, positions, base, dims):
    """x [T, heads, D]: elements 2i and 2i + 1 of the first dims turn together, the rest pass."""
    cos, sin = angles(positions, base, dims)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def rotate_halves(x, positions, base, dims):
    """x [T, heads, D]: elements i and i + dims/2 of the first dims turn together, the rest pass."""
    cos, sin = angles(positions, base, dims)
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


# ------------------------------------------------------------------ attention
def causal_weights(s, extra):
    """s [H, T, S] scores (the queries are the last T of the S positions), extra [H]: weights exp(s) over the keys up to
    the query's own, divided by their sum plus exp(extra)."""
    H, T, S = s.shape
    i, j = torch.arange(S - T, S)[:, None], torch.arange(S)[None, :]
    s = s.masked_fill(j > i, -math.inf)
    e = extra[:, None, None]
    top = torch.maximum(s.max(-1, keepdim=True).values, e)
    p = torch.exp(s - top)
    return p / (p.sum(-1, keepdim=True) + torch.exp(e - top))


def latent_attention(h, w, m, eps):
    T = h.shape[0]
    H, D, R, V, C = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos, rot = torch.arange(T), m["rot"]
    turn = lambda x: rotate_neighbours(x, pos, rot["base"], int(rot["dims"]))
    q = (h @ w["q"].T).view(T, H, D + R)
    qr = turn(q[..., D:])
    z = h @ w["dkv"].T
    c = rms_norm(z[:, :C], w["dkv.norm"], eps)
    kr = turn(z[:, None, C:])[:, 0]
    k = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, V)
    s = torch.einsum("thd,shd->hts", q[..., :D], k) + torch.einsum("thr,sr->hts", qr, kr)
    p = causal_weights(s * float(m["scale"]), w["sink"])
    return torch.einsum("hts,shv->thv", p, v).reshape(T, H * V) @ w["o"].T


def gated_attention(h, w, m, eps):
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    V = int(m.get("vdim") or D)
    pos, rot = torch.arange(T), m.get("rot")
    turn = lambda x: rotate_halves(x, pos, rot["base"], int(rot["dims"])) if rot else x
    q = turn(rms_norm(h @ w["q"].T, w["q.norm"], eps).view(T, H, D))
    k = turn(rms_norm(h @ w["k"].T, w["k.norm"], eps).view(T, G, D)).repeat_interleave(H // G, dim=1)
    v = (h @ w["v"].T).view(T, G, V).repeat_interleave(H // G, dim=1)
    p = causal_weights(torch.einsum("thd,shd->hts", q, k) * float(m["scale"]), torch.zeros(H, dtype=F64))
    o = torch.einsum("hts,shv->thv", p, v).reshape(T, H * V)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------ feed-forward
def clamped_ff(h, w, limit):
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def expert(x, gate, up, down):
    z = x @ gate.T
    return (z * torch.sigmoid(z) * (x @ up.T)) @ down.T


def route(h, w_router, top):
    """(expert numbers [T, top], their scores): the largest sigmoids of the logits, as they are."""
    s = torch.sigmoid(h @ w_router.T)
    ids = s.topk(top, dim=-1).indices
    return ids, s.gather(1, ids)


def experts_ff(h, w, mlp):
    ids, scores = route(h, w["router"], int(mlp["router"]["top"]))
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t].tolist(), scores[t]):
            y[t] += expert(s * h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
    if mlp.get("shared") is not None:
        y = y + torch.sigmoid(h @ w["shared.sg"].T) * expert(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return y


# ------------------------------------------------------------------ the model
def sub(weights, prefix):
    """The tensors whose names begin with prefix, by the rest of their names, in 64-bit."""
    return {k[len(prefix):]: v.to(F64) for k, v in weights.items() if k.startswith(prefix)}


def run_order(cfg):
    """The layers' numbers in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = int(loop["start"]), int(loop["stop"])
    return list(range(a)) + list(range(a, b)) * int(loop["times"]) + list(range(b, n))


def forward(cfg, weights, tokens, streams=None):
    """Logits [T, vocab] of one whole sequence. streams: a list that receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x = weights["embed"].to(F64)[torch.as_tensor(tokens, dtype=torch.long)]
    for i in run_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        h = layer_norm(x, weights[p + "norm1"].to(F64), weights[p + "norm1.b"].to(F64), eps)
        mixer = latent_attention if layer["type"] == "latent_attention" else gated_attention
        y = mixer(h, sub(weights, p + "mix."), layer["mixer"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            w = sub(weights, p + "mlp.")
            y = y + (clamped_ff(h, w, float(mlp["limit"])) if mlp["kind"] == "dense" else experts_ff(h, w, mlp))
        x = x + y
        if streams is not None:
            streams.append(x.clone())
    x = layer_norm(x, weights["final.norm"].to(F64), weights["final.norm.b"].to(F64), eps)
    return x @ weights["head"].to(F64).T


def read_folder(folder):
    """(config.json as a dictionary, name -> tensor in 64-bit) of a model folder."""
    import json
    import os
    from safetensors import safe_open
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name).to(F64)
    return cfg, w


def logits(config, tensors, tokens):
    return forward(config, tensors, tokens)


def greedy(config, tensors, prompt, n_new):
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(logits(config, tensors, toks)[-1].argmax()))
    return toks[len(prompt):]
