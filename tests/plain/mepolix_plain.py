"""Plain implementation of the Mepolix design: whole sequences, no cache, 64-bit, one function per mechanism.

A decoder whose config.json lists its layers one by one. A sublayer reads the stream as it is and enters it through a
layer norm (with a weight, without a bias) of its output:
    x <- x + norm1(mixer(x));   x <- x + norm2(ff(x))      (the feed-forward optional).
The mixer is a gated delta rule with one decay per head, or two mixers side by side on the same input: a grouped
attention (norms on queries and keys, stretched rotation, a learned sink per head) and a gated linear recurrence per
channel behind a short filter. A layer may use another layer's tensors; its memory is its own. The logits pass a soft
cap. This file shares nothing with the package; tests hold the engine against it.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


# ------------------------------------------------------------------ small things
def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def causal_filter(x, taps, bias=None, tail=None):
    """x [T, C], taps [C, K] (the last column is the current row's), zeros or `tail` [K - 1, C] before the start.
    Returns (filtered rows, the last K - 1 inputs)."""
    K = taps.shape[1]
    before = torch.zeros(K - 1, x.shape[1], dtype=x.dtype) if tail is None else tail
    xx = torch.cat([before, x], dim=0)
    y = sum(xx[i:i + x.shape[0]] * taps[:, i][None, :] for i in range(K))
    if bias is not None:
        y = y + bias
    return y, xx[xx.shape[0] - (K - 1):]


# ------------------------------------------------------------------ rotation
def stretched_frequencies(rot):
    """(frequency of every pair, factor on cos and sin) of a rotation over rot.dims elements, stretched for long
    contexts when rot.scaling is there."""
    n, base = int(rot["dims"]), float(rot["base"])
    i = torch.arange(n // 2, dtype=F64)
    f = base ** (-2.0 * i / n)
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    place = lambda turns: n * math.log(float(s["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(place(float(s["fast"]))), 0)
    hi = min(math.ceil(place(float(s["slow"]))), n - 1)
    ramp = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    factor = float(s["factor"])
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, rot):
    """x [T, heads, D]: the first rot.dims elements of every head turn, element i with i + dims/2."""
    if not rot:
        return x
    n = int(rot["dims"])
    f, m = stretched_frequencies(rot)
    a = positions.to(F64)[:, None] * f[None, :]
    cos, sin = (a.cos() * m)[:, None, :], (a.sin() * m)[:, None, :]
    u, v = x[..., :n // 2], x[..., n // 2:n]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., n:]], dim=-1)


# ------------------------------------------------------------------ attention with a learned sink
def sink_softmax(s, sink):
    """s [H, T, S] (masked with -inf) -> weights whose denominator also holds exp(sink) of the head."""
    m = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def sink_attention_heads(h, w, m, eps, positions=None):
    """The heads' results side by side, [T, H * vdim], before the output projection."""
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    Dv = int(m.get("vdim") or D)
    pos = torch.arange(T) if positions is None else positions
    q = rms((h @ w["q"].T).view(T, H, D), eps) * w["q.norm"]
    k = rms((h @ w["k"].T).view(T, G, D), eps) * w["k.norm"]
    v = (h @ w["v"].T).view(T, G, Dv)
    q, k = rotate_half(q, pos, m.get("rot")), rotate_half(k, pos, m.get("rot"))
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    s = torch.einsum("thd,shd->hts", q, k) * float(m["scale"])
    s = s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], -math.inf)
    return torch.einsum("hts,shd->thd", sink_softmax(s, w["sink"]), v).reshape(T, H * Dv)


def sink_attention(h, w, m, eps, positions=None):
    return sink_attention_heads(h, w, m, eps, positions) @ w["o"].T


# ------------------------------------------------------------------ gated linear recurrence per channel
def block_gates(u, w, blocks):
    """(r, i) [T, width] each: sigmoid of a matrix per block of neighbouring channels."""
    T = u.shape[0]
    ub = u.view(T, blocks, -1)
    gate = lambda n: torch.sigmoid(torch.einsum("tbc,bdc->tbd", ub, w[n]) + w[n + ".b"][None]).reshape(T, -1)
    return gate("ra"), gate("ri")


def channel_recurrence(u, r, i, lam, state=None):
    """S_t = a S_(t-1) + sqrt(1 - a^2) i u with log a = -8 r softplus(lam). Returns (all S [T, width], the last)."""
    log_a = -8.0 * r * softplus(lam)
    a = torch.exp(log_a)
    x = torch.sqrt(1.0 - a * a) * i * u
    S = torch.zeros(u.shape[1], dtype=F64) if state is None else state.clone()
    out = torch.empty_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + x[t]
        out[t] = S
    return out, S


def gated_recurrence(h, w, m, state=None, tail=None):
    """Returns (y [T, W], the state, the filter's last inputs)."""
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u, tail = causal_filter(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"], tail)
    r, i = block_gates(u, w, int(m["blocks"]))
    S, last = channel_recurrence(u, r, i, w["lam"], state)
    return (S * y) @ w["o"].T, last, tail


def parallel(h, w, m, eps):
    left = sink_attention(h, sub(w, "left."), m["left"], eps)
    right, _, _ = gated_recurrence(h, sub(w, "right."), m["right"])
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


# ------------------------------------------------------------------ gated delta rule, one decay per head
def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, g, state=None):
    """q, k [T, H, D], v [T, H, V], beta, g [T, H] -> (o [T, H, V], S [H, D, V]); the read-out sees the write."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64) if state is None else state.clone()
    o = torch.empty_like(v)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return o, S


def delta(h, w, m, eps, state=None, tails=None):
    """Returns (y [T, W], the state, the three filters' last inputs by name)."""
    T = h.shape[0]
    H, G, D, V = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    x, last = {}, {}
    for n in "qkv":
        y, last[n] = causal_filter(h @ w[n].T, w[n + ".conv"], None, None if tails is None else tails[n])
        x[n] = silu(y)
    q = unit(x["q"].view(T, G, D)).repeat_interleave(H // G, dim=1) * D ** -0.5
    k = unit(x["k"].view(T, G, D)).repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"])[None] * softplus(h @ w["a"].T + w["dt_bias"]))
    o, S = delta_rule(q, k, x["v"].view(T, H, V), beta, g, state)
    o = rms(o, eps) * w["norm"] * silu(h @ w["g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w["o"].T, S, last


# ------------------------------------------------------------------ feed-forward
def dense(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


# ------------------------------------------------------------------ the model
def sub(weights, prefix):
    """The tensors whose names begin with prefix, by the rest of their names, in 64-bit."""
    return {k[len(prefix):]: v.to(F64) for k, v in weights.items() if k.startswith(prefix)}


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
    return i


def forward(cfg, weights, tokens, streams=None):
    """Logits [T, vocab] of one whole sequence. streams: a list that receives the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = weights["embed"].to(F64)[torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."
        w = sub(weights, p + "mix.")
        if layer["type"] == "parallel":
            y = parallel(x, w, layer["mixer"], eps)
        else:
            y, _, _ = delta(x, w, layer["mixer"], eps)
        x = x + layer_norm(y, weights[p + "norm1"].to(F64), eps)
        if layer.get("mlp") is not None:
            x = x + layer_norm(dense(x, sub(weights, p + "mlp.")), weights[p + "norm2"].to(F64), eps)
        if streams is not None:
            streams.append(x.clone())
    x = layer_norm(x, weights["final.norm"].to(F64), eps)
    z = x @ weights["head"].to(F64).T
    c = float(cfg.get("logit_softcap") or 0.0)
    return c * torch.tanh(z / c) if c else z


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
