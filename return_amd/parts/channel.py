"""A gated linear recurrence per channel behind a short filter: a mixer whose memory is one number per channel.

    y = gelu_tanh(W_y h + b_y),   u = filter(W_x h + b_x)         two branches of `width` channels; a causal filter per
                                                                  channel with a bias, zeros before the start, no activation
    r = sigmoid(R_b u_b + rb),    i = sigmoid(I_b u_b + ib)       a square matrix per block b of neighbouring channels
    log a = -8 r softplus(lam),   S <- exp(log a) S + sqrt(1 - a^2) i u,   out = W_o (S * y)
with S = 0 before a request's first token. The gates' logits, the decay, its square root and the state are 32-bit.
Kept between steps per request: the filter's last taps - 1 inputs and S. (De et al., "Griffin: Mixing Gated Linear
Recurrences with Local Attention for Efficient Language Models", call it a real-gated linear recurrent unit.)

One product in front, [W_y; W_x]; the filter reads its columns of the result (its kernel adds b_x to every input), the
gates of both kinds, the recurrence and the output branch are the recurrence's kernels.
Parameters: hidden_size, width, blocks, conv_taps, inner (see BlendAttention: the part as one side of a mixer of several).
"""
from __future__ import annotations

import torch

from ..cache.spec import StateSpec
from .conv import filter_init
from .registry import register_part

DECAY_RATE = -8.0           # log a = DECAY_RATE * r * softplus(lam)


def _lam_init(shape, generator):
    """So that exp(DECAY_RATE * softplus(lam)) lies in (0.9, 0.999)."""
    a = 0.9 + 0.099 * torch.rand(*shape, generator=generator, dtype=torch.float32, device=generator.device)
    return torch.log(torch.expm1(torch.log(a) / DECAY_RATE))


def _small_bias(shape, generator):
    return 0.1 * torch.randn(*shape, generator=generator, dtype=torch.float32, device=generator.device)


class GatedChannelRecurrence:
    @staticmethod
    def tensor_shapes(params):
        W, C, B = params["hidden_size"], params["width"], params["blocks"]
        bw = C // B
        return {"y_proj": (C, W), "y_bias": (C,), "x_proj": (C, W), "x_bias": (C,), "conv": (C, params["conv_taps"]),
                "conv_bias": (C,), "r_gate": (B, bw, bw), "r_bias": (B, bw), "i_gate": (B, bw, bw), "i_bias": (B, bw),
                "lam": (C,), "o_proj": (W, C)}

    @staticmethod
    def random_init(params, role):
        if role == "conv":
            return filter_init
        if role == "lam":
            return _lam_init
        return _small_bias if role.endswith("bias") else "matrix"

    def __init__(self, params, tensors, rt, shared=None):
        self.rt = rt
        self.hidden = W = int(params["hidden_size"])
        C, B = self.width, self.blocks = int(params["width"]), int(params["blocks"])
        self.taps = int(params["conv_taps"])
        if C % B:
            raise ValueError(f"{C} channels do not form {B} equal blocks")
        self.inner = bool(params.get("inner"))
        note = (lambda w: w) if self.inner else rt.product
        # both branches' rows, each filled up with zero rows to a multiple of 16 so that the slices begin aligned; the
        # output projection has as many zero columns
        self.padded = -(-C // 16) * 16

        def padded(name):
            m = torch.zeros(self.padded, W, dtype=rt.dtype, device=rt.device)
            m[:C] = rt.matrix(tensors[name])
            return m
        self.w_in = note(torch.cat([padded("y_proj"), padded("x_proj")], dim=0).contiguous())
        w_o = torch.zeros(W, self.padded, dtype=rt.dtype, device=rt.device)
        w_o[:, :C] = rt.matrix(tensors["o_proj"])
        self.w_o = note(w_o)
        self.in_width, self.out_width = 2 * self.padded, self.padded
        self.y_bias, self.x_bias = rt.vector32(tensors["y_bias"]), rt.vector32(tensors["x_bias"])
        self.w_conv, self.conv_bias = rt.vector32(tensors["conv"]), rt.vector32(tensors["conv_bias"])
        self.w_gates = torch.stack([rt.matrix(tensors["r_gate"]), rt.matrix(tensors["i_gate"])], dim=1).contiguous()
        self.gate_bias = torch.stack([rt.vector32(tensors["r_bias"]).reshape(C), rt.vector32(tensors["i_bias"]).reshape(C)]).contiguous()
        lam = tensors["lam"].double()
        self.rate = rt.vector32(DECAY_RATE * (lam.clamp(min=0.0) + torch.log1p(torch.exp(-lam.abs()))))   # softplus in 64-bit

    def take_products(self):
        """(first weight [in_width, W], output projection [W, out_width]), given up to the caller."""
        products, self.w_in, self.w_o = (self.w_in, self.w_o), None, None
        return products

    def cache_spec(self):
        return StateSpec((("conv", (self.taps - 1, self.width), self.rt.dtype_name), ("S", (self.width,), "float32")))

    def forward(self, x, step, cache, write_cache=True):
        ops = self.rt.ops
        out = self.rt.empty(x.shape[0], self.out_width)
        self.run(ops.linear(x, self.w_in), step, cache, write_cache, out)
        return ops.linear(out, self.w_o)

    def run(self, z, step, cache, write_cache, out, out_scale=1.0):
        """From the first product's rows (columns of wider rows are fine) to S * y times out_scale in out (columns of
        wider rows too; the columns beyond `width` become zeros)."""
        if not write_cache:
            raise ValueError("a recurrent mixer advances its state with every call; it cannot only read it")
        ops = self.rt.ops
        u = self.rt.empty(z.shape[0], self.width)
        ops.causal_conv(z[:, self.padded:self.padded + self.width], self.w_conv, cache.tensors["conv"], step, u,
                        bias=self.conv_bias, in_bias=self.x_bias)
        ops.channel_recurrence(u, self.w_gates, self.gate_bias, self.rate, z[:, :self.width], self.y_bias,
                               cache.tensors["S"], step, out, out_scale)


register_part("mixer", "gated_channel_recurrence", GatedChannelRecurrence)
