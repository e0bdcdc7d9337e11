"""Several mixers side by side on the same input: the result is the sum of theirs, each times a factor.

    y = sum_s scale_s * mixer_s(x)

A side is a mixer part whose input goes into one product and whose output comes out of one, and which can be told to
leave both to its owner (its params get inner = True): take_products() gives its two weights up, in_width / out_width
are their outer sizes, and run(z, step, cache, write_cache, out, out_scale) does what lies between them, on columns of
wider rows. Then the sides share ONE first product (their weights stacked) and ONE last product (their output
projections next to each other along the inner size: the sum of the sides' results is formed in the product's 32-bit
sums). A side multiplies its rows by its factor in 32-bit, before it rounds them.
Parameters: hidden_size, sides: list of {"name", "kind", "params", "scale"}. Roles: the sides' own, behind "<name>.".
What the mixer keeps between steps is what its sides keep, in their order.
"""
from __future__ import annotations

import torch

from .registry import part_class, register_part


def _inner(side):
    return dict(side["params"], inner=True)


class SideBySideMixer:
    @staticmethod
    def tensor_shapes(params):
        return {f"{s['name']}.{role}": shape for s in params["sides"]
                for role, shape in part_class("mixer", s["kind"]).tensor_shapes(_inner(s)).items()}

    @staticmethod
    def random_init(params, role):
        name, own = role.split(".", 1)
        side = next(s for s in params["sides"] if s["name"] == name)
        cls = part_class("mixer", side["kind"])
        return cls.random_init(_inner(side), own) if hasattr(cls, "random_init") else "matrix"

    def __init__(self, params, tensors, rt, shared=None):
        self.rt = rt
        self.sides, self.scales = [], []
        firsts, lasts = [], []
        for s in params["sides"]:
            own = {role.split(".", 1)[1]: t for role, t in tensors.items() if role.split(".", 1)[0] == s["name"]}
            cls = part_class("mixer", s["kind"])
            if not hasattr(cls, "take_products"):
                raise ValueError(f"mixer {s['kind']!r} cannot be one side of several: it does not give up its products")
            side = cls(_inner(s), own, rt, shared)
            self.sides.append(side)
            self.scales.append(float(s.get("scale", 1.0)))
            first, last = side.take_products()
            # (slices of the shared rows begin at multiples of 16)
            pad_in, pad_out = -first.shape[0] % 16, -last.shape[1] % 16
            if pad_in:
                first = torch.cat([first, first.new_zeros(pad_in, first.shape[1])], dim=0)
            if pad_out:
                last = torch.cat([last, last.new_zeros(last.shape[0], pad_out)], dim=1)
            firsts.append(first)
            lasts.append(last)
        self.at_in = [sum(f.shape[0] for f in firsts[:i]) for i in range(len(firsts))]
        self.at_out = [sum(w.shape[1] for w in lasts[:i]) for i in range(len(lasts))]
        self.out_pads = [w.shape[1] - side.out_width for w, side in zip(lasts, self.sides)]
        self.inner_width = sum(w.shape[1] for w in lasts)
        self.w_in = rt.product(torch.cat(firsts, dim=0).contiguous())
        self.w_o = rt.product(torch.cat(lasts, dim=1).contiguous())
        self._specs = []
        for side in self.sides:
            spec = side.cache_spec()
            self._specs.append(() if spec is None else tuple(spec) if isinstance(spec, (tuple, list)) else (spec,))

    def cache_spec(self):
        specs = sum(self._specs, ())
        return None if not specs else specs[0] if len(specs) == 1 else specs

    def step_needs(self):
        tile_rows, columns = set(), set()
        for side in self.sides:
            needs = side.step_needs() if hasattr(side, "step_needs") else {}
            tile_rows.update(needs.get("prefill_tile_rows", ()))
            columns.update(needs.get("token_columns", ()))
        out = {}
        if tile_rows:
            out["prefill_tile_rows"] = tile_rows
        if columns:
            out["token_columns"] = tuple(sorted(columns))
        return out

    def forward(self, x, step, cache, write_cache=True):
        ops = self.rt.ops
        views = () if cache is None else tuple(cache) if isinstance(cache, (tuple, list)) else (cache,)
        z = ops.linear(x, self.w_in)
        o = self.rt.empty(x.shape[0], self.inner_width)
        at = 0
        for side, scale, spec, a, b, pad in zip(self.sides, self.scales, self._specs, self.at_in, self.at_out, self.out_pads):
            mine = views[at:at + len(spec)]
            at += len(spec)
            if pad:                                          # columns that the side does not write meet zero weights
                o[:, b + side.out_width:b + side.out_width + pad].zero_()
            side.run(z[:, a:a + side.in_width], step, mine[0] if len(mine) == 1 else mine or None, write_cache,
                     o[:, b:b + side.out_width], scale)
        return ops.linear(o, self.w_o)


register_part("mixer", "side_by_side", SideBySideMixer)
