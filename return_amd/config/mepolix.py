"""Configuration of the Mepolix decoder, read from its config.json keys.

The file names the design under "architecture" and describes every layer by itself:

    vocab, width                      sizes of the embedding and of the residual stream
    norm.eps                          epsilon of every norm
    logit_softcap                     c: the logits leave as c tanh(logits / c) (none: as they are)
    layers[i].type                    "parallel" or "delta": the layer's mixer
    layers[i].mixer                   parallel: left {heads, kv_heads, dim (a head's query and key), vdim (a head's
                                      value; dim unless given), scale, rot {base, dims, scaling {factor, original, fast,
                                      slow}} (scaling optional; no rot: no rotation)}, right {width, blocks, conv (taps)},
                                      left_scale, right_scale (1 unless given)
                                      delta: heads, kv_heads, dim, vdim, conv (taps)
    layers[i].mlp                     {"kind": "dense", "ff": size}, or null for a layer without feed-forward
    layers[i].weights_of              j: the layer has no tensors of its own and uses layer j's; it keeps a cache or
                                      state of its own, and the rest of its entry is layer j's
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, List, Optional

from .base import ConfigError, ModelConfig

MIXERS = ("parallel", "delta")


def _int(where: str, d: dict, key: str, least: int = 1) -> int:
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or float(v) != int(v) or int(v) < least:
        raise ConfigError(f"Mepolix: {where}.{key} must be an integer of at least {least}, got {v!r}")
    return int(v)


def _float(where: str, d: dict, key: str, positive: bool = False) -> float:
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or (positive and not v > 0):
        raise ConfigError(f"Mepolix: {where}.{key} must be a {'positive ' if positive else ''}number, got {v!r}")
    return float(v)


def _heads(where: str, m: dict) -> None:
    heads, kv = _int(where, m, "heads"), _int(where, m, "kv_heads")
    if heads % kv:
        raise ConfigError(f"Mepolix: {where}: {heads} heads are not a multiple of {kv} kv_heads")
    _int(where, m, "dim")


@dataclasses.dataclass(frozen=True)
class MepolixConfig(ModelConfig):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, Any]
    logit_softcap: Optional[float] = None

    def validate(self, raw):
        if self.vocab < 1 or self.width < 1:
            raise ConfigError(f"Mepolix: vocab {self.vocab} and width {self.width} must be positive")
        _float("norm", self.norm, "eps")
        if self.logit_softcap is not None and not (isinstance(self.logit_softcap, (int, float)) and self.logit_softcap >= 0):
            raise ConfigError(f"Mepolix: logit_softcap {self.logit_softcap!r} must be a number that is not negative")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("Mepolix: layers must be a list with at least one layer")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXERS:
                raise ConfigError(f"Mepolix: {where}.type must be one of {MIXERS}, got "
                                  f"{layer.get('type') if isinstance(layer, dict) else layer!r}")
            m = layer.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"Mepolix: {where}.mixer must be a dictionary")
            if layer["type"] == "parallel":
                self._check_parallel(where + ".mixer", m)
            else:
                _heads(where + ".mixer", m)
                _int(where + ".mixer", m, "vdim")
                _int(where + ".mixer", m, "conv")
            mlp = layer.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
                    raise ConfigError(f"Mepolix: {where}.mlp.kind must be 'dense' (or mlp null), got {mlp!r}")
                _int(where + ".mlp", mlp, "ff")
        for i, layer in enumerate(self.layers):
            if layer.get("weights_of") is None:
                continue
            where = f"layers[{i}]"
            j = _int(where, layer, "weights_of", 0)
            if j >= len(self.layers) or j == i:
                raise ConfigError(f"Mepolix: {where}.weights_of {j} is not another of the {len(self.layers)} layers")
            rest = lambda entry: {k: v for k, v in entry.items() if k != "weights_of"}
            if rest(layer) != rest(self.layers[j]):
                raise ConfigError(f"Mepolix: {where} uses the tensors of layers[{j}] but describes another layer")
            self.owner(i)

    @staticmethod
    def _check_parallel(where, m):
        left, right = m.get("left"), m.get("right")
        if not isinstance(left, dict) or not isinstance(right, dict):
            raise ConfigError(f"Mepolix: {where} must describe a left and a right mixer")
        _heads(where + ".left", left)
        if left.get("vdim") is not None:
            _int(where + ".left", left, "vdim")
        _float(where + ".left", left, "scale")
        rot = left.get("rot")
        if rot is not None:
            dims = _int(where + ".left.rot", rot, "dims", 2)
            if dims % 2 or dims > int(left["dim"]) or _float(where + ".left.rot", rot, "base", True) == 1.0:
                raise ConfigError(f"Mepolix: {where}.left.rot: dims {dims} must be even and at most dim {left['dim']}, "
                                  "base not 1")
            if rot.get("scaling") is not None:
                for key in ("factor", "original", "fast", "slow"):
                    _float(where + ".left.rot.scaling", rot["scaling"], key, True)
        width, blocks = _int(where + ".right", right, "width"), _int(where + ".right", right, "blocks")
        if width % blocks:
            raise ConfigError(f"Mepolix: {where}.right: width {width} is not a multiple of {blocks} blocks")
        _int(where + ".right", right, "conv")
        for key in ("left_scale", "right_scale"):
            if m.get(key) is not None:
                _float(where, m, key)

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses (itself, unless it names another)."""
        seen = set()
        while self.layers[i].get("weights_of") is not None:
            if i in seen:
                raise ConfigError(f"Mepolix: layers {sorted(seen)} use each other's tensors and none has its own")
            seen.add(i)
            i = int(self.layers[i]["weights_of"])
        return i

    def to_dict(self):
        out = {"architecture": self.architecture}
        for f in dataclasses.fields(self):
            if f.name != "architecture" and getattr(self, f.name) is not None:
                out[f.name] = getattr(self, f.name)
        return out
