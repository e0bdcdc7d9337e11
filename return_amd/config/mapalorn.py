"""Configuration of the Mapalorn decoder, read from its config.json keys.

The file names the design under "architecture" and describes every layer by itself:

    vocab, width                      sizes of the embedding and of the residual stream
    norm.eps                          epsilon of every norm
    layers[i].type                    "latent_attention" or "attention": the layer's mixer
    layers[i].mixer                   latent_attention: heads, dim (a head's query and key elements that do not turn), rot_dim
                                      (those that do), vdim (a head's value), kv_rank (the latent), scale, rot {base, dims}
                                      attention: heads, kv_heads, dim (a head's query and key), vdim (a head's value; dim
                                      unless given), scale, rot {base, dims} (no rot: no rotation)
    layers[i].mlp                     {"kind": "dense", "ff", "limit"}; {"kind": "moe", "expert": {"ff"}, "router": {"experts",
                                      "top"}, "shared": {"ff"} (optional)}; or null for a layer without feed-forward
    loop                              {"start", "stop", "times"}: layers start .. stop-1 run `times` times in a row (as a
                                      group, with the same weights, every pass with a cache of its own) before the rest
                                      (none: every layer runs once)
"""
from __future__ import annotations

import dataclasses
from typing import Any, Dict, List, Optional

from .base import ConfigError, ModelConfig

MIXERS = ("latent_attention", "attention")


def _int(where: str, d: dict, key: str, least: int = 1) -> int:
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or float(v) != int(v) or int(v) < least:
        raise ConfigError(f"Mapalorn: {where}.{key} must be an integer of at least {least}, got {v!r}")
    return int(v)


def _float(where: str, d: dict, key: str, positive: bool = False) -> float:
    v = d.get(key) if isinstance(d, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or (positive and not v > 0):
        raise ConfigError(f"Mapalorn: {where}.{key} must be a {'positive ' if positive else ''}number, got {v!r}")
    return float(v)


def _rotation(where: str, rot: Any, most: int, exactly: bool) -> None:
    dims = _int(where, rot, "dims", 2)
    _float(where, rot, "base", True)
    if dims % 2 or dims > most or (exactly and dims != most):
        raise ConfigError(f"Mapalorn: {where}.dims {dims} must be even and {'equal to' if exactly else 'at most'} {most}")


@dataclasses.dataclass(frozen=True)
class MapalornConfig(ModelConfig):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, Any]
    loop: Optional[Dict[str, Any]] = None

    def validate(self, raw):
        if self.vocab < 1 or self.width < 1:
            raise ConfigError(f"Mapalorn: vocab {self.vocab} and width {self.width} must be positive")
        _float("norm", self.norm, "eps")
        if not isinstance(self.layers, list) or not self.layers:
            raise ConfigError("Mapalorn: layers must be a list with at least one layer")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict) or layer.get("type") not in MIXERS:
                raise ConfigError(f"Mapalorn: {where}.type must be one of {MIXERS}, got "
                                  f"{layer.get('type') if isinstance(layer, dict) else layer!r}")
            m = layer.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"Mapalorn: {where}.mixer must be a dictionary")
            self._check_mixer(where + ".mixer", layer["type"], m)
            if layer.get("mlp") is not None:
                self._check_mlp(where + ".mlp", layer["mlp"])
        if self.loop is not None:
            a, b, _ = _int("loop", self.loop, "start", 0), _int("loop", self.loop, "stop"), _int("loop", self.loop, "times")
            if not a < b <= len(self.layers):
                raise ConfigError(f"Mapalorn: loop runs layers {a} to {b} of {len(self.layers)}")

    @staticmethod
    def _check_mixer(where, kind, m):
        heads = _int(where, m, "heads")
        _int(where, m, "dim")
        _float(where, m, "scale")
        if kind == "latent_attention":
            for key in ("vdim", "kv_rank"):
                _int(where, m, key)
            _rotation(where + ".rot", m.get("rot"), _int(where, m, "rot_dim", 2), True)
            return
        kv = _int(where, m, "kv_heads")
        if heads % kv:
            raise ConfigError(f"Mapalorn: {where}: {heads} heads are not a multiple of {kv} kv_heads")
        if m.get("vdim") is not None:
            _int(where, m, "vdim")
        if m.get("rot") is not None:
            _rotation(where + ".rot", m["rot"], int(m["dim"]), False)

    @staticmethod
    def _check_mlp(where, mlp):
        kind = mlp.get("kind") if isinstance(mlp, dict) else None
        if kind == "dense":
            _int(where, mlp, "ff")
            _float(where, mlp, "limit", True)
        elif kind == "moe":
            _int(where + ".expert", mlp.get("expert"), "ff")
            experts, top = _int(where + ".router", mlp.get("router"), "experts"), _int(where + ".router", mlp.get("router"), "top")
            if top > experts:
                raise ConfigError(f"Mapalorn: {where}.router: top {top} of {experts} experts")
            if mlp.get("shared") is not None:
                _int(where + ".shared", mlp["shared"], "ff")
        else:
            raise ConfigError(f"Mapalorn: {where}.kind must be 'dense' or 'moe' (or mlp null), got {mlp!r}")

    def run_order(self) -> List[int]:
        """The layers' numbers in the order they run."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        a, b = int(self.loop["start"]), int(self.loop["stop"])
        return list(range(a)) + list(range(a, b)) * int(self.loop["times"]) + list(range(b, n))

    def to_dict(self):
        out = {"architecture": self.architecture}
        for f in dataclasses.fields(self):
            if f.name != "architecture" and getattr(self, f.name) is not None:
                out[f.name] = getattr(self, f.name)
        return out
