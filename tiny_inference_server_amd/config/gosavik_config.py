"""Configuration of the Gosavik decoder, read from its config.json.

Keys: `vocab`, `width`, `norm.eps`, `streams` (copies of the residual stream), optionally `loop` ({"start", "stop",
"times"}: layers start .. stop-1 run `times` times in a row; absent or null: every layer once) and `layers`, a list with
one entry per layer: `type`, `mixer` and `mlp` ({"kind": "dense", "ff": n} or null for a layer without a feed-forward).

A "latent_attention" mixer gives `heads`, `dim`, `rot_dim`, `vdim`, `kv_rank`, `q_rank`, `scale`, and optionally `mask`
({"size": n}; absent: all earlier keys) and `rot` ({"dims", "base", "scaling": {"factor", "original", "fast", "slow"}};
absent or dims 0: no rotation; no scaling: plain frequencies). An "attention" mixer gives `heads`, `kv_heads`, `dim`,
`vdim`, `conv` (taps), `scale` and `rot` ({"dims", "base"}, optionally "scaling"; the base also turns the values).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, Mapping, Optional, Tuple

from .fikevik_config import _need, _number

MIXER_TYPES = ("latent_attention", "attention")
MLP_KINDS = ("dense",)


def _check_rot(rot, where, most):
    dims = _number(rot, "dims", where, int, 0)
    _need(dims % 2 == 0 and dims <= most, f"{where}.dims {dims}: an even number, at most {most}")
    if dims or "base" in rot:
        _need(_number(rot, "base", where, float) > 0, f"{where}.base must be positive")
    sc = rot.get("scaling")
    if sc is not None and dims:
        w = where + ".scaling"
        values = {k: _number(sc, k, w, float) for k in ("factor", "original", "fast", "slow")}
        _need(all(v > 0 for v in values.values()), f"{w}: factor, original, fast and slow must be positive")
        _need(float(rot["base"]) != 1.0, f"{where}.base 1 has no wavelengths to slow")


def _check_mixer(kind, m, where):
    _need(isinstance(m, Mapping), f"{where} must be an object")
    sizes = ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank") if kind == "latent_attention" else \
        ("heads", "kv_heads", "dim", "vdim", "conv")
    for k in sizes:
        _number(m, k, where, int, 1)
    _number(m, "scale", where, float)
    if m.get("mask") is not None:
        _number(m["mask"], "size", where + ".mask", int, 1)
    if kind == "latent_attention":
        if m.get("rot") is not None:
            _check_rot(m["rot"], where + ".rot", m["rot_dim"])
        return
    _need(m["heads"] % m["kv_heads"] == 0, f"{where}: {m['heads']} heads over {m['kv_heads']} kv_heads")
    _need(isinstance(m.get("rot"), Mapping) and "base" in m["rot"], f"config.json lacks {where}.rot.base")
    _check_rot(m["rot"], where + ".rot", m["dim"])
    _need(m["vdim"] % 2 == 0, f"{where}.vdim {m['vdim']}: values are turned in pairs of channels")


def _check_layer(i, entry):
    where = f"layers[{i}]"
    _need(isinstance(entry, Mapping), f"{where} must be an object")
    _need(entry.get("type") in MIXER_TYPES, f"{where}.type {entry.get('type')!r}: known are {', '.join(MIXER_TYPES)}")
    _check_mixer(entry["type"], entry.get("mixer"), where + ".mixer")
    mlp = entry.get("mlp")
    if mlp is None:
        return
    _need(isinstance(mlp, Mapping) and mlp.get("kind") in MLP_KINDS,
          f"{where}.mlp.kind {mlp.get('kind') if isinstance(mlp, Mapping) else mlp!r}: known are {', '.join(MLP_KINDS)}")
    _number(mlp, "ff", where + ".mlp", int, 1)


@dataclass(frozen=True)
class GosavikConfig:
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[Dict[str, Any], ...]
    loop: Optional[Tuple[int, int, int]] = None        # (start, stop, times)
    architecture: str = "Gosavik"
    extra: Dict[str, Any] = field(default_factory=dict, compare=False)

    def __post_init__(self):
        _need(self.vocab >= 1 and self.width >= 1, f"vocab {self.vocab} and width {self.width} must be at least 1")
        _need(self.streams >= 1, f"streams must be at least 1, got {self.streams}")
        _need(self.norm_eps >= 0, f"norm.eps must not be negative, got {self.norm_eps}")
        _need(len(self.layers) >= 1, "layers must not be empty")
        for i, entry in enumerate(self.layers):
            _check_layer(i, entry)
        if self.loop is not None:
            start, stop, times = self.loop
            _need(0 <= start < stop <= len(self.layers), f"loop: layers {start} .. {stop} - 1 of {len(self.layers)}")
            _need(times >= 1, f"loop.times must be at least 1, got {times}")

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "GosavikConfig":
        _need(isinstance(raw.get("layers"), list), "config.json lacks 'layers' (a list)")
        used = {"architecture", "vocab", "width", "streams", "norm", "layers", "loop"}
        loop = raw.get("loop")
        return cls(vocab=_number(raw, "vocab", "config", int, 1), width=_number(raw, "width", "config", int, 1),
                   streams=_number(raw, "streams", "config", int, 1), norm_eps=_number(raw.get("norm"), "eps", "norm", float),
                   layers=tuple(copy.deepcopy(dict(e)) if isinstance(e, Mapping) else e for e in raw["layers"]),
                   loop=tuple(_number(loop, k, "loop", int, 0) for k in ("start", "stop", "times")) if loop is not None else None,
                   architecture=str(raw.get("architecture", "Gosavik")),
                   extra={k: v for k, v in raw.items() if k not in used})

    def run_order(self) -> Tuple[int, ...]:
        """The layers' indices in the order they run."""
        n = len(self.layers)
        if self.loop is None:
            return tuple(range(n))
        start, stop, times = self.loop
        return tuple(range(start)) + tuple(range(start, stop)) * times + tuple(range(stop, n))

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
               "norm": {"eps": self.norm_eps}, "layers": copy.deepcopy(list(self.layers))}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return out
