"""Configuration of the Zakusun decoder: a list of layers, each attention through a cached latent and an optional feed-forward of
routed experts; grouped RMS norms before the sublayers, each followed by a short convolution over time; a weighted sum of
all layers so far behind every layer; sinusoidal positions added to the embedding, whose table is also the head, with
scaled logits.

``config.json`` is nested, and this class keeps it as it is read (``layers`` as a tuple of mappings), checked key by key
here so that the builder can rely on it:

  architecture, vocab, width, norm {eps, groups}, canon {taps} (absent: no convolution), logit_scale,
  layers[i] {type "latent_attention", mixer {heads, dim, vdim, kv_rank, scale}, mlp {...} or null}
    mlp:  kind "moe", expert {ff, limit}, router {experts, top}
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Tuple

from .base import ConfigError, ModelConfig
from .dekinex import _obj
from .sagalorn import _int, _num, _plain

MIXERS = ("latent_attention",)


def _check_mlp(where: str, mlp: Any):
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
        raise ConfigError(f"{where} must be null or an object of kind 'moe', got {mlp!r}")
    expert, router = _obj(where, mlp, "expert", True), _obj(where, mlp, "router", True)
    out = {"kind": "moe", "expert": {"ff": _int(f"{where}.expert", expert, "ff"), "limit": _num(f"{where}.expert", expert, "limit")},
           "router": {"experts": _int(f"{where}.router", router, "experts"), "top": _int(f"{where}.router", router, "top")}}
    if not out["expert"]["limit"] > 0:
        raise ConfigError(f"{where}.expert: 'limit' must be positive")
    if out["router"]["top"] > out["router"]["experts"]:
        raise ConfigError(f"{where}.router: 'top' ({out['router']['top']}) is above 'experts' ({out['router']['experts']})")
    return out


def _check_layer(i: int, layer: Any) -> Dict[str, Any]:
    where = f"layers[{i}]"
    if not isinstance(layer, dict) or layer.get("type") not in MIXERS or not isinstance(layer.get("mixer"), dict):
        raise ConfigError(f"{where} must have the 'type' {' or '.join(MIXERS)} and a 'mixer' object")
    m, mw = layer["mixer"], f"{where}.mixer"
    out: Dict[str, Any] = {k: _int(mw, m, k) for k in ("heads", "dim", "kv_rank")}
    out["vdim"] = _int(mw, m, "vdim", out["dim"])
    out["scale"] = _num(mw, m, "scale", 1.0 / math.sqrt(out["dim"]))
    return {"type": layer["type"], "mixer": out, "mlp": _check_mlp(f"{where}.mlp", layer.get("mlp"))}


@dataclass(frozen=True)
class ZakusunConfig(ModelConfig):
    architecture = "Zakusun"

    vocab: int
    width: int
    layers: Tuple[Dict[str, Any], ...]
    norm_eps: float
    norm_groups: int = 1
    canon_taps: int = 0
    logit_scale: float = 1.0

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "ZakusunConfig":
        where = "config.json of Zakusun"
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where} lacks a non-empty list 'layers'")
        norm = _obj(where, raw, "norm", True)
        eps, groups, width = _num("norm", norm, "eps"), _int("norm", norm, "groups", 1), _int(where, raw, "width")
        if not eps > 0:
            raise ConfigError("norm: 'eps' must be positive")
        if width % groups:
            raise ConfigError(f"norm: 'groups' ({groups}) must divide the width ({width})")
        canon = _obj(where, raw, "canon")
        return cls(vocab=_int(where, raw, "vocab"), width=width, layers=tuple(_check_layer(i, l) for i, l in enumerate(layers)),
                   norm_eps=eps, norm_groups=groups, canon_taps=_int("canon", canon, "taps") if canon is not None else 0,
                   logit_scale=_num(where, raw, "logit_scale", 1.0))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps, "groups": self.norm_groups}, "logit_scale": self.logit_scale,
                               "layers": [_plain(dict(l)) for l in self.layers]}
        if self.canon_taps:
            out["canon"] = {"taps": self.canon_taps}
        return out
