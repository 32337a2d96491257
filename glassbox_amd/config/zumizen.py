"""Configuration of the Zumizen decoder: a list of layers, each with one of two mixers (attention with a distance bias beside a gated
delta rule with a decay a head, or a gated delta rule with a decay a key channel) and an optional feed-forward of routed experts
whose weights multiply their input; RMS norms on the sublayers' outputs alone; a scaled embedding with a hashed table of token
pairs; bounded logits.

``config.json`` is nested, and this class keeps it as it is read (``layers`` as a tuple of mappings), checked key by
key here so that the builder can rely on it:

  architecture, vocab, width, norm {eps}, logit_softcap (absent: none),
  embedding {scale, bigram {buckets, mul_prev, mul_cur} (absent: the token's row alone)},
  layers[i] {type, mixer {...}, mlp {...} or null}
    parallel:      left {heads, kv_heads, dim, vdim, scale, mask {size} (absent: every earlier key)}, left_scale,
                   right {heads, kv_heads, dim, vdim, conv (taps)}, right_scale
    channel_delta: heads, kv_heads, dim, vdim, conv (taps), decay_rank, gate_rank (absent: as the checkpoint's tensors have them)
    mlp:           kind "moe", expert {ff}, router {experts, top}
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, ModelConfig
from .dekinex import _obj
from .sagalorn import _int, _num, _plain

MIXERS = ("parallel", "channel_delta")


def _heads(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    out: Dict[str, Any] = {"heads": _int(where, m, "heads"), "dim": _int(where, m, "dim")}
    out["kv_heads"] = _int(where, m, "kv_heads", out["heads"])
    if out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: heads ({out['heads']}) is not a multiple of kv_heads ({out['kv_heads']})")
    out["vdim"] = _int(where, m, "vdim", out["dim"])
    return out


def _delta(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    return {**_heads(where, m), "conv": _int(where, m, "conv", 1)}


def _attention(where: str, m: Dict[str, Any]) -> Dict[str, Any]:
    out = _heads(where, m)
    out["scale"] = _num(where, m, "scale", 1.0 / math.sqrt(out["dim"]))
    mask = _obj(where, m, "mask")
    if mask is not None:
        out["mask"] = {"size": _int(f"{where}.mask", mask, "size")}
    return out


def _check_layer(i: int, layer: Any) -> Dict[str, Any]:
    where = f"layers[{i}]"
    if not isinstance(layer, dict) or layer.get("type") not in MIXERS or not isinstance(layer.get("mixer"), dict):
        raise ConfigError(f"{where} must have a 'type' out of {', '.join(MIXERS)} and a 'mixer' object")
    kind, m = layer["type"], layer["mixer"]
    mw = f"{where}.mixer"
    if kind == "parallel":
        mixer = {"left": _attention(f"{mw}.left", _obj(mw, m, "left", True)), "left_scale": _num(mw, m, "left_scale", 1.0),
                 "right": _delta(f"{mw}.right", _obj(mw, m, "right", True)), "right_scale": _num(mw, m, "right_scale", 1.0)}
    else:
        mixer = _delta(mw, m)
        for key in ("decay_rank", "gate_rank"):
            if m.get(key) is not None:
                mixer[key] = _int(mw, m, key)
    mlp = layer.get("mlp")
    if mlp is not None:
        lw = f"{where}.mlp"
        if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
            raise ConfigError(f"{lw} must be null or an object of kind 'moe', got {mlp!r}")
        expert, router = _obj(lw, mlp, "expert", True), _obj(lw, mlp, "router", True)
        mlp = {"kind": "moe", "expert": {"ff": _int(f"{lw}.expert", expert, "ff")},
               "router": {"experts": _int(f"{lw}.router", router, "experts"), "top": _int(f"{lw}.router", router, "top")}}
        if mlp["router"]["top"] > mlp["router"]["experts"]:
            raise ConfigError(f"{lw}.router: 'top' ({mlp['router']['top']}) is above 'experts' ({mlp['router']['experts']})")
    return {"type": kind, "mixer": mixer, "mlp": mlp}


@dataclass(frozen=True)
class ZumizenConfig(ModelConfig):
    architecture = "Zumizen"

    vocab: int
    width: int
    layers: Tuple[Dict[str, Any], ...]
    norm_eps: float
    embedding_scale: float = 1.0
    bigram: Optional[Tuple[int, int, int]] = None   # (buckets, mul_prev, mul_cur)
    logit_softcap: float = 0.0                      # 0: none

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "ZumizenConfig":
        where = "config.json of Zumizen"
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError(f"{where} lacks a non-empty list 'layers'")
        checked = tuple(_check_layer(i, layer) for i, layer in enumerate(layers))
        eps = _num("norm", _obj(where, raw, "norm", True), "eps")
        if not eps > 0:
            raise ConfigError("norm: 'eps' must be positive")
        emb = _obj(where, raw, "embedding") or {}
        bigram = _obj("embedding", emb, "bigram")
        if bigram is not None:
            bigram = (_int("embedding.bigram", bigram, "buckets"), _int("embedding.bigram", bigram, "mul_prev", least=0),
                      _int("embedding.bigram", bigram, "mul_cur", least=0))
        cap = 0.0
        if raw.get("logit_softcap") is not None:
            cap = _num(where, raw, "logit_softcap")
            if not cap > 0:
                raise ConfigError(f"{where}: 'logit_softcap' must be positive")
        return cls(vocab=_int(where, raw, "vocab"), width=_int(where, raw, "width"), layers=checked, norm_eps=eps,
                   embedding_scale=_num("embedding", emb, "scale", 1.0), bigram=bigram, logit_softcap=cap)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
                               "layers": [{"type": l["type"], "mixer": _plain(l["mixer"]), "mlp": _plain(l["mlp"])}
                                          for l in self.layers]}
        if self.bigram is not None:
            out["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), self.bigram))
        if self.logit_softcap:
            out["logit_softcap"] = self.logit_softcap
        return out
