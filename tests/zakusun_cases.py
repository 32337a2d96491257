"""Small Zakusun configurations for the tests, and how their model folders are made.

Each differs from the others in every option: one to twenty heads, of 6 to 264 channels, keys larger and smaller than
values; latents narrower and wider than the heads, of 18 to 520 channels (some that the matrix-core kernel does not take);
norms in one to five groups; no convolution, or one to five taps; two to sixteen experts, one to all of them a token, some
with units that are always clamped; layers without a feed-forward, first, in the middle and last; layers of one kind in a
row and layers that all differ; sizes that are no multiple of 8; logit scales on both sides of 1.
Score scales are large enough that single keys carry visible weight.
"""
from __future__ import annotations

import os
from typing import Dict

import torch


def _moe(experts, top, ff, limit):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def _layer(heads, dim, vdim, kv_rank, scale, mlp):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}, "mlp": mlp}


_E = _layer(3, 16, 24, 64, 0.25, _moe(4, 4, 24, 2.0))

CASES: Dict[str, dict] = {
    # layers that all differ; keys larger than values; more experts than one token sees; a last layer without a feed-forward
    "A": dict(architecture="Zakusun", vocab=211, width=96, norm={"eps": 1e-5, "groups": 3}, canon={"taps": 3}, logit_scale=0.5,
              layers=[_layer(5, 24, 16, 40, 0.3, _moe(6, 2, 24, 0.8)), _layer(2, 32, 32, 128, 0.25, _moe(4, 1, 40, 5.0)),
                      _layer(4, 16, 48, 24, 0.4, None)]),
    # one group; a convolution of one tap (no state); more than sixteen heads; every expert for every token; a first layer
    # without a feed-forward
    "B": dict(architecture="Zakusun", vocab=130, width=64, norm={"eps": 3e-6, "groups": 1}, canon={"taps": 1}, logit_scale=2.0,
              layers=[_layer(18, 16, 32, 136, 0.5, None), _layer(1, 64, 8, 64, 0.2, _moe(4, 4, 32, 1.2)),
                      _layer(17, 8, 8, 256, 0.6, _moe(3, 2, 8, 30.0))]),
    # sizes that neither the matrix-core products nor the kernels by words take in bfloat16
    "C": dict(architecture="Zakusun", vocab=53, width=50, norm={"eps": 1e-5, "groups": 5}, canon={"taps": 2}, logit_scale=1.0,
              layers=[_layer(3, 10, 6, 18, 0.9, _moe(3, 1, 30, 0.4)), _layer(2, 6, 10, 7, 0.8, _moe(5, 3, 11, 1.0))]),
    # wide latents (the widest the matrix-core kernel takes, and one beyond it); heads beyond the matrix-core attention and
    # beyond the plain one; five taps
    "D": dict(architecture="Zakusun", vocab=160, width=128, norm={"eps": 2e-5, "groups": 2}, canon={"taps": 5}, logit_scale=0.1,
              layers=[_layer(20, 8, 40, 264, 0.5, _moe(16, 16, 8, 1.0)), _layer(2, 136, 64, 512, 0.2, _moe(4, 2, 64, 0.6)),
                      _layer(1, 264, 24, 520, 0.15, None), _layer(2, 24, 260, 96, 0.3, _moe(2, 1, 16, 3.0))]),
    # six layers of one kind, then one more without a feed-forward; no convolution
    "E": dict(architecture="Zakusun", vocab=97, width=72, norm={"eps": 1e-6, "groups": 2}, logit_scale=0.25,
              layers=[_E] * 5 + [dict(_E, mlp=None), _E]),
    # the same with a convolution
    "F": dict(architecture="Zakusun", vocab=97, width=72, norm={"eps": 1e-6, "groups": 3}, canon={"taps": 4}, logit_scale=0.7,
              layers=[_E] * 6),
}


def folder_of(base: str, name: str, seed: int = 0, std: float = 0.05) -> str:
    """Writes (once) the model folder of a case: random matrices, and vectors of sizes that matter (``_spread``)."""
    from glassbox_amd.config import config_from_dict
    from glassbox_amd.weights import write_random_model
    folder = os.path.join(base, f"zakusun_{name}_{seed}")
    if not os.path.exists(os.path.join(folder, "model.safetensors")):
        write_random_model(config_from_dict(CASES[name]), folder, seed, std=std, norm_init="uniform", dtype=torch.float32)
        _spread(folder, seed)
    return folder


def _spread(folder: str, seed: int) -> None:
    """The writer draws vectors as small as matrix entries; here they get sizes at which a fault shows: norm weights of
    either sign, convolution taps of the order of one, sinks that take a visible share, router biases that change which
    experts are chosen, weights over depth that differ and may be negative, and projections large enough that scores spread
    out and units reach their limits."""
    from glassbox_amd.weights import SafetensorsFile, save_file
    path = os.path.join(folder, "model.safetensors")
    f = SafetensorsFile(path)
    tensors = {n: f.tensor(n).clone() for n in f.names()}
    f.close()
    gen = torch.Generator().manual_seed(seed + 1000)
    draw = lambda t, s: torch.randn(t.shape, generator=gen) * s
    for n, t in tensors.items():
        last = n.rsplit(".", 1)[-1]
        if n == "embed":
            tensors[n] = draw(t, 0.7)
        elif last in ("norm1", "norm2"):
            tensors[n] = draw(t, 0.3) + 0.6
        elif last in ("canon1", "canon2"):
            tensors[n] = draw(t, 0.4)
        elif last == "dwa":
            tensors[n] = draw(t, 0.2)
            tensors[n][-1] += 0.8
        elif last == "sink":
            tensors[n] = draw(t, 1.0)
        elif n.endswith(".router.b"):
            tensors[n] = draw(t, 0.5)
        elif t.dim() == 2:   # a linear weight: rows of about the same length whatever the layer's sizes
            size = {"q": 1.5, "uk": 1.5, "router": 3.0, "g": 1.5, "gate": 1.5, "up": 1.5, "o": 0.6, "down": 0.6}.get(last, 1.0)
            tensors[n] = draw(t, size / t.shape[1] ** 0.5)
    save_file(tensors, path)


def rounded(w: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """The weights as a bfloat16 engine holds them: matrices rounded, vectors and the convolutions' taps (kept in 32-bit)
    as they are."""
    return {k: (v.to(torch.bfloat16).to(v.dtype) if v.dim() == 2 and ".canon" not in k else v) for k, v in w.items()}
