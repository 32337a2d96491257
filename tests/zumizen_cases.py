"""Small Zumizen configurations for the tests, and how their model folders are made.

Each differs from the others in every option: the two mixers in any order and number; one to six query heads a key head in
the attention and one to three value heads a key head in the delta rules; key sizes above and below value sizes, up to the
chunked recurrence's 64 and 128 channels and beyond them, heads that are no multiple of 16 and heads beyond the matrix-core
attention; runs of positions shorter than a page, across pages, and no runs at all; one to eight taps; narrow middles of
different and odd sizes; three to seventy experts, one to all of them a token; layers without a feed-forward, last and in the
middle; with and without the table of token pairs and the logits' bound; factors of the two mixers on both sides of 1, one
of them negative, one zero; sizes that are no multiple of 8.
"""
from __future__ import annotations

import os
from typing import Dict

import torch


def _moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def _left(heads, kv_heads, dim, vdim, scale, run=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if run:
        out["mask"] = {"size": run}
    return out


def _delta(heads, kv_heads, dim, vdim, conv, ranks=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}
    if ranks:
        out["decay_rank"], out["gate_rank"] = ranks
    return out


def _parallel(left, left_scale, right, right_scale, mlp):
    return {"type": "parallel", "mixer": {"left": left, "left_scale": left_scale, "right": right, "right_scale": right_scale}, "mlp": mlp}


def _channel(mixer, mlp):
    return {"type": "channel_delta", "mixer": mixer, "mlp": mlp}


CASES: Dict[str, dict] = {
    # both mixers, each twice; runs of 24 and 50; two query heads a key head, two value heads a delta key head
    "A": dict(architecture="Zumizen", vocab=211, width=64, norm={"eps": 1e-5}, logit_softcap=9.0,
              embedding={"scale": 3.0, "bigram": {"buckets": 37, "mul_prev": 11, "mul_cur": 5}},
              layers=[_parallel(_left(4, 2, 24, 16, 0.4, 24), 0.6, _delta(4, 2, 16, 24, 3), 0.9, _moe(6, 1, 24)),
                      _channel(_delta(2, 2, 32, 16, 4, (24, 8)), _moe(6, 2, 16)),
                      _parallel(_left(3, 3, 16, 32, 0.3, 50), 1.4, _delta(2, 1, 40, 8, 2), 0.5, _moe(5, 3, 32)),
                      _channel(_delta(3, 3, 24, 24, 2, (8, 16)), None)]),
    # no runs, no pairs, no bound; one key head for six query heads; one tap; every expert chosen; a factor below zero
    "B": dict(architecture="Zumizen", vocab=130, width=96, norm={"eps": 3e-6}, embedding={"scale": 0.7},
              layers=[_channel(_delta(3, 1, 64, 48, 1, (16, 24)), _moe(4, 4, 40)),
                      _parallel(_left(6, 1, 48, 48, 0.2), -0.8, _delta(3, 3, 16, 64, 4), 1.7, None),
                      _parallel(_left(2, 2, 64, 64, 0.15, 33), 1.0, _delta(6, 2, 32, 32, 1), 1.0, _moe(3, 1, 64))]),
    # sizes that the matrix-core products do not take in bfloat16; runs shorter than a page; odd heads and middles
    "C": dict(architecture="Zumizen", vocab=53, width=50, norm={"eps": 1e-5}, logit_softcap=30.0,
              embedding={"scale": 1.0, "bigram": {"buckets": 1, "mul_prev": 3, "mul_cur": 2}},
              layers=[_parallel(_left(3, 3, 10, 6, 0.9, 7), 0.7, _delta(3, 3, 6, 9, 2), 1.2, _moe(3, 1, 30)),
                      _channel(_delta(2, 1, 10, 5, 3, (5, 7)), _moe(5, 3, 12))]),
    # heads beyond the matrix-core attention; key sizes above 64 and above 128; many taps; seventy experts
    "D": dict(architecture="Zumizen", vocab=160, width=128, norm={"eps": 2e-5}, logit_softcap=4.0,
              embedding={"scale": 12.0, "bigram": {"buckets": 1009, "mul_prev": 100003, "mul_cur": 7919}},
              layers=[_channel(_delta(2, 2, 96, 144, 5, (32, 40)), _moe(70, 3, 8)),
                      _parallel(_left(2, 1, 136, 136, 0.2, 64), 0.9, _delta(2, 2, 128, 32, 8), 0.4, _moe(8, 8, 16)),
                      _channel(_delta(2, 1, 160, 20, 4, (8, 8)), _moe(4, 2, 24)),
                      _parallel(_left(8, 1, 48, 64, 0.25, 200), 0.0, _delta(1, 1, 72, 80, 3), 1.1, _moe(16, 2, 32))]),
    # layers of two kinds in turn, three times over
    "E": dict(architecture="Zumizen", vocab=97, width=72, norm={"eps": 1e-6}, logit_softcap=20.0,
              embedding={"scale": 5.0, "bigram": {"buckets": 50, "mul_prev": 2, "mul_cur": 9}},
              layers=[_parallel(_left(2, 1, 16, 16, 0.5, 40), 0.8, _delta(2, 1, 24, 16, 4), 0.9, _moe(8, 2, 24)),
                      _channel(_delta(2, 2, 16, 32, 3, (16, 8)), _moe(8, 2, 24))] * 3),
}


def folder_of(base: str, name: str, seed: int = 0, std: float = 0.05, calm: bool = False) -> str:
    """Writes (once) the model folder of a case: random matrices, and vectors of sizes that matter (``_spread``).  ``calm``: every
    router's rows are multiples of one row, so that which experts a token goes to hangs on one sign and not, here and there, on
    less than rounding to bfloat16 moves two logits by."""
    from glassbox_amd.config import config_from_dict
    from glassbox_amd.weights import write_random_model
    folder = os.path.join(base, f"zumizen_{name}_{seed}" + ("_calm" if calm else ""))
    if not os.path.exists(os.path.join(folder, "model.safetensors")):
        write_random_model(config_from_dict(CASES[name]), folder, seed, std=std, norm_init="uniform", dtype=torch.float32)
        _spread(folder, seed, calm)
    return folder


def _spread(folder: str, seed: int, calm: bool) -> None:
    """The writer draws vectors as small as matrix entries; here they get sizes at which a fault shows: biases of the order of
    what they are added to, norm weights of either sign, taps of the order of one, decays between almost none and almost
    all a token, projections large enough that scores, betas, gates and the choice of experts spread out."""
    from glassbox_amd.weights import SafetensorsFile, save_file
    path = os.path.join(folder, "model.safetensors")
    f = SafetensorsFile(path)
    tensors = {n: f.tensor(n).clone() for n in f.names()}
    f.close()
    gen = torch.Generator().manual_seed(seed + 1000)
    draw = lambda t, s: torch.randn(t.shape, generator=gen) * s
    for n, t in tensors.items():
        last = n.rsplit(".", 1)[-1]
        if n.endswith((".norm1", ".norm2")):
            tensors[n] = draw(t, 0.3) + 0.4
        elif n.endswith((".q.norm", ".k.norm", ".mix.norm", ".right.norm")):
            tensors[n] = draw(t, 0.4) + 1.0
        elif n.endswith((".q.b", ".k.b", ".o.b")):
            tensors[n] = draw(t, 0.3)
        elif n.endswith(".v.b"):
            tensors[n] = draw(t, 0.1)
        elif last == "conv":
            tensors[n] = draw(t, 0.6)
        elif last == "A_log":
            tensors[n] = draw(t, 1.5) - 0.5
        elif last == "dt_bias":
            tensors[n] = draw(t, 1.5) - 2.0
        elif last in ("embed", "bigram", "head"):
            tensors[n] = t * 8.0
        elif last in ("q", "k", "a", "a1", "a2", "b", "g", "g1", "g2", "router"):
            tensors[n] = t * 6.0
        elif last in ("gate", "up", "down", "v", "o"):
            tensors[n] = t * 3.0
        if last == "router" and calm:
            steps = torch.randperm(t.shape[0], generator=gen).float() - (t.shape[0] - 1) / 2 + 0.25
            tensors[n] = steps[:, None] * tensors[n][:1] * (4.0 / t.shape[0])
    save_file(tensors, path)


def rounded(w: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """The weights as a bfloat16 engine holds them: matrices rounded, vectors and the convolutions' taps (kept in 32-bit)
    as they are."""
    return {k: (v.to(torch.bfloat16).to(v.dtype) if v.dim() == 2 and not k.endswith(".conv") else v) for k, v in w.items()}
