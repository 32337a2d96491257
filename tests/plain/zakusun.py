"""Plain, slow implementation of the Zakusun decoder: whole sequences, no cache, no state carried between calls.

One function per mechanism, float64 throughout, sharing no code with the engine.  ``cfg`` is the parsed
``config.json`` as it stands (nested), ``w`` maps the checkpoint's tensor names to tensors.

Notation: T tokens at positions 0..T-1; H heads of dk key and dv value channels; a linear weight W is stored [out, in] and
applied as x W^T.  X[0] is the embedded sequence, X[i + 1] what layer i makes of what it is given.

A layer:  x <- x + mixer(c1(n1(x)));  x <- x + experts(c2(n2(x))), every n an RMS norm in groups of channels and every
c(h) = h + a causal convolution of h over time; then what goes on is a weighted sum of X[0] ... X[i + 1].
``forward(..., coarse=True)`` rounds the activations to bfloat16 where a bfloat16 engine may: how far that moves a
position's logits is the scale of the device tests' bfloat16 tolerance.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch

from .llama import read_safetensors

F64 = torch.float64


def load_folder(folder: str):
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    w = {k: v.to(F64) for k, v in read_safetensors(os.path.join(folder, "model.safetensors")).items()}
    return cfg, w


def exact(x: torch.Tensor) -> torch.Tensor:
    return x


def bf16(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.bfloat16).to(F64)


# ---------------------------------------------------------------------------------------------- embedding
def sinusoid(positions: torch.Tensor, width: int) -> torch.Tensor:
    """[T, width]: channels 2i and 2i + 1 are sine and cosine of p * 10000^(-2i / width)."""
    out = torch.zeros(len(positions), width, dtype=F64)
    for c in range(width):
        i = c // 2
        ang = positions.to(F64) * 10000.0 ** (-2.0 * i / width)
        out[:, c] = torch.sin(ang) if c % 2 == 0 else torch.cos(ang)
    return out


def embed(cfg: dict, w, tokens: List[int]) -> torch.Tensor:
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    return x + sinusoid(torch.arange(len(tokens)), cfg["width"])


# ---------------------------------------------------------------------------------------------- norms, convolution
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def group_norm(x: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Every one of ``groups`` equal runs of neighbouring channels divided by its own root mean square; one weight a
    channel."""
    T, d = x.shape
    return unit_rms(x.reshape(T, groups, d // groups), eps).reshape(T, d) * weight


def with_conv(h: torch.Tensor, taps_w: Optional[torch.Tensor]) -> torch.Tensor:
    """h_t + sum_j w[:, j] h_(t - taps + 1 + j), zeros before the first token; taps_w [d, taps] (None: no convolution)."""
    if taps_w is None:
        return h
    T = h.shape[0]
    taps = taps_w.shape[1]
    y = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += taps_w[:, j] * h[s]
    return y


def depth_average(weights: torch.Tensor, history: List[torch.Tensor]) -> torch.Tensor:
    """sum_j weights[j] history[j]."""
    out = torch.zeros_like(history[0])
    for j, x in enumerate(history):
        out += weights[j] * x
    return out


# ---------------------------------------------------------------------------------------------- attention
def softmax_with_sink(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """s [H, T, T], sink [H]: p_ij = exp(s_ij) / (exp(sink_h) + sum over j' <= i of exp(s_ij')).  The sink has no
    value, so the weights of a row sum to less than one."""
    T = s.shape[-1]
    s = s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], float("-inf"))
    top = torch.maximum(s.max(-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - top))


def latent(w, pre: str, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    """[T, kv_rank]: what keys and values of all heads are made of."""
    return rnd(unit_rms(rnd(h @ w[pre + "dkv"].T), eps) * w[pre + "dkv.norm"])


def attend(q, k, v, scale: float, sink) -> torch.Tensor:
    """q, k [T, H, dk], v [T, H, dv] -> [T, H, dv]: causal, a sink a head in the denominator."""
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    return torch.einsum("hij,jhd->ihd", softmax_with_sink(s, sink), v)


def latent_attention(w, pre: str, m: dict, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = rnd(h @ w[pre + "q"].T).view(T, H, dk)
    c = latent(w, pre, eps, h, rnd)
    k = rnd(c @ w[pre + "uk"].T).view(T, H, dk)
    v = rnd(c @ w[pre + "uv"].T).view(T, H, dv)
    o = rnd(attend(q, k, v, m["scale"], w[pre + "sink"]).reshape(T, H * dv))
    gate = torch.sigmoid(rnd(h @ w[pre + "g"].T))
    return rnd(o * gate) @ w[pre + "o"].T


def latent_attention_absorbed(w, pre: str, m: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    """The same result by another route: every head's query taken through W_uk into the latent's space, scores and
    weighted sums over the latents themselves, the sum taken through W_uv."""
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T).view(T, H, dk)
    c = latent(w, pre, eps, h)
    ql = torch.einsum("thd,hdr->thr", q, w[pre + "uk"].view(H, dk, -1))
    o = attend(ql, c[:, None].expand(-1, H, -1), c[:, None].expand(-1, H, -1), m["scale"], w[pre + "sink"])
    o = torch.einsum("thr,hvr->thv", o, w[pre + "uv"].view(H, dv, -1)).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


# ---------------------------------------------------------------------------------------------- feed-forward
def clamped_unit(w, pre: str, limit: float, x: torch.Tensor, rnd=exact) -> torch.Tensor:
    g = rnd(x @ w[pre + "gate"].T).clamp(max=limit)
    u = rnd(x @ w[pre + "up"].T).clamp(min=-limit, max=limit)
    return rnd(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def route(z: torch.Tensor, top: int):
    """z [T, E] the logits, bias included -> (ids [T, top], weights [T, top]): the largest logits, softmax over them."""
    best = torch.topk(z, top, dim=-1)
    return best.indices, torch.softmax(best.values, -1)


def route_margin(z: torch.Tensor, top: int) -> torch.Tensor:
    """[T]: how far the last chosen logit lies above the first that was not; infinite if every expert is chosen."""
    if top == z.shape[-1]:
        return torch.full((z.shape[0],), float("inf"), dtype=z.dtype)
    ordered = z.sort(-1, descending=True).values
    return ordered[:, top - 1] - ordered[:, top]


def experts(w, pre: str, mlp: dict, x: torch.Tensor, rnd=exact, margins: Optional[list] = None) -> torch.Tensor:
    r = mlp["router"]
    z = x @ w[pre + "router"].T + w[pre + "router.b"]
    ids, weights = route(z, r["top"])
    if margins is not None:
        margins.append(route_margin(z, r["top"]))
    y = torch.zeros_like(x)
    for e in range(r["experts"]):
        chosen = ids == e
        rows = chosen.any(-1)
        if rows.any():
            share = (weights * chosen).sum(-1)[rows]
            y[rows] += share[:, None] * clamped_unit(w, f"{pre}e{e}.", mlp["expert"]["limit"], x[rows], rnd)
    return y


# ---------------------------------------------------------------------------------------------- the model
def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], coarse: bool = False,
            tap: Optional[list] = None, margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  ``tap`` receives what every layer hands on, ``margins`` every router's
    ``route_margin``."""
    rnd = bf16 if coarse else exact
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = embed(cfg, w, tokens)
    history = [x]
    for i, layer in enumerate(cfg["layers"]):
        name = f"l{i}."
        h = rnd(with_conv(group_norm(x, w[name + "norm1"], groups, eps), w.get(name + "canon1")))
        x = x + latent_attention(w, name + "mix.", layer["mixer"], eps, h, rnd)
        if layer.get("mlp") is not None:
            h = rnd(with_conv(group_norm(x, w[name + "norm2"], groups, eps), w.get(name + "canon2")))
            x = x + experts(w, name + "mlp.", layer["mlp"], h, rnd, margins)
        history.append(x)
        x = depth_average(w[name + "dwa"], history)
        if tap is not None:
            tap.append(x.clone())
    return rnd(group_norm(x, w["final.norm"], groups, eps)) @ w["embed"].T * cfg["logit_scale"]
