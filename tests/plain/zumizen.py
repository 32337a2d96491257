"""Plain, slow implementation of the Zumizen decoder: whole sequences, no cache, no state carried between calls.

One function per mechanism, float64 throughout, sharing no code with the engine.  ``cfg`` is the parsed
``config.json`` as it stands (nested), ``w`` maps the checkpoint's tensor names to tensors.

Notation: T tokens at positions 0..T-1; H (query or value) heads, G key/value (or query/key) heads, head h uses number
h // (H / G); dk key size, dv value size per head; a linear weight W is stored [out, in] and applied as x W^T.

A layer:  x <- x + n1(mixer(x));  x <- x + n2(experts(x)), n1 and n2 RMS norms with a weight.
``forward(..., coarse=k)`` rounds the activations to bfloat16 where a bfloat16 engine may, k = 1, 2, ... in so many ways: how far
that moves a position's logits is the scale of the device tests' bfloat16 tolerance.
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


def bf16(x: torch.Tensor, sample: int = 0) -> torch.Tensor:
    """Rounded to bfloat16; with ``sample`` on a grid stretched by a few ten-thousandths, which rounds other values up."""
    s = 1.0 + 0.00037 * sample
    return (x * s).to(torch.bfloat16).to(F64) / s


# ---------------------------------------------------------------------------------------------- embedding
def pair_row(before: Optional[int], token: int, buckets: int, mul_prev: int, mul_cur: int) -> int:
    """Which row of the pair table a token takes; ``before`` None: the sequence's first token."""
    return buckets if before is None else (before * mul_prev + token * mul_cur) % buckets


def embed(cfg: dict, w, tokens: List[int]) -> torch.Tensor:
    emb = cfg.get("embedding") or {}
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)] * emb.get("scale", 1.0)
    pairs = emb.get("bigram")
    if pairs:
        rows = [pair_row(tokens[t - 1] if t else None, tok, pairs["buckets"], pairs["mul_prev"], pairs["mul_cur"])
                for t, tok in enumerate(tokens)]
        x = x + w["bigram"][torch.tensor(rows, dtype=torch.long)]
    return x


# ---------------------------------------------------------------------------------------------- norms, small things
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def unit_length(x: torch.Tensor) -> torch.Tensor:
    """x / sqrt(sum(x^2) + 1e-6) over the last dimension."""
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0.0)


def causal_conv(u: torch.Tensor, taps_w: torch.Tensor) -> torch.Tensor:
    """u [T, C], taps_w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the first token."""
    T, C = u.shape
    taps = taps_w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += taps_w[:, j] * u[s]
    return y


# ---------------------------------------------------------------------------------------------- attention
def slopes(H: int) -> torch.Tensor:
    """What a key's distance costs a score, head by head: 2^(-8 (h + 1) / H)."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=F64)


def visible(T: int, chunk: int = 0) -> torch.Tensor:
    """[T, T] truth values: query i sees key j if j <= i and, with chunks, both lie in the same run of ``chunk``
    positions counted from 0."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if chunk:
        ok = ok & (i // chunk == j // chunk)
    return ok


def biased_scores(q: torch.Tensor, k: torch.Tensor, scale: float) -> torch.Tensor:
    """q [T, H, dk], k [T, G, dk] -> [H, T, T]: (q_i . k_j) scale - slope_h (i - j)."""
    T, H = q.shape[:2]
    group = H // k.shape[1]
    s = torch.stack([q[:, h] @ k[:, h // group].T for h in range(H)]) * scale
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(F64)
    return s - slopes(H)[:, None, None] * dist


def softmax_plus_one(s: torch.Tensor, mask: torch.Tensor) -> torch.Tensor:
    """p_ij = exp(s_ij) / (1 + sum over visible j' of exp(s_ij'))."""
    s = s.masked_fill(~mask[None], float("-inf"))
    top = s.max(-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(-top))


def attention_heads(w, pre: str, m: dict, eps: float, h: torch.Tensor, rnd=exact):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] as scores and sums read them."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (rnd(h @ w[pre + n].T + w[pre + n + ".b"]) for n in ("q", "k", "v"))
    q = unit_rms(q.view(T, H, dk), eps) * w[pre + "q.norm"]
    k = unit_rms(k.view(T, G, dk), eps) * w[pre + "k.norm"]
    return rnd(q), rnd(k), v.view(T, G, dv)


def attention(w, pre: str, m: dict, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    T, H = h.shape[0], m["heads"]
    q, k, v = attention_heads(w, pre, m, eps, h, rnd)
    p = softmax_plus_one(biased_scores(q, k, m["scale"]), visible(T, (m.get("mask") or {"size": 0})["size"]))
    group = H // m["kv_heads"]
    o = torch.stack([p[i] @ v[:, i // group] for i in range(H)], 1)
    return rnd(o.reshape(T, H * m["vdim"])) @ w[pre + "o"].T + w[pre + "o.b"]


# ---------------------------------------------------------------------------------------------- gated delta rule
def delta_rule(q, k, v, g, beta):
    """q, k [T, H, dk], v [T, H, dv], g [T, H, dk], beta [T, H] -> [T, H, dv].  Per head, S [dk, dv] from zero:
    S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = S * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta_heads(w, pre: str, m: dict, h: torch.Tensor, rnd=exact):
    """q, k [T, H, dk] of length one (q times dk^(-1/2)), v [T, H, dv]: the recurrence's operands."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (rnd(silu(causal_conv(rnd(h @ w[pre + n].T), w[pre + n + ".conv"]))) for n in ("q", "k", "v"))
    group = H // G
    q = (unit_length(q.view(T, G, dk)) * dk ** -0.5).repeat_interleave(group, 1)
    k = unit_length(k.view(T, G, dk)).repeat_interleave(group, 1)
    return q, k, v.view(T, H, dv)


def head_decay(w, pre: str, m: dict, h: torch.Tensor) -> torch.Tensor:
    """[T, H, dk]: one decay a head and token, the same for its key channels."""
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))
    return g[:, :, None].expand(-1, -1, m["dim"])


def channel_decay(w, pre: str, m: dict, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    """[T, H, dk]: one decay a head, key channel and token."""
    z = rnd(h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "dt_bias"]
    rate = torch.exp(w[pre + "A_log"])[None, :, None]
    return torch.exp(-rate * softplus(z).view(h.shape[0], m["heads"], m["dim"]))


def delta_output(w, pre: str, m: dict, eps: float, o: torch.Tensor, gate: torch.Tensor, rnd=exact) -> torch.Tensor:
    """Every head's o divided by its root mean square, times the heads' shared weight, times ``gate`` [T, H dv]; W_o."""
    T = o.shape[0]
    y = (unit_rms(o, eps) * w[pre + "norm"]).reshape(T, m["heads"] * m["vdim"]) * gate
    return rnd(y) @ w[pre + "o"].T


def gated_delta(w, pre: str, m: dict, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    q, k, v = delta_heads(w, pre, m, h, rnd)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    o = delta_rule(q, k, v, head_decay(w, pre, m, h), beta)
    return delta_output(w, pre, m, eps, o, silu(rnd(h @ w[pre + "g"].T)), rnd)


def channel_delta(w, pre: str, m: dict, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    q, k, v = delta_heads(w, pre, m, h, rnd)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    o = delta_rule(q, k, v, channel_decay(w, pre, m, h, rnd), beta)
    gate = torch.sigmoid(rnd(rnd(h @ w[pre + "g1"].T) @ w[pre + "g2"].T))
    return delta_output(w, pre, m, eps, o, gate, rnd)


def mixer(w, pre: str, layer: dict, eps: float, h: torch.Tensor, rnd=exact) -> torch.Tensor:
    m = layer["mixer"]
    if layer["type"] == "parallel":
        return (m["left_scale"] * attention(w, pre + "left.", m["left"], eps, h, rnd)
                + m["right_scale"] * gated_delta(w, pre + "right.", m["right"], eps, h, rnd))
    if layer["type"] == "channel_delta":
        return channel_delta(w, pre, m, eps, h, rnd)
    raise ValueError(layer["type"])


# ---------------------------------------------------------------------------------------------- feed-forward
def gated_unit(w, pre: str, x: torch.Tensor, rnd=exact) -> torch.Tensor:
    return rnd(silu(x @ w[pre + "gate"].T) * (x @ w[pre + "up"].T)) @ w[pre + "down"].T


def route(z: torch.Tensor, top: int):
    """z [T, E] -> (ids [T, top], weights [T, top]): the largest of sigmoid(z), as they stand (found by z, whose order is theirs:
    far from zero sigmoids are one number in any precision)."""
    z, ids = torch.topk(z, top, dim=-1)
    return ids, torch.sigmoid(z)


def route_margin(z: torch.Tensor, top: int) -> torch.Tensor:
    """[T]: by how much (of a logit) a token's choice is clear; infinite where nothing lost."""
    if top >= z.shape[1]:
        return torch.full((z.shape[0],), float("inf"), dtype=z.dtype)
    ordered = z.sort(-1, descending=True).values
    return ordered[:, top - 1] - ordered[:, top]


def experts(w, pre: str, mlp: dict, x: torch.Tensor, rnd=exact, margins: Optional[list] = None) -> torch.Tensor:
    """sum over a token's experts of expert(weight * x): the weight goes in, not out."""
    r = mlp["router"]
    z = x @ w[pre + "router"].T
    ids, weights = route(z, r["top"])
    if margins is not None:
        margins.append(route_margin(z, r["top"]))
    y = torch.zeros_like(x)
    for e in range(r["experts"]):
        chosen = ids == e
        rows = chosen.any(-1)
        if rows.any():
            share = (weights * chosen).sum(-1)[rows]
            y[rows] += gated_unit(w, f"{pre}e{e}.", share[:, None] * x[rows], rnd)
    return y


# ---------------------------------------------------------------------------------------------- the model
def capped(z: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return cap * torch.tanh(z / cap) if cap else z


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], coarse: int = 0,
            tap: Optional[list] = None, margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  ``tap`` receives the residual after every layer, ``margins`` every
    router's ``route_margin``."""
    rnd = (lambda t: bf16(t, coarse - 1)) if coarse else exact
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, tokens)
    for i, layer in enumerate(cfg["layers"]):
        name = f"l{i}."
        x = x + unit_rms(mixer(w, name + "mix.", layer, eps, rnd(x), rnd), eps) * w[name + "norm1"]
        if layer.get("mlp") is not None:
            y = experts(w, name + "mlp.", layer["mlp"], rnd(x), rnd, margins)
            x = x + unit_rms(y, eps) * w[name + "norm2"]
        if tap is not None:
            tap.append(x.clone())
    return capped(rnd(unit_rms(x, eps) * w["final.norm"]) @ w["head"].T, cfg.get("logit_softcap"))
