"""The gated delta rule: a matrix memory whose decayed content is corrected towards each token's value.

q = W_q h and k = W_k h (``n_qk_heads`` heads of ``key_dim`` channels), v = W_v h (``n_heads`` of ``value_dim``); head h uses the
query and key head h // (n_heads / n_qk_heads).  Every channel of the three passes a short causal convolution over time
(``q.conv`` ... [channels, taps], zeros before the first token) and silu; q and k are then made unit vectors a head,
x / sqrt(sum(x^2) + 1e-6), and q is multiplied by key_dim^(-1/2).  With beta = sigmoid(W_b h), one number a head, and a decay g
in (0, 1), per head

  S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

from S = 0, and each head's o is divided by its root mean square, multiplied by ``norm`` (a weight the heads share) and by
act(gate), and projected by ``o``.  Options:

* ``decay``: "head": g = exp(-exp(A_log_h) softplus(W_a h + dt_bias)), one a head and token (``a``); "channel": one a head, key
  channel and token, with W_a2 (W_a1 h) through a narrow middle in W_a h's place (``a1``, ``a2``), acting on the rows of S;
* ``gate``: "full": W_g h (``g``); "low": W_g2 (W_g1 h) through a narrow middle (``g1``, ``g2``); ``gate_act``: "silu" | "sigmoid";
* ``result_scale``: the result counts times this number (on the norm's weight).

One product makes the projections; with narrow middles one more makes the decay's and the gate's logits together.  A request's
state is S and the last projections of its convolutions, 32-bit.  Everything from the unit lengths on is 32-bit in both
precisions."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from .base import LayerCache, Mixer, StateSpec, TensorSpec, product, product_in_slices


def _filled(rows: int, width: int, like: torch.Tensor) -> list:
    """Zero rows that fill ``rows`` up to a multiple of 8."""
    return [torch.zeros((-rows % 8, width), dtype=like.dtype, device=like.device)] if rows % 8 else []


class GatedDeltaRule(Mixer):
    replayable = True
    taped = True
    accepts_store = True

    def __init__(self, width: int, n_heads: int, n_qk_heads: int, key_dim: int, value_dim: int, taps: int, eps: float,
                 decay: str = "head", gate: str = "full", gate_act: str = "silu", decay_rank: Optional[int] = None,
                 gate_rank: Optional[int] = None, result_scale: float = 1.0):
        """``decay_rank``, ``gate_rank``: the narrow middles; None takes them from the checkpoint's tensors."""
        if n_heads % n_qk_heads:
            raise ValueError(f"{n_heads} value heads are not a multiple of {n_qk_heads} query and key heads")
        if decay not in ("head", "channel") or gate not in ("full", "low") or gate_act not in ("silu", "sigmoid"):
            raise ValueError("decay: head | channel; gate: full | low; gate_act: silu | sigmoid")
        if (decay == "channel") != (gate == "low"):
            raise ValueError("a decay a key channel comes with a gate through a narrow middle: one product makes both")
        self.width, self.n_heads, self.n_qk_heads = width, n_heads, n_qk_heads
        self.key_dim, self.value_dim, self.taps, self.eps = key_dim, value_dim, int(taps), float(eps)
        self.decay, self.gate, self.gate_act, self.result_scale = decay, gate, gate_act, float(result_scale)
        self.decay_rank, self.gate_rank = decay_rank, gate_rank
        self.v_dim = n_heads * value_dim
        self.channels = 2 * n_qk_heads * key_dim + self.v_dim
        self.mixed_cols = self.v_dim
        self.state_spec = StateSpec((ops.delta_slot(n_heads, n_qk_heads, key_dim, value_dim, self.taps)[0],), torch.float32, 0.0)
        self.w_in = self.w_low = self.wo = self.wconv = self.rate = self.dt = self.norm_weight = None
        self.low_at = self.low_cols = self.b_at = self.a_at = 0

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        H, G, D, V, d = self.n_heads, self.n_qk_heads, self.key_dim, self.value_dim, self.width
        specs = {}
        for name, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
            specs[name] = TensorSpec((rows, d))
            specs[name + ".conv"] = TensorSpec((rows, self.taps), kind="f32")
        specs["b"] = TensorSpec((H, d))
        specs["A_log"] = TensorSpec((H,), kind="f32")
        specs["norm"] = TensorSpec((V,), kind="f32", init="ones")
        if self.decay == "head":
            specs["a"] = TensorSpec((H, d))
            specs["dt_bias"] = TensorSpec((H,), kind="f32")
        else:
            r = -1 if self.decay_rank is None else self.decay_rank
            specs.update({"a1": TensorSpec((r, d)), "a2": TensorSpec((H * D, r)), "dt_bias": TensorSpec((H * D,), kind="f32")})
        if self.gate == "full":
            specs["g"] = TensorSpec((H * V, d))
        else:
            r = -1 if self.gate_rank is None else self.gate_rank
            specs.update({"g1": TensorSpec((r, d)), "g2": TensorSpec((H * V, r))})
        specs["o"] = TensorSpec((d, H * V))
        return specs

    def load(self, tensors):
        d = self.width
        parts = [tensors["q"], tensors["k"], tensors["v"]] + ([tensors["g"]] if self.gate == "full" else [])
        rows = lambda: sum(p.shape[0] for p in parts)
        if self.decay == "channel":
            a1, a2, g1, g2 = (tensors[n] for n in ("a1", "a2", "g1", "g2"))
            if a1.shape[0] != a2.shape[1] or g1.shape[0] != g2.shape[1]:
                raise ValueError(f"narrow middles: a1 has {a1.shape[0]} rows and a2 {a2.shape[1]} columns, g1 {g1.shape[0]} and g2 "
                                 f"{g2.shape[1]}")
            parts += _filled(rows(), d, a1)   # (the middles begin at a 16-byte word and fill whole ones: a product reads them)
            self.low_at = rows()
            parts += [a1, g1] + _filled(a1.shape[0] + g1.shape[0], d, a1)
            self.low_cols = rows() - self.low_at
            self.w_low = torch.zeros((a2.shape[0] + g2.shape[0], self.low_cols), dtype=a2.dtype, device=a2.device)
            self.w_low[:a2.shape[0], :a2.shape[1]] = a2
            self.w_low[a2.shape[0]:, a1.shape[0]:a1.shape[0] + g1.shape[0]] = g2
        self.b_at = rows()
        parts.append(tensors["b"])
        self.a_at = rows()
        if self.decay == "head":
            parts.append(tensors["a"])
        parts += _filled(rows(), d, tensors["b"])
        self.w_in = torch.cat(parts, 0)
        self.wo = tensors["o"].contiguous()
        # a row a tap: neighbouring channels' weights of one tap lie side by side
        self.wconv = torch.cat([tensors[n + ".conv"] for n in ("q", "k", "v")], 0).float().t().contiguous()
        self.rate = torch.exp(tensors["A_log"].float()).contiguous()
        self.dt = tensors["dt_bias"].float().contiguous()
        self.norm_weight = (tensors["norm"].float() * self.result_scale).contiguous()

    def streamed_matrices(self):
        return [t for t in (self.w_in, self.w_low, self.wo) if t is not None]

    def problems(self, dtype, page_size):
        out = []   # (sizes that the matrix-core products do not take go through the plain product)
        if self.key_dim > ops.DELTA_MAX_KEY_DIM:
            out.append(("dim", f"{self.key_dim} is above {ops.DELTA_MAX_KEY_DIM}, the largest key size the recurrence kernels take"))
        if self.value_dim > ops.DELTA_MAX_VALUE_DIM:
            out.append(("vdim", f"{self.value_dim} is above {ops.DELTA_MAX_VALUE_DIM}, the largest value size the recurrence kernels take"))
        if not 1 <= self.taps <= ops.CONV_MAX_TAPS:
            out.append(("taps", f"{self.taps}: the convolution's kernel takes 1 to {ops.CONV_MAX_TAPS}"))
        return out

    def forward(self, ctx, h, residual, cache: Optional[LayerCache], store: bool = False):
        """Adds the mixed rows into ``residual``; with ``store`` writes them there instead (float32 either way) or leaves
        them in slices, and returns what ``product_in_slices`` does."""
        n = h.shape[0]
        proj = ctx.buffer("delta_proj", (n, self.w_in.shape[0]), ctx.dtype)
        product(ctx, h, self.w_in, proj)
        mixed = ctx.buffer("delta_mixed", (n, self.mixed_cols), ctx.dtype)
        self.mix(ctx, proj, mixed, cache)
        if store:   # the caller's pass over the rows adds the slices of a product that divides k
            return product_in_slices(ctx, mixed, self.wo, residual)
        product(ctx, mixed, self.wo, residual, accumulate=True)
        return None

    def mix(self, ctx, proj, mixed, cache: Optional[LayerCache]) -> None:
        """From the stacked projections (``w_in``) to the rows that the output projection (``wo``) reads; both may be columns
        of wider rows."""
        if cache is None or cache.state is None:
            raise ValueError("GatedDeltaRule needs a layer cache with state")
        n, H, D = proj.shape[0], self.n_heads, self.key_dim
        z = None
        if self.decay == "channel":
            low = ctx.buffer("delta_low", (n, self.w_low.shape[0]), torch.float32)   # [decay logits | gate logits]
            product(ctx, proj[:, self.low_at:self.low_at + self.low_cols], self.w_low, low)
            z, gate = low[:, :H * D], low[:, H * D:]
        else:
            gate = proj[:, self.channels:self.channels + self.v_dim]
        ops.delta_rule(proj, 0, self.b_at, self.a_at, self.wconv, self.rate, self.dt, z, cache.state, ctx, H, self.n_qk_heads, D,
                       self.value_dim, gate, self.gate_act == "sigmoid", self.norm_weight, self.eps, mixed)
