"""Two mixers that read the same rows, their results added: left(h) + right(h).

Each is a mixer that can be taken apart (``w_in``, ``mix(ctx, proj, mixed, cache)``, ``mixed_cols``, ``wo``, perhaps ``b_out``: see
``GatedAttention`` and ``GatedDeltaRule``; a factor on a result is the mixer's own ``result_scale``): one product makes the projections of
both, each turns its columns into its columns of the rows that one output product reads, and that product adds the two results
up.  They share a cache layer, one of them its pages, one its state."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from .base import LayerCache, Mixer, Part, product, product_in_slices


class SideBySide(Mixer):
    replayable = True
    taped = True
    accepts_store = True
    hands_on_bias = True

    def __init__(self, left: Mixer, right: Mixer, names=("left", "right")):
        for what in ("cache_spec", "state_spec"):
            if getattr(left, what) is not None and getattr(right, what) is not None:
                raise ValueError("mixers side by side: a cache layer has the pages of one of them and the state of one of them")
        self.left, self.right = left, right
        self.names = tuple(names)
        self.cache_spec = left.cache_spec if left.cache_spec is not None else right.cache_spec
        self.state_spec = left.state_spec if left.state_spec is not None else right.state_spec
        self.w_in = self.wo = self.b_out = None
        self.left_rows = 0

    def children(self) -> Dict[str, Part]:
        return dict(zip(self.names, (self.left, self.right)))

    def load_tree(self, tensors, prefix: str = "") -> None:
        super().load_tree(tensors, prefix)
        left, right = self.left, self.right
        self.left_rows = left.w_in.shape[0]                  # (a multiple of 8: the right one's rows begin at 16-byte words)
        self.w_in = torch.cat([left.w_in, right.w_in], 0)
        self.wo = torch.cat([left.wo, right.wo], 1).contiguous()
        biases = [b for b in (getattr(left, "b_out", None), getattr(right, "b_out", None)) if b is not None]
        self.b_out = sum(biases[1:], biases[0]).contiguous() if biases else None
        left.w_in = left.wo = right.w_in = right.wo = None   # (held once, here)

    def streamed_matrices(self):
        inner = [t for m in (self.left, self.right) for t in m.streamed_matrices() if t is not None]
        return [self.w_in, self.wo] + inner

    def forward(self, ctx, h, residual, cache: Optional[LayerCache], store: bool = False, hand_on_bias: bool = False):
        """Adds the mixed rows into ``residual``; with ``store`` writes them there instead (float32 either way) or leaves
        them in slices, and returns what ``product_in_slices`` does (``hand_on_bias``: the outputs' bias, not yet added, as a
        third entry)."""
        n = h.shape[0]
        proj = ctx.buffer("side_proj", (n, self.w_in.shape[0]), ctx.dtype)
        product(ctx, h, self.w_in, proj)
        cols = self.left.mixed_cols
        both = self.wo.shape[1]
        mixed = ctx.buffer("side_mixed", (n, -(-both // 8) * 8), ctx.dtype)[:, :both]   # (rows begin at 16-byte words)
        self.left.mix(ctx, proj[:, :self.left_rows], mixed[:, :cols], cache)
        self.right.mix(ctx, proj[:, self.left_rows:], mixed[:, cols:], cache)
        if store and (self.b_out is None or hand_on_bias):   # the caller's pass over the rows adds the slices
            made = product_in_slices(ctx, mixed, self.wo, residual)
            return made + (self.b_out,) if hand_on_bias else made
        product(ctx, mixed, self.wo, residual, accumulate=not store)
        if self.b_out is not None:
            ops.add_bias(residual, self.b_out)
        return (residual, 1) if store else None
