"""A short causal convolution over time on the residual itself: what a mixer reads is h = x + conv(x),
conv(x)[t] = sum_j w[:, j] x[t - taps + 1 + j] over the request's own tokens (``weight`` [width, taps], no bias, zeros
before the first token).  The request's last taps - 1 rows of x are its state, in 32-bit like the residual."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from .base import LayerCache, Part, StateSpec, TensorSpec
from .norm import GroupRMSNorm


class TimeConv(Part):
    replayable = True
    taped = True

    def __init__(self, width: int, taps: int):
        """``taps`` 0: no convolution, the rows are the residual rounded to the activations' type."""
        self.width, self.taps = int(width), int(taps)
        self.state_spec = StateSpec((self.taps - 1, self.width), torch.float32, 0.0) if self.taps > 1 else None
        self.weight: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {"weight": TensorSpec((self.width, self.taps), kind="f32")} if self.taps else {}

    def load(self, tensors):
        if self.taps:
            self.weight = tensors["weight"].float().t().contiguous()   # a row a tap: neighbouring channels side by side

    def problems(self, dtype, page_size):
        if self.taps > ops.TIME_CONV_MAX_TAPS:
            return [("taps", f"{self.taps} is above {ops.TIME_CONV_MAX_TAPS}, the longest convolution the kernel takes")]
        return []

    def entry_spec(self, ctx, n: int, cache: Optional[LayerCache]):
        """``(weight, state)`` for ``ops.norm_add(conv=)`` if the pass that adds a normed sublayer into the residual may
        make this convolution's rows as well (every request of the step brings one row), else None."""
        if not self.taps:
            return (None, None)   # the rows are the new residual, whatever the step
        if (int(ctx.host["max_q_len"]) != 1 or not ops.norm_add_takes_rows(self.width)
                or (self.taps > 1 and (cache is None or cache.state is None))):
            return None
        return (self.weight, cache.state if self.taps > 1 else None)

    def forward(self, ctx, x, cache: Optional[LayerCache], out_name: str = "h") -> torch.Tensor:
        """The rows a mixer reads, in the activations' type; moves the requests' state on (call it before x changes)."""
        if self.taps > 1 and (cache is None or cache.state is None):
            raise ValueError("TimeConv needs its state (the last rows of each request)")
        out = ctx.buffer(out_name, tuple(x.shape), ctx.dtype)
        ops.time_conv(x, self.weight, cache.state if self.taps > 1 else None, ctx, out)
        return out


class ConvolvedNorm(Part):
    """What a sublayer reads of the residual: h = g + conv(g), g the grouped RMS norm of the residual (``GroupRMSNorm``) and
    conv(g)[t] = sum_j w[:, j] g[t - taps + 1 + j] over the request's own tokens (``conv`` [width, taps], no bias, zeros before the
    first token; ``taps`` 0: no convolution).  The request's last taps - 1 rows of g are its state, in 32-bit; several of these
    may keep theirs side by side in one slot ([convolutions, taps - 1, width]), this one at ``place``.

    ``after`` is also the pass that makes the residual: it adds the sublayer before into it and forms a sum over depth
    (``parts.depth``), so that a step of single tokens needs one kernel between two sublayers."""
    replayable = True
    taped = True

    def __init__(self, norm: GroupRMSNorm, taps: int, place: int = 0, names=("norm", "conv")):
        self.norm, self.width, self.taps, self.place = norm, norm.width, int(taps), int(place)
        self.names = tuple(names)
        self.weight: Optional[torch.Tensor] = None

    def children(self) -> Dict[str, Part]:
        return {self.names[0]: self.norm}

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.names[1]: TensorSpec((self.width, self.taps), kind="f32")} if self.taps else {}

    def load(self, tensors):
        if self.taps:
            self.weight = tensors[self.names[1]].float().t().contiguous()   # a row a tap: neighbouring channels side by side

    def problems(self, dtype, page_size):
        out = super().problems(dtype, page_size)
        if self.taps > ops.NORM_CONV_MAX_TAPS:
            out.append(("taps", f"{self.taps} is above {ops.NORM_CONV_MAX_TAPS}, the longest convolution the kernel takes"))
        return out

    def after(self, ctx, x, cache: Optional[LayerCache], y=None, slices: int = 1, average=None, out_name: str = "h") -> torch.Tensor:
        """x += y (float32, or ``slices`` pieces of it), ``average = (hist, coef, out)`` as ``ops.residual_rows`` takes it, and the
        rows of the result (x, or out) that the sublayer reads, in the activations' type; moves the requests' state on."""
        state = None
        if self.taps > 1:
            if cache is None or cache.state is None:
                raise ValueError("ConvolvedNorm needs its state (the last rows of each request)")
            state = cache.state[:, self.place]
        n, norm = x.shape[0], self.norm
        h = ctx.buffer(out_name, (n, self.width), ctx.dtype)
        if int(ctx.host["max_q_len"]) == 1 and ctx.tuned:   # single tokens: their rows need nothing of the step's other rows
            ops.residual_rows(x, y, slices, average, norm.weight, norm.groups, norm.eps, h=h,
                              conv=(self.weight, state) if self.taps else None, ctx=ctx)
            return h
        scales = ctx.buffer("norm_scales", (n, norm.groups), torch.float32)
        ops.residual_rows(x, y, slices, average, groups=norm.groups, eps=norm.eps, scales=scales)
        ops.norm_conv(average[2] if average is not None else x, scales, norm.weight, self.weight, state, ctx, h)
        return h
