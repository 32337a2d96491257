"""A decoder assembled from parts, with the order of its layers as data.

``blocks`` are the layers that own weights.  ``schedule`` is the list of calls
that a step makes, in order: each names a block and the cache layer it writes
(``cache``) or, instead, a cache layer that it only reads (``reads``).  A block
may be named twice (shared weights, each call with a cache layer of its own),
and a call may read the cache that an earlier call wrote.  For Llama the
schedule is simply block i with cache layer i
(crates/glassbox-core/src/model.rs:251).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import torch

from .. import ops
from .base import CacheSpec, LayerCache, Norm, Normed, Part, PreNormed, StateSpec, TensorSpec
from .depth import DepthAverage
from .embedding import Embedding, LMHead
from .tape import LayerTapes


@dataclass(frozen=True)
class LayerCall:
    block: int
    cache: Optional[int] = None   # cache layer this call writes and reads
    reads: Optional[int] = None   # or: cache layer of another call that this one only reads
    enter: Optional[int] = None   # the number of the pass over a repeated run that begins with this call (``PassEntry``)


class PassEntry(Part):
    """What a model adds to the residual where a pass over a repeated run of layers begins: before every pass but
    the first the embedding's output (the residual as it was before the first layer), and before every pass, the first
    too, row t of ``step`` ([passes, width]), t the number of the pass.  32-bit."""
    replayable = True

    def __init__(self, passes: int, width: int, add_embedding: bool = True):
        self.passes, self.width, self.add_embedding = int(passes), int(width), bool(add_embedding)
        self.step: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {"step": TensorSpec((self.passes, self.width), kind="f32", init="normal")}

    def load(self, tensors):
        self.step = tensors["step"].contiguous()

    def forward(self, ctx, x, embedded, t: int) -> None:
        if not 0 <= t < self.passes:
            raise ValueError(f"pass {t} of {self.passes}")
        ops.axpy_rows(x, embedded if (t > 0 and self.add_embedding) else None, 1.0, self.step[t])


class DecoderModel(Part):
    replayable = True

    def __init__(self, config, embedding: Embedding, blocks: Sequence[Part], schedule: Sequence[LayerCall],
                 final_norm: Norm, head: LMHead, names=("model.embed_tokens", "model.layers.{}", "model.norm", "lm_head"),
                 ignorable: Sequence[str] = (), arg_keys: Optional[Dict[str, str]] = None, sources=None,
                 streams: Optional[int] = None, passes: Optional[PassEntry] = None, passes_name: str = "loop",
                 depth: Optional[Sequence[DepthAverage]] = None, depth_name: str = "depth{}"):
        self.config = config
        #: what is added to the residual where a pass over a repeated run begins (``LayerCall.enter``), or None
        self.passes, self.passes_name = passes, passes_name
        if passes is not None and streams is not None:
            raise ValueError("a residual of several streams has no pass entries")
        #: one ``DepthAverage`` a schedule entry: what goes on behind it is a sum over all results so far.  The blocks are
        #: then ``ConvNormBlock``s (or anything with ``in1.after`` and a ``forward`` that returns what is still to be added)
        self.depth, self.depth_name = None if depth is None else list(depth), depth_name
        if self.depth is not None and (streams is not None or passes is not None or len(self.depth) != len(schedule)
                                       or any(a.inputs != i + 2 for i, a in enumerate(self.depth))):
            raise ValueError("sums over depth: one for every schedule entry, over its number + 2 inputs, on a single residual")
        #: None: one residual [n, width]; a number: the residual is so many streams, [streams, n, width], which the
        #: embedding fills alike and the blocks and the final norm take as such (parts.streams)
        self.streams = streams
        #: where the checkpoint keeps a tensor that it names or cuts otherwise than the parts do: a mapping, or a
        #: function, from the model's tensor name to the checkpoint's name or to (name, first row, last row) of a
        #: tensor that holds several stacked by rows; None for a tensor of the same name (weights.loader)
        self.sources = sources
        #: constructor argument of a part -> the key of config.json that set it, for messages
        self.arg_keys = dict(arg_keys or {})
        self.embedding, self.blocks, self.schedule = embedding, list(blocks), list(schedule)
        self.final_norm, self.head = final_norm, head
        self.names = tuple(names)
        self.ignorable = tuple(ignorable)   # tensors a checkpoint may hold that the model does not use
        self.vocab_size = embedding.vocab
        self.width = embedding.width
        self._check_schedule()
        self._taped: Optional[List[bool]] = None       # which blocks let their launches be recorded (parts.tape)
        self.loads = 0                                # times the weights were loaded: recorded tensors are theirs

    # structure ------------------------------------------------------------------
    def children(self) -> Dict[str, Part]:
        out: Dict[str, Part] = {self.names[0]: self.embedding}
        for i, b in enumerate(self.blocks):
            out[self.names[1].format(i)] = b
        out[self.names[2]] = self.final_norm
        out[self.names[3]] = self.head
        if self.passes is not None:
            out[self.passes_name] = self.passes
        for i, average in enumerate(self.depth or ()):
            out[self.depth_name.format(i)] = average
        return out

    def source_of(self, name: str):
        if self.sources is None:
            return None
        return self.sources(name) if callable(self.sources) else self.sources.get(name)

    def _check_schedule(self) -> None:
        owners: Dict[int, int] = {}
        for pos, call in enumerate(self.schedule):
            if not 0 <= call.block < len(self.blocks):
                raise ValueError(f"schedule entry {pos} names block {call.block}, there are {len(self.blocks)}")
            if call.cache is not None and call.reads is not None:
                raise ValueError(f"schedule entry {pos} both owns and borrows a cache layer")
            if call.cache is not None:
                if call.cache in owners:
                    raise ValueError(f"cache layer {call.cache} is written by schedule entries {owners[call.cache]} and {pos}")
                owners[call.cache] = pos
        for pos, call in enumerate(self.schedule):
            if call.reads is not None and (call.reads not in owners or owners[call.reads] >= pos):
                raise ValueError(f"schedule entry {pos} reads cache layer {call.reads}, which no earlier entry writes")
        self.num_cache_layers = (max(owners) + 1) if owners else 0
        if sorted(owners) != list(range(self.num_cache_layers)):
            raise ValueError("cache layers must be numbered 0..n-1 without gaps")
        self._owners = owners
        for pos, call in enumerate(self.schedule):
            if call.enter is not None and self.passes is None:
                raise ValueError(f"schedule entry {pos} begins a pass, and the model has no pass entry")
        #: an embedding that keeps something of each request from step to step gets a cache layer of its own, the last
        self.embedding_cache = self.num_cache_layers if getattr(self.embedding, "state_spec", None) is not None else None

    def cache_specs(self) -> List[Optional[CacheSpec]]:
        """What each cache layer holds: the block that writes it says."""
        out = [self.blocks[self.schedule[self._owners[c]].block].cache_spec() for c in range(self.num_cache_layers)]
        return out + ([None] if self.embedding_cache is not None else [])

    def state_specs(self) -> List[Optional[StateSpec]]:
        out = [self.blocks[self.schedule[self._owners[c]].block].state_spec() for c in range(self.num_cache_layers)]
        return out + ([self.embedding.state_spec] if self.embedding_cache is not None else [])

    # the step ---------------------------------------------------------------------
    def forward(self, ctx, caches: Sequence[LayerCache]) -> torch.Tensor:
        """Runs the tokens of ``ctx`` through every scheduled layer; logits [wanted, vocab] float32."""
        if self.depth is not None:
            return self._forward_averaged(ctx, caches)
        shape = (ctx.n, self.width) if self.streams is None else (self.streams, ctx.n, self.width)
        embedded = None
        keep = self.passes is not None and self.passes.add_embedding
        if keep:   # the embedding writes a second copy, which later passes add to the residual
            shape = (2,) + shape
        x = ctx.buffer("x", shape, torch.float32)
        if self.embedding_cache is not None:
            self.embedding.forward(ctx, x, caches[self.embedding_cache])
        else:
            self.embedding.forward(ctx, x)
        if keep:
            x, embedded = x[0], x[1]
        pre = pre_kind = None   # what the block before prepared of this block's first norm (or of the rows it reads)
        if self._taped is None:
            self._taped = [b.all_taped() for b in self.blocks]
        tapes = None
        if getattr(ctx, "layer_tapes", False) and any(self._taped):
            tapes = LayerTapes(ctx, ctx.workspace.tape_sites, self.loads)
        for i, call in enumerate(self.schedule):
            if call.cache is not None:
                cache = caches[call.cache]
            elif call.reads is not None:
                src = caches[call.reads]
                cache = LayerCache(src.k_pages, src.v_pages, src.group, src.state, writable=False)
            else:
                cache = None
            block = self.blocks[call.block]
            if call.enter is not None:
                self.passes.forward(ctx, x, embedded, call.enter)
                pre = pre_kind = None   # (what the block before prepared was of the residual before this)
            # what a block hands to the next: the work of that block's first norm (entry_norm), or the rows its mixer
            # reads (entry_rows, which also needs the cache layer that holds the next block's state)
            handover = "entry_norm" if hasattr(block, "entry_norm") else "entry_rows" if hasattr(block, "entry_rows") else None
            more = {}
            if handover:
                last = i + 1 == len(self.schedule)
                after = None if last else self.blocks[self.schedule[i + 1].block]
                if not last and self.schedule[i + 1].enter is not None:
                    after = None   # the residual changes before the next block reads it: nothing to prepare
                more = {"pre": pre if pre_kind == handover else None, "emit": None}
                if handover == "entry_norm" and hasattr(after, "entry_norm"):
                    more["emit"] = after.entry_norm(ctx, ctx.n)
                elif handover == "entry_rows" and hasattr(after, "entry_rows"):
                    nxt = self.schedule[i + 1]
                    more["emit"] = after.entry_rows(ctx, ctx.n, caches[nxt.cache] if nxt.cache is not None else None)
                if handover == "entry_norm" and last and self._head_takes_prepared(ctx):
                    # the last block prepares the final norm as it would the next block's first
                    more["emit"] = self.final_norm.emit_spec(ctx, ctx.n)
            if tapes is not None and self._taped[call.block]:
                # the first layer of a kind walks through its parts and is recorded; the others are replayed
                out = tapes.forward(i, block, x, cache, more)
            else:
                out = block.forward(ctx, x, cache, **more)
            pre, pre_kind = (out, handover) if handover else (None, None)
        if ctx.want.numel() == 0:
            return ctx.buffer("logits", (0, self.vocab_size), torch.float32)
        if self._head_takes_prepared(ctx) and isinstance(pre, (PreNormed, Normed)):
            return self.head.forward(ctx, pre.rows, prepared=pre if isinstance(pre, PreNormed) else None)
        rows = self.final_norm.forward(ctx, x, rows=ctx.want, out_name="h_out")
        return self.head.forward(ctx, rows)

    def _forward_averaged(self, ctx, caches: Sequence[LayerCache]) -> torch.Tensor:
        """The same for a model with sums over depth.  The step's rows keep every layer's result: x[i + 1] is the residual that
        layer i reads and adds into, X_(i + 1) from then on, and the sum behind it begins x[i + 2].  One pass over the rows
        adds a layer's last sublayer, forms the sum and makes the rows that the next layer's mixer reads."""
        x = ctx.buffer("x_by_depth", (len(self.schedule) + 2, ctx.n, self.width), torch.float32)
        self.embedding.forward(ctx, x[:2])
        if self._taped is None:
            self._taped = [b.all_taped() for b in self.blocks]
        tapes = None
        if getattr(ctx, "layer_tapes", False) and any(self._taped):
            tapes = LayerTapes(ctx, ctx.workspace.tape_sites, self.loads, moving=True)
        cache_of = lambda call: caches[call.cache] if call.cache is not None else None
        h = self.blocks[self.schedule[0].block].in1.after(ctx, x[1], cache_of(self.schedule[0]))
        for i, call in enumerate(self.schedule):
            block, cache = self.blocks[call.block], cache_of(call)
            if tapes is not None and self._taped[call.block]:
                made = tapes.forward(i, block, x[i + 1], cache, {"pre": h})
            else:
                made = block.forward(ctx, x[i + 1], cache, pre=h)
            y, slices = made if made is not None else (None, 1)
            if i + 1 < len(self.schedule):
                after = self.schedule[i + 1]
                h = self.blocks[after.block].in1.after(ctx, x[i + 1], cache_of(after), y, slices,
                                                       self.depth[i].spec(x, x[i + 2]))
            else:
                self.depth[i].forward(ctx, x[i + 1], x, x[i + 2], y, slices)
        if ctx.want.numel() == 0:
            return ctx.buffer("logits", (0, self.vocab_size), torch.float32)
        return self.head.forward(ctx, self.final_norm.forward(ctx, x[-1], rows=ctx.want, out_name="h_out"))

    def _head_takes_prepared(self, ctx) -> bool:
        """Whether the product that ends the last block may prepare the final norm for the vocabulary product: every
        row's logits are wanted, in the rows' order (a step of single tokens), and the rows are few."""
        return (bool(ctx.host.get("want_all")) and ops.head_takes_parts(ctx.n)
                and hasattr(self.final_norm, "emit_spec") and getattr(self.head, "accepts_prepared", False))

    def load_tree(self, tensors, prefix: str = "") -> None:
        super().load_tree(tensors, prefix)
        self.loads += 1   # what engines keep of the layers' tensors (parts.tape) is of the weights before

    def streamed_matrices(self) -> List[torch.Tensor]:
        """Every tensor a step reads whole, once each: those of the scheduled blocks (a block named twice, or a
        table that two parts share, counts once) and of the head; each part says which are its own."""
        seen, out = set(), []
        parts = [self.blocks[call.block] for call in self.schedule] + [self.final_norm, self.head]
        for part in parts:
            for t in part.streamed_matrices():
                if t.data_ptr() not in seen:
                    seen.add(t.data_ptr())
                    out.append(t)
        return out

    def weight_bytes(self) -> int:
        """Bytes of the matrices a decode step reads once (model.rs:175-184: norm vectors excluded)."""
        return sum(t.numel() * t.element_size() for t in self.streamed_matrices())

    def refusals(self, dtype, page_size: int) -> List[str]:
        """One line for each thing the kernels would refuse at these settings, every part asked
        (``Part.problems``); a complaint that many layers share is given once, with the first layer that has it.
        ``arg_keys`` (from the builder) says which key of config.json set a part's argument."""
        seen, lines = set(), []
        for name, part in self.children().items():
            for arg, why in part.problems(dtype, page_size):
                if (arg, why) in seen:
                    continue
                seen.add((arg, why))
                key = self.arg_keys.get(arg)
                lines.append(f"{name}: {arg}" + (f" (config.json: {key})" if key else "") + f": {why}")
        return lines
