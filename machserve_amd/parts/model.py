"""A decoder built from a :class:`ModelSpec`: embedding, blocks chosen layer by layer from
the registries, final norm, output head.  ``order`` is the list of layers a step runs; it
may name a layer twice.  Only the rows whose logits are wanted reach the head
(the reference computes the head for every row, ``crates/mach-model/src/batched.rs:4594-4626``).
"""
from __future__ import annotations

from typing import List, Optional

import torch

from ..config.specs import ModelSpec
from .base import Block, MultiStream, Part, ResidualStream, Runtime, StepContext, TensorDecl, require_kernel_sizes
from .registry import BLOCKS, EMBEDDINGS, HEADS, NORMS, register_embedding, register_head


@register_embedding("embedding")
class Embedding(Part):
    """Rows of a table, times the spec's ``scale`` (1 for an embedding that is not scaled)."""

    def tensor_decls(self):
        return [TensorDecl("weight", (self.spec.vocab, self.spec.width), "matrix")]

    def load(self, t):
        self.weight = t["weight"]

    def forward(self, tokens: torch.Tensor) -> torch.Tensor:
        return self.rt.ops.embed(tokens, self.weight, getattr(self.spec, "scale", 1.0))


@register_embedding("pair_embedding")
class PairEmbedding(Part):
    """Rows of a table plus rows of a second table chosen by the token and the one before it in its request: row
    ``(previous * mul_prev + token * mul_cur) mod buckets``, and the last row (``buckets``) for a request's first token.
    The previous token is state of the request (one integer a slot), so an embedding of this kind reads the step
    (``reads_step``) and asks the cache manager for a state like a mixer does."""
    reads_step = True

    def tensor_decls(self):
        s = self.spec
        return [TensorDecl("weight", (s.vocab, s.width), "matrix"), TensorDecl("pairs", (s.buckets + 1, s.width), "matrix")]

    def load(self, t):
        self.weight, self.pairs = t["weight"], t["pairs"]

    def cache_request(self):
        from .base import StateRequest
        return StateRequest({"token": ()}, torch.int32)

    def bind_cache(self, binding):
        self.prev = binding.tensors["token"]

    def forward_step(self, ctx: StepContext) -> torch.Tensor:
        s = self.spec
        return self.rt.ops.embed_pair(ctx.tokens, self.weight, self.pairs, self.prev, ctx.seq_q_start, ctx.seq_q_len, ctx.seq_pos0,
                                      ctx.seq_slot, s.mul_prev, s.mul_cur, s.buckets)


@register_head("linear")
class Head(Part):
    """Output projection, times the spec's ``scale``, then capped by a tanh if the spec has a ``softcap``; tied to the embedding table when the spec says so, or
    when it leaves it open and the checkpoint has no head tensor
    (``crates/mach-model/src/loader.rs:1025-1033``).  A head is built with the model's embedding part as
    its third argument and has ``forward(h) -> float32 logits`` and ``vocab`` in its spec."""

    def __init__(self, spec, rt, embedding):
        super().__init__(spec, rt)
        self.embedding = embedding
        self.weight = None

    def tensor_decls(self):
        if self.spec.tied is True:
            return []
        return [TensorDecl("weight", (self.spec.vocab, self.spec.width), "matrix", optional=self.spec.tied is None)]

    def ignored_tensors(self):
        """Checkpoint names that may be present without being used."""
        return [self.spec.tensors.get("weight", "weight")] if self.spec.tied is True else []

    def load(self, t):
        self.weight = t.get("weight")

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        w = self.weight if self.weight is not None else self.embedding.weight
        logits = self.rt.ops.linear(h, w, None, out_f32=True)
        scale, cap = getattr(self.spec, "scale", 1.0), getattr(self.spec, "softcap", 0.0)
        if cap:
            self.rt.ops.softcap(logits, scale, cap)  # scale, then cap * tanh(. / cap), in one pass
        elif scale != 1.0:
            logits *= scale
        return logits


class LoopSteps(Part):
    """What is added to the stream ahead of each pass over looped layers: the embedding's output again (in every pass but the
    first) and the pass's own row of a small table, both in 32-bit."""

    def tensor_decls(self):
        return [TensorDecl("step", (len(self.spec.starts), self.spec.width), "vector")]

    def load(self, t):
        self.rows = [t["step"][i].contiguous() for i in range(len(self.spec.starts))]

    def open(self, number: int, stream: ResidualStream, first: Optional[torch.Tensor]) -> None:
        self.rt.ops.open_pass(stream.open(), first if number > 0 else None, self.rows[number])


class DecoderModel:
    def __init__(self, spec: ModelSpec, rt: Runtime):
        spec.validate()
        self.spec, self.rt = spec, rt
        require_kernel_sizes(rt, "output head", [("width", spec.embedding.width)])
        self.embedding = EMBEDDINGS.build(spec.embedding, rt)
        self.blocks: List[Block] = []
        for layer in spec.layers:  # a block builds its own parts from the fields of its layer's spec
            self.blocks.append(BLOCKS.get(layer.block)(layer, rt))
        self.order = list(spec.order)
        steps = getattr(spec, "loop_steps", None)
        self.loop_steps = LoopSteps(steps, rt) if steps is not None else None
        self._passes = {p: t for t, p in enumerate(steps.starts)} if steps is not None else {}
        self.final_norm = NORMS.build(spec.final_norm, rt)
        self.head = HEADS.build(spec.head, rt, self.embedding)
        self._bindings, self._rebind = [], False
        # Debugging aid: a callable (name, float32 stream [rows, width]) that sees the residual stream after the
        # embedding and after every run of a layer (crates/mach-model/src/batched.rs:3040-3088 dumps the same
        # points).  While it is set the step function runs every step as it is, from no captured graph.
        self.observer = None

    # ------------------------------------------------------------------ structure
    def parts(self) -> List[Part]:
        out: List[Part] = [self.embedding]
        for b in self.blocks:
            for p in b.parts():
                out.append(p)
                out.extend(getattr(p, "sub_parts", lambda: [])())
        if self.loop_steps is not None:
            out.append(self.loop_steps)
        out += [self.final_norm, self.head]
        return out

    def cache_requests(self):
        """One cache request per *position of the order*: a layer that runs twice shares its
        weights between the two runs, but each run keeps a cache (or state) of its own, so
        what a run reads never depends on how the tokens were cut into steps.  A layer that
        reads another layer's cache reads that of the layer's latest earlier run."""
        from .base import SharedKVRequest

        def placed(req, p, i):
            if isinstance(req, SharedKVRequest):
                earlier = [q for q in range(p) if self.order[q] == req.source_layer]
                if not earlier:
                    raise ValueError(f"layer {i} reads the cache of layer {req.source_layer}, which has not run before it")
                return SharedKVRequest(earlier[-1])
            return req

        out = []
        for p, i in enumerate(self.order):
            req = self.blocks[i].cache_request()
            out.append([placed(r, p, i) for r in req] if isinstance(req, (list, tuple)) else placed(req, p, i))
        if hasattr(self.embedding, "cache_request"):  # an embedding with state of its own: one more entry after the layers'
            out.append(self.embedding.cache_request())
        return out

    def bind_cache(self, device_cache) -> None:
        self._bindings = [device_cache.binding(p) for p in range(len(self.order))]
        for p, i in enumerate(self.order):  # a layer that runs once keeps its binding for good
            if self._bindings[p] is not None:
                self.blocks[i].bind_cache(self._bindings[p])
        self._rebind = len(set(self.order)) != len(self.order)
        if hasattr(self.embedding, "cache_request"):
            self.embedding.bind_cache(device_cache.binding(len(self.order)))

    def attention_rows_per_token(self) -> List[int]:
        return sorted({g for b in self.blocks for m in b.mixers() for g in [m.attention_rows_per_token()] if g})

    def attention_rows_per_block(self) -> Optional[int]:
        """The unit of the attention work lists, which every mixer's kernel must share (the lists are made
        once per step); None if no mixer wants them."""
        units = {(u, type(m).__name__, getattr(m.spec, "head_dim", None))
                 for b in self.blocks for m in b.mixers() for u in [m.attention_rows_per_block()] if u}
        if len({u for u, _, _ in units}) > 1:
            raise ValueError("the mixers' attention kernels take blocks of different numbers of rows: "
                             + ", ".join(f"{name} (head size {hd}): {u}" for u, name, hd in sorted(units)))
        return next(iter(units))[0] if units else None

    def position_axes(self) -> int:
        """Numbers per position of a step: the most that any position encoding of the model reads."""
        return max([getattr(p, "axes", 1) for p in self.parts()] + [1])

    @property
    def vocab(self) -> int:
        return self.spec.head.vocab

    # ------------------------------------------------------------------ the forward pass
    def forward(self, ctx: StepContext) -> Optional[torch.Tensor]:
        """Run the step's rows through the layers in ``order``; float32 logits ``[W, vocab]`` of
        the wanted rows, or None when none is wanted."""
        # What the layers of one pass share (a table of the rows' rotation angles) is made anew in every pass: a context
        # is run once to load everything and once more under capture, and what the first run left would be missing
        # from the captured graph, which would then rotate every later step by the first step's positions.
        ctx.shared.clear()
        embedding = self.embedding
        x = embedding.forward_step(ctx) if getattr(embedding, "reads_step", False) else embedding.forward(ctx.tokens)
        streams = getattr(self.spec, "streams", None)  # several residual streams that all start as the embedding
        stream = MultiStream(x, streams, self.rt.ops) if streams else ResidualStream(x, self.rt.ops)
        watch = self.observer
        if watch is not None:
            watch("embedding", stream.value())
        first = x.clone() if len(self._passes) > 1 else None  # the layers add to x in place
        for p, i in enumerate(self.order):
            if p in self._passes:
                self.loop_steps.open(self._passes[p], stream, first)
            if self._rebind and self._bindings[p] is not None:
                self.blocks[i].bind_cache(self._bindings[p])
            self.blocks[i].forward(stream, ctx)
            if watch is not None:  # the sums still pending are added first: the value is the whole stream
                watch(f"layer{p:02d}", stream.value())
        if ctx.want_rows.numel() == 0:
            return None
        if streams:  # the sum of the streams, of the wanted rows only
            return self.head.forward(self.final_norm.forward(stream.read(None, ctx.want_rows)))
        return self.head.forward(self.final_norm.forward(stream, rows=ctx.want_rows))
