"""A decoder put together from a `ModelSpec`: embedding, the layers run in the order of the
schedule, final norm, head (simply/model_lib.py:2750 TransformerLM, apply :2935-3189).

The model knows nothing of any one architecture: every part is built from its registry by
the kind that the spec names.
"""
from __future__ import annotations

import dataclasses
from typing import Callable, Mapping

import torch

from .. import parts as _parts  # noqa: F401  (registers the built-in parts)
from ..config.spec import LayerSpec, ModelSpec, PartSpec
from ..kernels import ops
from ..parts.base import Block, ParamSpec, Part, PendingNorm
from ..parts.streams import StreamSum, begin_streams
from ..registry import BLOCKS, EMBEDDINGS, FEED_FORWARDS, HEADS, MIXERS, NORMS, PASS_INPUTS, STREAM_PARTS
from ..weights import binding


def _build_layer(spec: LayerSpec) -> Block:
    mixer = MIXERS.build(spec.mixer.kind, **spec.mixer.params)
    ffn = None if spec.feed_forward is None else FEED_FORWARDS.build(spec.feed_forward.kind, **spec.feed_forward.params)
    norms = {name: NORMS.build(ns.kind, **ns.params) for name, ns in spec.norms.items()}
    if spec.extras:
        extras = tuple(STREAM_PARTS.build(es.kind, **es.params) for es in spec.extras)
        return BLOCKS.build(spec.block.kind, mixer, ffn, norms, extras=extras, **spec.block.params)
    return BLOCKS.build(spec.block.kind, mixer, ffn, norms, **spec.block.params)


class DecoderModel:
    def __init__(self, spec: ModelSpec):
        spec.validate()
        self.spec = spec
        self.embedding = EMBEDDINGS.build(spec.embedding.kind, **spec.embedding.params)
        self.head = HEADS.build(spec.head.kind, **spec.head.params)
        self.final_norm = NORMS.build(spec.final_norm.kind, **spec.final_norm.params)
        self.pass_input = None if spec.pass_input is None else PASS_INPUTS.build(spec.pass_input.kind, **spec.pass_input.params)
        self.layers: list[Block] = [_build_layer(ls) for ls in spec.layers]
        self.stream_sum = None if spec.streams is None else StreamSum(spec.streams)
        self.loaded = False

    # ------------------------------------------------------------------ tensors
    def _bindings(self) -> list[tuple[Part, PartSpec]]:
        out: list[tuple[Part, PartSpec]] = [(self.embedding, self.spec.embedding)]
        if self.pass_input is not None:
            out.append((self.pass_input, self.spec.pass_input))
        for block, ls in zip(self.layers, self.spec.layers):
            if ls.block.tensors:   # (a block arrangement with weights of its own)
                out.append((block, ls.block))
            out.append((block.mixer, ls.mixer))
            if ls.feed_forward is not None:
                out.append((block.feed_forward, ls.feed_forward))
            for name, ns in ls.norms.items():
                out.append((block.norms[name], ns))
            for part, es in zip(getattr(block, "extras", ()), ls.extras):
                out.append((part, es))
        out.append((self.final_norm, self.spec.final_norm))
        out.append((self.head, self.spec.head))
        return out

    def tensor_bindings(self) -> list[tuple[Part, str, ParamSpec, "binding.Binding"]]:
        """For every parameter of every part: (part, the part's name for it, what the part expects, how it is
        obtained from stored tensors).  A spec that names a plain tensor means that tensor as it is."""
        out = []
        for part, ps in self._bindings():
            for local, pspec in part.param_specs().items():
                if local not in ps.tensors:
                    raise ValueError(f"part {ps.kind!r} needs a tensor {local!r} that its spec does not name")
                b = binding.normalize(ps.tensors[local], pspec.shape)
                try:
                    got = binding.shape_of(b)
                except binding.BindingError as e:
                    raise ValueError(f"part {ps.kind!r}, tensor {local!r}: {e}") from None
                if tuple(got) != tuple(pspec.shape):
                    raise ValueError(f"part {ps.kind!r}, tensor {local!r}: the binding gives shape {list(got)}, the "
                                     f"part expects {list(pspec.shape)}")
                out.append((part, local, pspec, b))
        return out

    def expected_tensors(self) -> dict[str, ParamSpec]:
        """Stored tensor name in the model folder -> what is expected of it (its stored shape; role and random
        initialisation of the parameter that it feeds), in a fixed order."""
        expected: dict[str, ParamSpec] = {}
        for _, _, pspec, b in self.tensor_bindings():
            for leaf in binding.leaves(b):
                if leaf.name in expected and expected[leaf.name].shape != leaf.shape:
                    raise ValueError(f"tensor {leaf.name!r} is used with shapes {expected[leaf.name].shape} and "
                                     f"{leaf.shape}")
                expected.setdefault(leaf.name, dataclasses.replace(pspec, shape=leaf.shape))
        return expected

    def load_tensors(self, tensors: Mapping[str, torch.Tensor]) -> None:
        """`tensors`: stored name -> device tensor in its final dtype.  Every part receives its parameters as its
        spec's bindings make them from these."""
        from ..kernels import packing

        per_part: dict[int, tuple[Part, dict[str, torch.Tensor]]] = {}
        for part, local, _, b in self.tensor_bindings():
            per_part.setdefault(id(part), (part, {}))[1][local] = binding.evaluate(b, tensors.__getitem__)
        try:
            for part, _ in self._bindings():
                part.load(per_part.get(id(part), (part, {}))[1])
        finally:
            packing.clear_cache()   # sharing of re-laid tensors (tied table and head) ends with the load
        if self.stream_sum is not None:
            self.stream_sum.to_device(next(iter(tensors.values())).device)
        self.loaded = True

    # ------------------------------------------------------------------ cache
    def cache_needs(self):
        """For each schedule entry: (need of its mixer or None, cache_from); then, if the embedding keeps something
        per request, one more entry for it (its view is the one behind the schedule's)."""
        needs = [(self.layers[e.layer].mixer.cache_need(), e.cache_from) for e in self.spec.schedule]
        own = getattr(self.embedding, "cache_need", None)
        if own is not None and own() is not None:
            needs.append((own(), None))
        return needs

    # ------------------------------------------------------------------ forward
    def forward(self, tokens: torch.Tensor, ctx, cache_views, logit_rows: torch.Tensor | None,
                logits_out: torch.Tensor | None = None, after_layer=None) -> torch.Tensor | None:
        """Runs this step's tokens through the schedule.  Returns float32 logits [R, V] at the rows of
        the step that `logit_rows` (int32 [R]) names (in `logits_out` if that is given), or None if it is None or
        empty.  `after_layer(i, h)`, if given, is shown the residual stream behind every schedule entry (tests,
        inspection: every pending sum is then done at once)."""
        schedule = self.spec.schedule
        if getattr(self.embedding, "needs_context", False):
            own = len(cache_views) > len(schedule)
            h = self.embedding.forward(tokens, ctx, cache_views[len(schedule)] if own else None)
        else:
            h = self.embedding.forward(tokens)
        # a pass of a loop that is given the input again adds the embedding's output to the stream, or begins with a
        # part that reads both
        again = h.clone() if any(e.add_embedding or e.begins_pass is not None for e in schedule) else None
        if self.stream_sum is not None:
            h = begin_streams(h, self.spec.streams)
        normed = None
        for i, entry in enumerate(schedule):
            block = self.layers[entry.layer]
            if entry.add_embedding:
                if isinstance(normed, PendingNorm):
                    h = normed.settle()
                ops.residual_add_norm(again, h)
                normed = None
            if entry.begins_pass is not None:
                if isinstance(normed, PendingNorm):
                    h = normed.settle()
                h, normed = self.pass_input.forward(h, again, entry.begins_pass, ctx, block.first_norm())
            nxt = None
            if i + 1 < len(schedule) and not schedule[i + 1].add_embedding and schedule[i + 1].begins_pass is None:
                nxt = self.layers[schedule[i + 1].layer].first_norm()
            h, normed = block.forward(h, ctx, cache_views[i], normed, nxt)
            if after_layer is not None:
                if isinstance(normed, PendingNorm):
                    h = normed.settle()
                after_layer(i, h if self.stream_sum is None else self.stream_sum.plain(h))
        if logit_rows is None or logit_rows.numel() == 0:
            return None
        if self.stream_sum is not None:
            return self.head.forward(self.stream_sum.normed_rows(h, logit_rows, self.final_norm, ctx.dtype), out=logits_out)
        if isinstance(normed, PendingNorm):
            # the last block's residual sum is still pending: the final norm of the wanted rows comes out of the
            # same kernel (the residual stream itself is of no use to anyone after the last block)
            pending = PendingNorm(normed.residual, normed.y, normed.post_norm, self.final_norm, ctx.dtype)
            return self.head.forward(pending.rows_through(logit_rows), out=logits_out)
        rows = ops.gather_rows(h, logit_rows)
        return self.head.forward(PendingNorm(rows, None, None, self.final_norm, ctx.dtype), out=logits_out)
