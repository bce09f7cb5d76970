"""Architecture-neutral description of a decoder: what the parts are and in which
order they run.  An architecture's typed configuration (for instance
`Gemma2Config`) is turned into a `ModelSpec`; everything below the configuration
(model, cache manager, step function) reads only the `ModelSpec`.

The layer pattern follows simply/model_lib.py:2839-2844 (each block gets its kind
from a pattern) but as data: every layer carries its own part specs, and the order
in which layers run is a list of `ScheduleEntry`, which may name a layer twice or
let an entry read the cache that an earlier entry wrote.
"""
from __future__ import annotations

import dataclasses
from typing import Any, Mapping


@dataclasses.dataclass(frozen=True)
class PartSpec:
    """One part: `kind` is a name in the part's registry, `params` are its sizes and
    constants, `tensors` maps the part's own parameter names to tensor names in the
    model folder."""

    kind: str
    params: Mapping[str, Any] = dataclasses.field(default_factory=dict)
    tensors: Mapping[str, str] = dataclasses.field(default_factory=dict)


@dataclasses.dataclass(frozen=True)
class LayerSpec:
    """A block: an arrangement (`block.kind`) of a mixer, a feed-forward (None: the layer has none, for block
    arrangements that allow it) and norms."""

    block: PartSpec
    mixer: PartSpec
    feed_forward: "PartSpec | None"
    norms: Mapping[str, PartSpec] = dataclasses.field(default_factory=dict)
    #: parts that update the residual stream themselves at the block's end (registry STREAM_PARTS), in their order
    extras: "tuple[PartSpec, ...]" = ()


@dataclasses.dataclass(frozen=True)
class ScheduleEntry:
    """Run layer `layer` (a layer may be named by several entries: each has a cache or state of its own).  `cache_from` names an earlier schedule entry (by its index
    in the schedule) whose cache this entry reads instead of keeping its own."""

    layer: int
    cache_from: int | None = None
    #: the embedding's output of this step is added to the residual stream before this entry runs (a pass of a loop
    #: over layers that is given the input again)
    add_embedding: bool = False
    #: the number of the pass of a loop over layers that begins with this entry: the model's `pass_input` part is run on
    #: the stream before it (None: no pass begins here)
    begins_pass: int | None = None


@dataclasses.dataclass(frozen=True)
class ModelSpec:
    architecture: str
    hidden_size: int
    vocab_size: int
    embedding: PartSpec
    layers: tuple[LayerSpec, ...]
    schedule: tuple[ScheduleEntry, ...]
    final_norm: PartSpec
    head: PartSpec
    max_position: int
    eos_token_ids: tuple[int, ...] = ()
    initializer_range: float = 0.02
    #: tensor names that a model folder may hold beside the expected ones, each with the expected tensor whose
    #: copy it must be (a tied head stored once more under its own name): checked for equality, then left unread
    copies: Mapping[str, str] = dataclasses.field(default_factory=dict)
    #: tensor names that a model folder may hold and that the model does not read (norms around a feed-forward that
    #: a layer does not have)
    ignorable: tuple[str, ...] = ()
    #: what is done to the stream before every pass of a loop (registry PASS_INPUTS), for entries with `begins_pass`
    pass_input: "PartSpec | None" = None
    #: None: the residual is one row per token; n: every token has n parallel streams, all equal to the embedding's output
    #: at the start and summed at the end (every layer's block arrangement is then one of streams)
    streams: "int | None" = None

    def validate(self) -> None:
        n = len(self.layers)
        for i, e in enumerate(self.schedule):
            if not 0 <= e.layer < n:
                raise ValueError(f"schedule entry {i} names layer {e.layer}, but there are {n} layers")
            if e.cache_from is not None:
                if not 0 <= e.cache_from < i:
                    raise ValueError(
                        f"schedule entry {i} reads the cache of entry {e.cache_from}, which does not run before it")
                if self.schedule[e.cache_from].cache_from is not None:
                    raise ValueError(
                        f"schedule entry {i} reads the cache of entry {e.cache_from}, which itself has none")
        if self.pass_input is None and any(e.begins_pass is not None for e in self.schedule):
            raise ValueError("a schedule entry begins a pass, but the model has no pass input")
        if self.streams is not None:
            if self.streams < 1 or any(l.block.params.get("streams") != self.streams for l in self.layers):
                raise ValueError(f"a residual of {self.streams} streams: every layer's block arrangement takes as many")
            if any(e.begins_pass is not None or e.add_embedding for e in self.schedule):
                raise ValueError("a residual of several streams has no passes that are given the embedding again")
        elif any("streams" in l.block.params for l in self.layers):
            raise ValueError("a block arrangement of streams needs a model with streams")
        for name, of in self.copies.items():
            if name == of:
                raise ValueError(f"tensor {name!r} is declared a copy of itself")
