"""The decoder that every architecture is an instance of: embedding, a schedule
of layer calls, final norm, output head.

The schedule is a list. An entry names a layer and may name it again (the same
weights run twice, each call with a cache entry of its own), or may read the
cache entry of an earlier call instead of owning one. Before an entry the stream may be made anew
from what it holds and what it began with (the beginning of a pass of layers that run several times).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from ..parts.base import Block, CacheNeeds, Norm, Runtime, WeightSpec
from ..parts.embedding import Embedding, OutputHead


@dataclass(frozen=True)
class LayerCall:
    """One entry of the schedule: run `layer`; keep its keys/values/state in the
    cache entry of this call, or read (not write) the entry of call `reads_cache_of`. enters: a pass begins with this
    call, and the model's `entry` comes before it."""
    layer: int
    reads_cache_of: Optional[int] = None
    enters: bool = False


@dataclass
class ModelSpec:
    config: object
    embedding: Embedding
    layers: List[Block]
    final_norm: Norm
    head: OutputHead
    schedule: Optional[List[LayerCall]] = None
    streams: Optional[object] = None        # a residual stream in several copies (parts/block.py: ResidualStreams), or None for one
    entry: Optional[object] = None          # what comes before the calls that begin a pass (parts/block.py: PassEntry)

    def __post_init__(self):
        if self.schedule is None:
            self.schedule = [LayerCall(i) for i in range(len(self.layers))]
        if self.entry is not None and self.streams is not None:
            raise ValueError("passes are entered on one residual stream, not on copies of it")
        for index, call in enumerate(self.schedule):
            if call.enters and self.entry is None:
                raise ValueError(f"schedule entry {index} begins a pass, and the model has no entry for it")
            if not 0 <= call.layer < len(self.layers):
                raise ValueError(f"schedule entry {index} names layer {call.layer} of {len(self.layers)}")
            if call.reads_cache_of is not None:
                source = call.reads_cache_of
                if not 0 <= source < index:
                    raise ValueError(f"schedule entry {index} reads the cache of entry {source}, "
                                     "which must be an earlier entry")
                if self.schedule[source].reads_cache_of is not None:
                    raise ValueError(f"schedule entry {index} reads the cache of entry {source}, "
                                     "which owns none")
                if (self.layers[call.layer].cache_needs()
                        != self.layers[self.schedule[source].layer].cache_needs()):
                    raise ValueError(f"schedule entry {index} reads the cache of entry {source}, "
                                     "whose layer keeps something else")

    def parts(self):
        return [self.embedding, *self.layers, self.final_norm, self.head] + ([self.streams] if self.streams is not None else []) + (
            [self.entry] if self.entry is not None else [])

    def weight_specs(self) -> Dict[str, WeightSpec]:
        specs: Dict[str, WeightSpec] = {}
        for part in self.parts():
            for name, spec in part.weight_specs().items():
                if name in specs and specs[name] != spec:
                    raise ValueError(f"tensor {name} is declared twice with different shapes")
                specs[name] = spec
        return specs

    def capturable(self) -> bool:
        """Whether a decode step of this model can be recorded as a graph and replayed."""
        return all(part.capturable for part in self.parts())

    def ignored_names(self) -> List[str]:
        """Tensors that a checkpoint may carry and that no part reads."""
        return [name for part in self.parts() for name in getattr(part, "ignored_names", lambda: [])()]

    def cache_needs(self) -> List[Optional[CacheNeeds]]:
        """For each schedule entry what its cache entry holds, None if it reads another's; then, if the embedding keeps
        something per sequence (`keeps_state`), one more entry for it."""
        needs = [None if call.reads_cache_of is not None else self.layers[call.layer].cache_needs()
                 for call in self.schedule]
        if getattr(self.embedding, "keeps_state", False):
            needs.append(self.embedding.cache_needs())
        return needs

    def cache_sources(self) -> List[int]:
        """For each entry of `cache_needs` the entry whose storage it reads: itself, unless the schedule says otherwise."""
        sources = [index if call.reads_cache_of is None else call.reads_cache_of for index, call in enumerate(self.schedule)]
        if getattr(self.embedding, "keeps_state", False):
            sources.append(len(sources))
        return sources


class DecoderModel:
    """A ModelSpec with its weights bound: runs the tokens of one step."""

    def __init__(self, spec: ModelSpec, tensors: Dict[str, torch.Tensor], runtime: Runtime):
        self.spec = spec
        self.config = spec.config
        self.runtime = runtime
        for part in spec.parts():
            part.bind(tensors, runtime)

    def _first_reads_stream(self) -> bool:
        """Whether the first block reads the stream itself in the compute dtype and the embedding can hand it that beside the stream."""
        spec = self.spec
        first = spec.layers[spec.schedule[0].layer]
        reads = first.first_norm() if getattr(first, "passes_norms", False) else None
        return (getattr(reads, "reads_stream", False) and spec.streams is None and not spec.schedule[0].enters and self.runtime.dtype != torch.float32
                and getattr(spec.embedding, "norm_name", None) is not None)

    def forward(self, batch, cache) -> torch.Tensor:
        """Logits [len(batch.logit_rows), vocab] in float32 for the tokens of `batch`."""
        spec = self.spec
        h = None            # what the next block reads first (its first norm of x), where the part before it has made it already
        if getattr(spec.embedding, "keeps_state", False):       # its cache entry follows the schedule's
            x = spec.embedding.forward_step(batch, cache.layer_cache(len(spec.schedule)))
        elif self._first_reads_stream():
            h = self.runtime.empty((batch.n_tokens, spec.embedding.hidden))
            x = spec.embedding.forward_copied(batch.token_ids, batch.positions, h)
        else:
            x = spec.embedding.forward(batch.token_ids, batch.positions)
        if spec.streams is not None:                             # the blocks then work on the copies [tokens, copies, hidden]
            x = spec.streams.open(x)
        opened = spec.entry.open(x) if spec.entry is not None else None      # (before any layer: the stream still is what the embedding left)
        for index, call in enumerate(spec.schedule):
            block = spec.layers[call.layer]
            if call.enters:
                spec.entry.forward(x, opened)
            if not getattr(block, "passes_norms", False):
                block.forward(x, batch, cache.layer_cache(index))
                h = None
                continue
            last = index + 1 == len(spec.schedule) or spec.schedule[index + 1].enters      # (what follows does not read the stream as this block leaves it)
            after = None if last else spec.layers[spec.schedule[index + 1].layer]
            then = after.first_norm() if after is not None and getattr(after, "passes_norms", False) else None
            h = block.forward(x, batch, cache.layer_cache(index), h=h, then=then)
        if batch.n_logit_rows == 0:
            return self.runtime.empty((0, spec.head.vocab), torch.float32, outlives_the_step=True)
        if spec.streams is not None:
            y = spec.streams.close(x, spec.final_norm, rows=batch.logit_rows)
        else:
            y = spec.final_norm.forward(x, rows=batch.logit_rows)
        return spec.head.forward(y)
