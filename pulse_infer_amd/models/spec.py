"""An architecture written down as data.

A ``ModelSpec`` lists the layers of a decoder (each a choice of block
arrangement, mixer, feed-forward and norm, every one with its own sizes and
constants), the position encodings they refer to, and the order in which the
layers run.  The order is a list of ``RunSpec``: it may name a layer twice
(the weights are shared, each run has a cache of its own) or let a run read
the cache that an earlier run wrote.  Nothing in here knows which model it
describes; configuration classes produce it, ``CausalLM`` consumes it.
"""
from __future__ import annotations

from dataclasses import dataclass, field, replace
from typing import Any, Dict, List, Optional, Tuple


@dataclass(frozen=True)
class PartSpec:
    """One part: the registered kind and the parameters it is built with."""

    kind: str
    params: Dict[str, Any] = field(default_factory=dict)

    def __hash__(self) -> int:  # params are small, flat dictionaries
        return hash((self.kind, tuple(sorted((k, repr(v)) for k, v in self.params.items()))))


@dataclass(frozen=True)
class LayerSpec:
    """One decoder layer: which parts it is made of and where its weights are.

    ``norms`` names a norm for every place the block arrangement has one ("mixer_norm" and "ffn_norm" for the
    pre-norm block; another arrangement may name more): each is a ``PartSpec`` of its own, so the norms of a layer
    may differ in kind and in constants.  The block's parameters say under which tensor prefix each of them loads.
    """

    prefix: str
    mixer: PartSpec
    ffn: Optional[PartSpec]      # None: the layer has no feed-forward (for block arrangements that allow it)
    norms: Dict[str, PartSpec]
    block: PartSpec = field(default_factory=lambda: PartSpec("prenorm", {"mixer_norm": "input_layernorm",
                                                                         "ffn_norm": "post_attention_layernorm"}))

    def norm(self, place: str) -> PartSpec:
        try:
            return self.norms[place]
        except KeyError:
            raise KeyError(f"layer '{self.prefix}' names no norm for '{place}' (it has {sorted(self.norms)})") from None

    def with_parts(self, **changes: Any) -> "LayerSpec":
        """A copy with some of its fields replaced."""
        return replace(self, **changes)

    def __hash__(self) -> int:
        return hash((self.prefix, self.mixer, self.ffn, tuple(sorted(self.norms.items())), self.block))


@dataclass(frozen=True)
class RunSpec:
    """One entry of the execution order.

    ``layer`` indexes ``ModelSpec.layers``.  ``cache_of`` is the index (in the
    order) of an earlier run whose cache this run reads instead of owning one.
    ``offset`` = (tensor, row): that row of a tensor listed in ``ModelSpec.offsets`` is added to the residual of every
    token right before the run (the marker of a pass over layers that run several times).
    ``rejoin``: a tensor W listed in ``ModelSpec.rejoins``; before the run (and before its offset) the residual x becomes
    W [x; x0], x0 the residual as the embedding left it.
    """

    layer: int
    cache_of: Optional[int] = None
    offset: Optional[Tuple[str, int]] = None
    rejoin: Optional[str] = None


@dataclass
class ModelSpec:
    architecture: str
    vocab_size: int
    hidden_size: int
    max_positions: int
    embedding: PartSpec
    layers: List[LayerSpec]
    order: List[RunSpec]
    final_norm: PartSpec
    head: PartSpec
    final_norm_prefix: str = "model.norm"
    # position encodings by name; mixers refer to them through params["position"]
    positions: Dict[str, PartSpec] = field(default_factory=dict)
    # rows of the residual a token (hyper-connections keep several streams); the embedding fills them all, blocks and
    # the final norm must be of kinds that read that many
    streams: int = 1
    # tensors [rows, hidden_size] whose rows runs add to the residual (``RunSpec.offset``): name -> rows
    offsets: Dict[str, int] = field(default_factory=dict)
    # tensors [hidden_size, 2 hidden_size] through which runs bring the embedding's output back into the residual
    # (``RunSpec.rejoin``)
    rejoins: List[str] = field(default_factory=list)

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a model needs at least one layer")
        if self.streams < 1:
            raise ValueError(f"a residual has at least one stream, got {self.streams}")
        for index, run in enumerate(self.order):
            if not 0 <= run.layer < len(self.layers):
                raise ValueError(f"order[{index}] names layer {run.layer}, the model has {len(self.layers)}")
            if run.offset is not None:
                name, row = run.offset
                if name not in self.offsets or not 0 <= row < self.offsets[name]:
                    raise ValueError(f"order[{index}].offset names row {row} of '{name}', the model lists {self.offsets}")
                if self.streams != 1:
                    raise ValueError("offsets are added to a residual of one stream")
            if run.rejoin is not None:
                if run.rejoin not in self.rejoins:
                    raise ValueError(f"order[{index}].rejoin names '{run.rejoin}', the model lists {self.rejoins}")
                if self.streams != 1:
                    raise ValueError("the embedding's output is brought back into a residual of one stream")
            if run.cache_of is not None:
                if not 0 <= run.cache_of < index:
                    raise ValueError(f"order[{index}].cache_of must name an earlier run, got {run.cache_of}")
                if self.order[run.cache_of].cache_of is not None:
                    raise ValueError(f"order[{index}].cache_of names run {run.cache_of}, which owns no cache")
