"""A model as data: which parts make up each layer, with their sizes and constants, and
the order in which layers run.

An architecture's definition (models/*.py) turns its typed configuration into a ModelSpec;
parts.model.Model builds the parts a ModelSpec names from the part registries.  Nothing in
a part names the model it is in.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Mapping, Optional, Tuple


@dataclass(frozen=True)
class PartSpec:
    """One part: its kind (a name in the registry of its role) and its parameters."""
    kind: str
    params: Mapping[str, Any] = field(default_factory=dict)

    def get(self, key, default=None):
        return self.params.get(key, default)

    def __getitem__(self, key):
        return self.params[key]


@dataclass(frozen=True)
class LayerSpec:
    """One layer with weights of its own.

    block     how the parts below are arranged (a kind in the block registry)
    parts     role -> PartSpec; the roles a block knows ("mixer", "feed_forward",
              "mixer_norm", "feed_forward_norm" for the pre-norm residual block)
    name      the layer's prefix in checkpoint tensor names ("model.layers.3")
    names     role -> the part's name below that prefix ("self_attn", "mlp", ...)
    """
    block: PartSpec
    parts: Mapping[str, PartSpec]
    name: str
    names: Mapping[str, str]


@dataclass(frozen=True)
class LayerRun:
    """One entry of the execution order.

    layer     index into ModelSpec.layers: whose weights run.  A layer may be named twice.
    cache_of  None: the run has a cache of its own.  An index of an earlier entry of the
              order: the run reads that entry's cache and writes none.
    add_embedding  the embedding's output (as it was before the first entry) is added to the residual
              stream before the run: the start of a pass over layers that run several times.
    """
    layer: int
    cache_of: Optional[int] = None
    add_embedding: bool = False


@dataclass(frozen=True)
class ModelSpec:
    architecture: str
    hidden_size: int
    vocab_size: int
    max_position: int
    dtype: str                                   # "bfloat16" | "float32": config.json's
    embedding: PartSpec                          # params: name
    layers: Tuple[LayerSpec, ...]
    order: Tuple[LayerRun, ...]
    final_norm: PartSpec                         # params: name + the norm's own
    head: PartSpec                               # params: name, tied
    position_encodings: Mapping[str, PartSpec]   # shared by name among the mixers
    tables: Mapping[str, PartSpec] = field(default_factory=dict)     # params: name + the table's own; shared by name among the layers
    eos_token_ids: Tuple[int, ...] = ()
    # How the checkpoint names its tensors where that is not "<part>.<parameter>": pairs (suffix,
    # replacement) tried in turn on every derived name, the first that fits is applied
    # ((".weight", "") for a checkpoint that calls a matrix by its part's name alone).
    checkpoint_names: Tuple[Tuple[str, str], ...] = ()

    def checkpoint_name(self, derived: str) -> str:
        for suffix, replacement in self.checkpoint_names:
            if derived.endswith(suffix):
                return derived[: len(derived) - len(suffix)] + replacement
        return derived

    def validate(self) -> None:
        if self.order and self.order[0].add_embedding:
            raise ValueError("order[0] adds the embedding, which is what the stream holds before it")
        for i, run in enumerate(self.order):
            if not 0 <= run.layer < len(self.layers):
                raise ValueError(f"order[{i}] names layer {run.layer}; there are {len(self.layers)}")
            if run.cache_of is not None:
                if not 0 <= run.cache_of < i:
                    raise ValueError(f"order[{i}] reads the cache of entry {run.cache_of}, which must run earlier")
                if self.order[run.cache_of].cache_of is not None:
                    raise ValueError(f"order[{i}] reads the cache of entry {run.cache_of}, which has none of its own")


# ---------------------------------------------------------------------------- cache needs
@dataclass(frozen=True)
class PagedKV:
    """Keys and values of every token, in pages.  window None: all keys stay; an integer:
    a query at position p reads positions > p - window only, and pages wholly before that
    are given back.  chunk: a query at position p reads positions >= floor(p / chunk) * chunk only
    (the sequence is cut into chunks counted from its position 0, and no query looks out of its
    own); pages wholly before the chunk of the next query are given back.  v_head_dim: the size of
    a head's values where it is not head_dim.  keep_first (with a window): every query also reads
    the first keep_first positions of its sequence, whose pages are never given back."""
    num_kv_heads: int
    head_dim: int
    window: Optional[int] = None
    v_head_dim: Optional[int] = None
    chunk: Optional[int] = None
    keep_first: int = 0

    @property
    def value_dim(self) -> int:
        return self.head_dim if self.v_head_dim is None else self.v_head_dim


@dataclass(frozen=True)
class FixedState:
    """State of fixed size per request, kept in a slot: name -> (shape, dtype name)."""
    tensors: Mapping[str, Tuple[Tuple[int, ...], str]]


@dataclass(frozen=True)
class CombinedNeed:
    """What a run needs whose mixer is made of several: each part's need, in the parts' order.  At
    most one of them may be paged keys and values and at most one fixed state (the run's LayerCache
    has one place for each)."""
    parts: Tuple[Any, ...]

    def __post_init__(self):
        paged = [p for p in self.parts if isinstance(p, PagedKV)]
        fixed = [p for p in self.parts if isinstance(p, FixedState)]
        if len(paged) > 1 or len(fixed) > 1 or len(paged) + len(fixed) != len(self.parts):
            raise ValueError("a combined cache need holds at most one PagedKV and one FixedState")


def paged_need(need):
    """The PagedKV of a need (its own, or the one inside a combined need), else None."""
    for part in getattr(need, "parts", (need,)):
        if hasattr(part, "num_kv_heads"):
            return part
    return None


def state_need(need):
    """The FixedState of a need (its own, or the one inside a combined need), else None."""
    for part in getattr(need, "parts", (need,)):
        if hasattr(part, "tensors"):
            return part
    return None
