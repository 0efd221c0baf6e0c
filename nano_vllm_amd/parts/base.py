"""What every part is: a holder of named parameters with a forward method.

A part declares its parameters (local name -> ParamDecl); the model allocates them, the
loader fills them by checkpoint tensor name, and the part reads them from self.weights.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Mapping, Optional, Tuple

import torch


@dataclass(frozen=True)
class Source:
    """A checkpoint tensor that fills rows [row, row + rows) of a parameter."""
    name: str                 # name below the part's prefix, e.g. "q_proj.weight"
    row: int
    rows: int


@dataclass(frozen=True)
class ParamDecl:
    shape: Tuple[int, ...]
    # "model": the model's element type; "stored32": float32 if the checkpoint stores float32,
    # else the model's element type; "float32"; "int32" (integer tables)
    dtype: str = "model"
    # None: one tensor of the parameter's own name.  Rows that no source fills are zero (a packed matrix whose
    # product should have rows of a whole number of vectors).
    sources: Optional[Tuple[Source, ...]] = None
    init: str = "normal"                             # random-weights mode: "normal" | "norm"
    # A size of -1 in `shape` is one that the checkpoint's tensor decides (a rank that no configuration
    # names); default_shape then says what random-weights mode draws.  Only for parameters of one source.
    default_shape: Optional[Tuple[int, ...]] = None

    def fits(self, shape) -> bool:
        return len(shape) == len(self.shape) and all(w == -1 or w == g for w, g in zip(self.shape, shape))

    @property
    def drawn_shape(self) -> Tuple[int, ...]:
        """The shape random-weights mode gives the parameter."""
        if -1 not in self.shape:
            return tuple(self.shape)
        if self.default_shape is None or not self.fits(self.default_shape):
            raise ValueError(f"a parameter of shape {self.shape} needs a default shape for its free sizes")
        return tuple(self.default_shape)


@dataclass
class NormedAddend:
    """A sublayer's output on its way into a float32 residual stream through a norm of its own:
    the stream takes mult * x / sqrt(mean(x^2) + eps) * weight.  The norm that follows (the next
    sublayer's, or the model's last) adds it while it reads the stream, in the same pass."""
    x: object                         # [rows, width] of the element type (or a product left as partial sums)
    weight: torch.Tensor              # [width]
    eps: float
    mult: float = 1.0
    offset: float = 0.0               # the factor is (offset + weight): 1 for a weight that is stored around zero


@dataclass
class ScaledPair:
    """left_scale * left + right_scale * right, left to the norm that takes it (alone in a NormedAddend) to add up while it
    reads the two; `tensor()` gives the finished sum."""
    left: object                      # [rows, width] of the element type (or a product left as partial sums)
    right: object
    left_scale: float
    right_scale: float
    kernels: object

    def tensor(self) -> torch.Tensor:
        return self.kernels.pair_scaled_sum(self.left, self.left_scale, self.right, self.right_scale)


@dataclass
class StreamAddend:
    """A float32 tensor [rows, width] that enters a float32 residual stream as it is, beside a NormedAddend."""
    x: torch.Tensor


@dataclass
class ScaledAddend:
    """A sublayer's output on its way into a float32 residual stream through a learned vector: the stream
    takes x * scale, channel by channel (layer scale).  The norm that follows adds it while it reads the stream."""
    x: object                         # [rows, width] of the element type (or a product left as partial sums)
    scale: torch.Tensor               # [width]


@dataclass
class BuildContext:
    """What a part may use while it is built."""
    kernels: object                   # the operations (kernels.ops.HipKernels or a stand-in of the same methods)
    device: torch.device
    dtype: torch.dtype                # the model's element type
    hidden_size: int
    max_position: int
    position_encodings: Dict[str, object] = field(default_factory=dict)
    tables: Dict[str, object] = field(default_factory=dict)           # the model's shared tables of the tokens


class Part:
    """Base of mixers, feed-forwards, norms, position encodings and blocks."""

    # A mixer with per-request state says True when its forward, for a step of single tokens,
    # reads the step's metadata on the device only (batch.state_slots, batch.seq_starts, ... as
    # tensors; no .tolist() or .item(), nothing decided on the host from their values): such a step
    # can be captured once and replayed for other requests.  Rows that pad a captured batch carry a
    # state slot of their own that no request holds (the state tensors' last row).
    replays_state_steps = False

    # The kernel modules (kernels.build.MODULES) this part calls beyond those every model calls
    # (rows, norms, products, gating): they are compiled together before the model's first step.
    # What a part calls without naming it here is compiled when first called.
    kernel_modules: Tuple[str, ...] = ()

    def __init__(self, params: Mapping, build: BuildContext):
        self.params = dict(params)
        self.kernels = build.kernels
        self.weights: Dict[str, torch.Tensor] = {}

    def param_decls(self) -> Dict[str, ParamDecl]:
        return {}

    def children(self) -> Dict[str, "Part"]:
        """Sub-parts, by the name under which their parameters appear."""
        return {}

    def on_weights_loaded(self) -> None:
        """Called once every parameter is filled (derived tensors are made here)."""


def named_params(part: Part, prefix: str) -> List[Tuple[str, Part, str, ParamDecl]]:
    """(full parameter name, owner, local name, declaration) of a part and its sub-parts."""
    out = []
    for local, decl in part.param_decls().items():
        out.append((f"{prefix}.{local}" if prefix else local, part, local, decl))
    for name, child in part.children().items():
        out.extend(named_params(child, f"{prefix}.{name}" if prefix and name else (prefix or name)))
    return out
