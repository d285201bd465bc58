"""Operations on the residual stream between layers (a model's run order may name one in front of
a layer call).  ``forward(hidden, pending, first) -> hidden``: ``pending`` are branch outputs not
yet added to the stream, ``first`` is the stream as the embedding left it (in the products' type, or with
``first_in_stream_type`` in the stream's).  An operation with ``defers`` is asked for ``defer(hidden, delta,
first) -> (hidden, delta)`` instead: it may leave its work to whoever reads the stream next."""
from __future__ import annotations

import dataclasses
from typing import Dict, Optional

import torch

from ..config.registry import STREAM_OPS
from ..models.spec import TensorSpec
from ..ops import kernels as K
from .base import Part, PendingNorm
from .linear import Linear


@STREAM_OPS.register("reinject")
class Reinject(Part):
    """``h <- W [h ; h0]``: the stream joined with the embedding output and projected back to its
    width (``W`` is ``[width, 2 width]``, the stream's columns first).  The product takes the
    weights' type; its result goes into the stream in the stream's type."""

    graph_safe = True

    def __init__(self, prefix: str = "", *, width: int, weight_name: str = "weight"):
        super().__init__(prefix)
        self.width = int(width)
        self.weight_name = prefix + weight_name
        self.linear: Optional[Linear] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.weight_name: TensorSpec((self.width, 2 * self.width))}

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.linear = Linear(tensors[self.weight_name])

    def activation_elements(self) -> int:
        return 3 * self.width

    def forward(self, hidden: torch.Tensor, pending, first: torch.Tensor) -> torch.Tensor:
        joined = torch.empty((hidden.shape[0], 2 * self.width), dtype=self.linear.weight.dtype, device=hidden.device)
        K.stream_join(hidden, first, joined, deltas=pending)
        return self.linear(joined, out=hidden)


@STREAM_OPS.register("add_first")
class AddFirst(Part):
    """``h <- h + h0``: the embedding output added to the stream, both in 32-bit.  A branch output that is still to
    enter under a norm takes it along (:class:`~.base.PendingNorm`): the sum is made in the pass that reads the
    stream next, and the operation costs no launch of its own."""

    graph_safe = True
    defers = True
    first_in_stream_type = True

    def __init__(self, prefix: str = ""):
        super().__init__(prefix)

    def defer(self, hidden: torch.Tensor, delta, first: torch.Tensor):
        if hidden.dtype != torch.float32:
            raise TypeError("the embedding output is added to a stream kept in 32-bit")
        if isinstance(delta, PendingNorm) and delta.addend is None:
            return hidden, dataclasses.replace(delta, addend=first)
        outputs = () if delta is None else (tuple(delta) if isinstance(delta, (tuple, list)) else (delta,))
        if getattr(delta, "scale", 1.0) != 1.0 or not all(isinstance(d, torch.Tensor) for d in outputs):
            raise TypeError("pending branch outputs are added as they are here, or under their norm")
        for y in outputs:
            K.sandwich_step(hidden, y=y)
        K.sandwich_step(hidden, addend=first)
        return hidden, None
