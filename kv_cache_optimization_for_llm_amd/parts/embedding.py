"""How a step's tokens become the first rows of the residual stream, where that is more than a gather.

:class:`TokenPairEmbedding` (``"token_pairs"``): a token's row of the token table times a constant, plus a row of a
second table that the token and the one before it pick together, ``row = (previous * mul_prev + token * mul_cur) mod
buckets`` (a sequence's first token takes the table's last row, number ``buckets``), under a norm.  The previous token
is part of a request's state: a portion of a prompt and a decoded token find it where the step before left it.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..config.registry import EMBEDDINGS, NORMS
from ..models.spec import PartSpec, TensorSpec
from ..ops import kernels as K
from .base import Embedding, StateSpec


@EMBEDDINGS.register("token_pairs")
class TokenPairEmbedding(Embedding):
    graph_safe = True

    def __init__(self, prefix: str = "", *, vocab_size: int, width: int, table_name: str, scale: float = 1.0,
                 pair_name: Optional[str] = None, buckets: int = 0, mul_prev: int = 0, mul_cur: int = 0,
                 norm: Optional[PartSpec] = None):
        """``pair_name``: the second table, ``[buckets + 1, width]`` (None: there is none).  ``norm``: a norm of kind
        ``"dynamic_tanh"`` (it runs inside the same pass) or None."""
        super().__init__(prefix)
        self.vocab_size, self.width, self.scale = int(vocab_size), int(width), float(scale)
        self.table_name, self.pair_name = prefix + table_name, None if pair_name is None else prefix + pair_name
        self.buckets, self.mul_prev, self.mul_cur = int(buckets), int(mul_prev), int(mul_cur)
        if self.pair_name is not None and (self.buckets < 1 or self.mul_prev < 0 or self.mul_cur < 0):
            raise ValueError(f"{self.pair_name}: at least one row beside the last, multipliers that are not negative")
        self.norm = None if norm is None else NORMS.get(norm.kind)(**norm.params)
        if self.norm is not None and getattr(self.norm, "pass_kind", None) != "tanh":
            raise ValueError(f"the embedding's pass runs a norm of kind 'dynamic_tanh', not a {type(self.norm).__name__}")
        self.table: Optional[torch.Tensor] = None
        self.pairs: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        specs = {self.table_name: TensorSpec((self.vocab_size, self.width))}
        if self.pair_name is not None:
            specs[self.pair_name] = TensorSpec((self.buckets + 1, self.width))
        if self.norm is not None:
            specs.update(self.norm.tensor_specs())
        return specs

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.table = tensors[self.table_name]
        self.pairs = None if self.pair_name is None else tensors[self.pair_name]
        if self.norm is not None:
            self.norm.load(tensors)

    def state_spec(self) -> StateSpec:
        return StateSpec((1,), torch.int32)         # the last token's id plus one (0: a fresh seat)

    def forward(self, batch, out: torch.Tensor, state: Optional[torch.Tensor] = None) -> torch.Tensor:
        if out.dtype != torch.float32 or state is None:
            raise TypeError("an embedding of token pairs fills a stream kept in 32-bit and keeps a state per request")
        return K.pair_embed(out, self.table, self.scale, self.pairs, self.mul_prev, self.mul_cur,
                            self.norm.pass_args() if self.norm is not None else None, batch.token_ids, state,
                            batch.entry_q_start, batch.entry_seat, getattr(batch, "feedback", None))
