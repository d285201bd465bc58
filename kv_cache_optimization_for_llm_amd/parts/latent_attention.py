"""Attention over a low-rank key/value entry (latent attention).

Per token the cache holds ONE row for all heads: a latent vector ``c`` of ``rank`` elements (the
down-projected input, RMS-normed with a weight) and a rotated key part ``k_r`` of ``rot_dim``
elements that every head shares.  Head ``h`` has an unrotated key ``U_k[h] c``, a value
``U_v[h] c`` and a query ``[q_p[h] ; q_r[h]]`` (``dim`` unrotated and ``rot_dim`` rotated
elements):

    score_h(i, j) = (q_p[h]_i . U_k[h] c_j + q_r[h]_i . k_r_j) * scale
    out_h(i)      = sum_j p_h(i, j) U_v[h] c_j

Keys and values are never expanded.  The key expansion moves to the query side,
``q_p . U_k c = (U_k^T q_p) . c``, so a head's query becomes a row ``[U_k[h]^T q_p[h] ; q_r[h]]`` of
the cache's own layout and every head attends over the same rows (one shared "kv head" of
``rank + rot_dim`` elements whose first ``rank`` are also the value); the value expansion moves
behind the attention, ``sum_j p U_v c_j = U_v (sum_j p c_j)``.  What a step costs per cached token
is then independent of the number of heads' key and value sizes, and a prompt cut anywhere
continues from the rows alone.

Options: queries through a latent of their own (``c_q = RMSnorm(W_dq x)``, ``q = W_uq c_q``), a softmax sink
per head (``exp(sink_h)`` added to the denominator; no key, no value, not scaled), a sigmoid output
gate read from the mixer's input (one number a head, or one an element of the concatenated heads), a
window with kept first positions.  Softmax, the latents' norms and the rotation are fp32.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..config.registry import MIXERS, POSITION_ENCODINGS
from ..models.spec import PartSpec, TensorSpec
from ..ops import kernels as K
from ..ops import latent_attention as lat_ops
from .base import CacheArray, KVCacheSpec, Mixer, MixerContext, NormedRows
from .linear import Linear


def latent_cache_spec(rank: int, rot_dim: int, kind: str = "full", window: int = 0, keep_first: int = 0) -> KVCacheSpec:
    """One row ``[latent (rank) ; rotated key part (rot_dim)]`` per token, pages ``[page_size, rank + rot_dim]``."""
    arrays = (CacheArray("latent", (int(rank) + int(rot_dim),), token_axis=0),)
    return KVCacheSpec(arrays, kind, int(window), int(keep_first) if kind == "window" else 0)


@MIXERS.register("latent_attention")
class LatentAttention(Mixer):
    graph_safe = True

    def __init__(self, prefix: str, *, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int,
                 value_dim: int, rank: int, scale: float, norm_eps: float, position: PartSpec, sink: bool = False,
                 gate=False, window: int = 0, keep_first: int = 0, q_rank: int = 0,
                 tensor_names: Optional[Dict[str, str]] = None):
        """``head_dim``: unrotated query/key elements per head; ``rot_dim``: rotated ones (the
        ``position`` encoding must rotate exactly these); ``rank``: size of the latent.
        ``q_rank`` > 0: queries come from a latent of that size, normed with a weight and ``norm_eps``.
        ``gate``: False, True or "head" (one number a head), "element" (one an element of the concatenated heads).
        ``tensor_names`` maps ``q`` (with ``q_rank``: the matrix behind the latent), ``q_down``, ``q_norm``,
        ``down``, ``down_norm``, ``up_k``, ``up_v``, ``sink``, ``gate``, ``o`` to the tensors' names behind ``prefix``."""
        super().__init__(prefix)
        self.hidden_size, self.num_heads, self.head_dim = int(hidden_size), int(num_heads), int(head_dim)
        self.rot_dim, self.value_dim, self.rank = int(rot_dim), int(value_dim), int(rank)
        self.scale, self.norm_eps = float(scale), float(norm_eps)
        if gate not in (False, True, "head", "element"):
            raise ValueError(f"{prefix}: gate {gate!r} is not one of False, 'head', 'element'")
        self.has_sink, self.has_gate, self.gate_elements = bool(sink), bool(gate), gate == "element"
        self.q_rank = int(q_rank)
        self.window = int(window)
        self.keep_first = int(keep_first) if self.window > 0 else 0
        names = dict(q="q_proj.weight", q_down="q_down.weight", q_norm="q_norm.weight", down="kv_down.weight", down_norm="kv_norm.weight", up_k="k_up.weight",
                     up_v="v_up.weight", sink="sinks", gate="gate.weight", o="o_proj.weight")
        names.update(tensor_names or {})
        self.names = {key: prefix + name for key, name in names.items()}
        self.position = POSITION_ENCODINGS.get(position.kind)(**position.params)
        if getattr(self.position, "rotary_dim", None) != self.rot_dim or getattr(self.position, "unit_norm_eps", None) is not None:
            raise ValueError("latent attention needs a rotary encoding over exactly its rot_dim elements")
        self.key_dim = self.rank + self.rot_dim
        self.proj: Optional[Linear] = None          # [q or its latent ; down ; gate] joined
        self.q_up: Optional[Linear] = None          # the queries from their latent
        self.o: Optional[Linear] = None
        self.up_k_t = self.up_v = self.norm_weight = self.q_norm_weight = self.sinks = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        n, H, W = self.names, self.num_heads, self.hidden_size
        specs = {
            n["q"]: TensorSpec((H * (self.head_dim + self.rot_dim), self.q_rank or W)),
            n["down"]: TensorSpec((self.key_dim, W)),
            n["down_norm"]: TensorSpec((self.rank,), init="norm", role="vector"),
            n["up_k"]: TensorSpec((H * self.head_dim, self.rank)),
            n["up_v"]: TensorSpec((H * self.value_dim, self.rank)),
            n["o"]: TensorSpec((W, H * self.value_dim)),
        }
        if self.q_rank:
            specs[n["q_down"]] = TensorSpec((self.q_rank, W))
            specs[n["q_norm"]] = TensorSpec((self.q_rank,), init="norm", role="vector")
        if self.has_sink:
            specs[n["sink"]] = TensorSpec((H,), init="normal", role="vector")
        if self.has_gate:
            specs[n["gate"]] = TensorSpec((self._gates(), W))
        return specs

    def _gates(self) -> int:
        return self.num_heads * (self.value_dim if self.gate_elements else 1)

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        n, H = self.names, self.num_heads
        mats = [tensors[n["q_down" if self.q_rank else "q"]], tensors[n["down"]]] + ([tensors[n["gate"]]] if self.has_gate else [])
        if len({m.dtype for m in mats}) != 1:
            raise ValueError(f"{self.prefix}: the input projections are stored in different dtypes")
        self.proj = Linear(torch.cat(mats, dim=0))
        self.kv_off = self.q_rank or H * (self.head_dim + self.rot_dim)
        self.gate_off = self.kv_off + self.key_dim
        self.q_up = Linear(tensors[n["q"]]) if self.q_rank else None
        self.q_norm_weight = tensors[n["q_norm"]].contiguous() if self.q_rank else None
        self.o = Linear(tensors[n["o"]])
        # U_k per head, transposed: the query-side product reads [heads, rank, dim]
        self.up_k_t = tensors[n["up_k"]].view(H, self.head_dim, self.rank).transpose(1, 2).contiguous()
        self.up_v = tensors[n["up_v"]].view(H, self.value_dim, self.rank).contiguous()
        self.norm_weight = tensors[n["down_norm"]].contiguous()
        self.sinks = tensors[n["sink"]].to(torch.float32).contiguous() if self.has_sink else None

    def kv_cache_spec(self) -> KVCacheSpec:
        return latent_cache_spec(self.rank, self.rot_dim, kind="window" if self.window > 0 else "full",
                                 window=self.window, keep_first=self.keep_first)

    def activation_elements(self) -> int:
        H = self.num_heads
        return (self.proj.out_features if self.proj is not None else 0) + H * (self.key_dim + self.rank + self.value_dim) \
            + (self.q_rank + H * (self.head_dim + self.rot_dim) if self.q_rank else 0) + self.hidden_size

    def forward(self, x, ctx: MixerContext, tail=None):
        if isinstance(x, NormedRows):
            x = x.materialize()
        batch, kv = ctx.batch, ctx.kv
        if kv is None:
            raise K.KernelError("latent attention: the mixer has no cache view")
        T, H = x.shape[0], self.num_heads
        y = self.proj(x)                                                    # [T, q or its latent | entry | gates]
        q_lat = torch.empty((T, H, self.key_dim), dtype=x.dtype, device=x.device)
        cos, sin = self.position.tables(x.device)
        interleaved = self.position.pairing == "interleaved"
        write = kv.writes
        c_q = torch.empty((T, self.q_rank), dtype=x.dtype, device=x.device) if self.q_rank else None
        K.latent_encode_cache(y, self.kv_off, None if self.q_rank else q_lat, kv.arrays["latent"] if write else None,
                              self.norm_weight, self.norm_eps, cos, sin, batch.positions,
                              kv.slot_mapping if write else None, H, self.head_dim, self.rank, interleaved=interleaved,
                              c_q=c_q, q_norm_weight=self.q_norm_weight)
        q = (self.q_up(c_q) if self.q_rank else y[:, :self.kv_off]).view(T, H, self.head_dim + self.rot_dim)
        # queries from a latent exist only now: their rotated parts are turned in the expansion's launch
        rotate = (q[:, :, self.head_dim:], q_lat[:, :, self.rank:], cos, sin, batch.positions, interleaved) if self.q_rank else None
        # the key expansion on the query side: q_lat[:, h, :rank] = U_k[h]^T q_p[h]
        lat_ops.heads_product(q[:, :, :self.head_dim], self.up_k_t, q_lat[:, :, :self.rank], rotate=rotate)
        o_lat = torch.empty((T, H, self.rank), dtype=x.dtype, device=x.device)
        lat_ops.latent_attention(q_lat, o_lat, kv, batch, self.scale, self.window, self.keep_first, self.sinks)
        out = torch.empty((T, H * self.value_dim), dtype=x.dtype, device=x.device)
        # the value expansion behind the attention, the output gate in the same pass
        gates = y[:, self.gate_off:self.gate_off + self._gates()] if self.has_gate else None
        if self.gate_elements:
            gates = gates.unflatten(1, (H, self.value_dim))
        lat_ops.heads_product(o_lat, self.up_v, out.view(T, H, self.value_dim), gates=gates)
        return self.o(out)
