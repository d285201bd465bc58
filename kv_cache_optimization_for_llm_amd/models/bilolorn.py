"""The Bilolorn decoder as data: its ``config.json`` -> ModelSpec.

A decoder over a residual stream kept in 32-bit whose branches stand between two layer norms (weight
and bias): ``x += n1b(mixer(n1(x))); x += n2b(ff(n2(x)))``.  The mixer of every layer is latent
attention: queries through a low-rank row of their own, one low-rank key/value row and one rotated key
part per token for all heads, rotation of neighbouring elements, a sink per head in the softmax's
denominator, and a sigmoid gate for every element of the concatenated heads.  The feed-forward is dense
(``down(relu(up(x))^2)``), a set of gated silu experts that a table picks by token id - equal weights, no
router - beside an expert every token uses, or absent.  The token table's rows enter times a constant.
A run of layers may be repeated with the same weights, every pass over a cache of its own; in front of
every pass but the first the embedding output is added to the stream.  Layer norm at the end, then the
output matrix ``head``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from .gadopel import _need
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

LAYER_TYPES = ("latent_attention",)
FEED_FORWARD_KINDS = ("dense", "moe")


def _positive(m: Any, keys, where: str) -> None:
    for key in keys:
        if _need(m, key, where) <= 0:
            raise ConfigError(f"config.json: {where}.{key} must be positive")


def _check_mixer(m: Any, where: str) -> None:
    _positive(m, ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"), where)
    _need(m, "scale", where, float)
    rot = m.get("rot")
    dims = _need(rot, "dims", where + ".rot")
    if _need(rot, "base", where + ".rot", float) <= 0:
        raise ConfigError(f"config.json: {where}.rot.base must be positive")
    if dims != m["rot_dim"] or dims % 2:
        raise ConfigError(f"config.json: {where}: the rotation covers rot.dims = {dims} elements, the rotated part has "
                          f"rot_dim = {m['rot_dim']} (an even number)")


def _check_mlp(mlp: Any, where: str) -> None:
    if not isinstance(mlp, Mapping) or mlp.get("kind") not in FEED_FORWARD_KINDS:
        raise ConfigError(f"config.json: {where}.kind must be one of {FEED_FORWARD_KINDS}")
    if mlp["kind"] == "dense":
        _positive(mlp, ("ff",), where)
        return
    _positive(mlp.get("expert"), ("ff",), where + ".expert")
    r = mlp.get("router")
    experts, top = _need(r, "experts", where + ".router"), _need(r, "top", where + ".router")
    if not 0 < top <= experts:
        raise ConfigError(f"config.json: {where}.router: top {top} of {experts} experts")
    if mlp.get("shared") is not None:
        _positive(mlp["shared"], ("ff",), where + ".shared")


@dataclass(frozen=True)
class BilolornConfig:
    """``config.json`` of a Bilolorn model, checked: ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` (absent:
    1), ``layers`` (per layer ``type``, ``mixer`` and ``mlp`` or null) and the optional ``loop`` (``start``, ``stop``,
    ``times``)."""

    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[Mapping[str, Any], ...]
    loop: Optional[Tuple[int, int, int]]
    max_positions: int

    @staticmethod
    def from_dict(d: Mapping[str, Any]) -> "BilolornConfig":
        _positive(d, ("vocab", "width"), "the model")
        eps = _need(d.get("norm"), "eps", "norm", float)
        if eps < 0:
            raise ConfigError("config.json: norm.eps must not be negative")
        scale = 1.0 if (d.get("embedding") or {}).get("scale") is None else _need(d["embedding"], "scale", "embedding", float)
        layers = d.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            if not isinstance(layer, Mapping) or layer.get("type") not in LAYER_TYPES:
                raise ConfigError(f"config.json: {where}.type must be one of {LAYER_TYPES}")
            _check_mixer(layer.get("mixer"), where + ".mixer")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], where + ".mlp")
        loop = d.get("loop")
        if loop is not None:
            a, b, n = (_need(loop, k, "loop") for k in ("start", "stop", "times"))
            if not (0 <= a < b <= len(layers)) or n < 1:
                raise ConfigError(f"config.json: loop {a}..{b} x {n} does not fit {len(layers)} layers")
            loop = (a, b, n)
        return BilolornConfig(vocab=d["vocab"], width=d["width"], norm_eps=eps, embedding_scale=scale, layers=tuple(layers),
                              loop=loop, max_positions=int(d.get("max_positions", 1 << 17)))


def _norm(prefix: str, name: str, width: int, eps: float) -> PartSpec:
    return PartSpec("layernorm", dict(prefix=prefix, width=width, eps=eps, weight_name=name, bias_name=name + ".b"))


def _mixer(m: Mapping[str, Any], p: str, W: int, eps: float, max_positions: int) -> PartSpec:
    position = PartSpec("rotary", dict(head_dim=int(m["rot_dim"]), max_positions=max_positions, theta=float(m["rot"]["base"]),
                                       pairing="interleaved", frequencies="plain_f64"))
    return PartSpec("latent_attention", dict(
        prefix=p, hidden_size=W, num_heads=int(m["heads"]), head_dim=int(m["dim"]), rot_dim=int(m["rot_dim"]),
        value_dim=int(m["vdim"]), rank=int(m["kv_rank"]), q_rank=int(m["q_rank"]), scale=float(m["scale"]), norm_eps=eps,
        position=position, sink=True, gate="element",
        tensor_names=dict(q_down="dq", q_norm="dq.norm", q="uq", down="dkv", down_norm="dkv.norm", up_k="uk", up_v="uv",
                          sink="sink", gate="g", o="o")))


def _feed_forward(mlp: Optional[Mapping[str, Any]], p: str, W: int, vocab: int) -> PartSpec:
    if mlp is None:
        return PartSpec("none")
    if mlp["kind"] == "dense":
        return PartSpec("mlp", dict(prefix=p, hidden_size=W, intermediate_size=int(mlp["ff"]), activation="relu2"))
    r, shared = mlp["router"], mlp.get("shared")
    return PartSpec("routed_experts", dict(
        prefix=p, hidden_size=W, intermediate_size=int(mlp["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]),
        activation="silu", gated=True, correction=False, router="table", table_rows=vocab,
        shared_intermediate=int(shared["ff"]) if shared else 0))


def bilolorn_spec(cfg: BilolornConfig) -> ModelSpec:
    W, eps = cfg.width, cfg.norm_eps
    layers, ignorable = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        norms = {"mixer": _norm(p, "norm1", W, eps), "mixer_out": _norm(p, "norm1b", W, eps)}
        if layer.get("mlp") is not None:
            norms.update(feed_forward=_norm(p, "norm2", W, eps), feed_forward_out=_norm(p, "norm2b", W, eps))
        else:
            ignorable += [p + "norm2", p + "norm2.b", p + "norm2b", p + "norm2b.b"]    # nothing to norm for such a layer
        layers.append(LayerSpec(block=PartSpec("sandwich_norm"),
                                mixer=_mixer(layer["mixer"], p + "mix.", W, eps, cfg.max_positions),
                                feed_forward=_feed_forward(layer.get("mlp"), p + "mlp.", W, cfg.vocab), norms=norms, prefix=p))
    # run order: the layers before the loop, the looped run `times` times (every pass over cache slots of its
    # own, the embedding output added in front of every pass but the first), then the rest
    n = len(layers)
    a, b, times = cfg.loop if cfg.loop is not None else (n, n, 0)
    runs = [(i, None) for i in range(a)]
    for k in range(times):
        runs += [(i, 0 if k > 0 and i == a else None) for i in range(a, b)]
    runs += [(i, None) for i in range(b, n)]
    return ModelSpec(
        architecture="Bilolorn", hidden_size=W, vocab_size=cfg.vocab, embedding_name="embed", layers=tuple(layers),
        order=tuple(LayerCall(layer=i, cache=slot, before=before) for slot, (i, before) in enumerate(runs)),
        final_norm=_norm("final.", "norm", W, eps), final_norm_prefix="final.", head_name="head",
        max_positions=cfg.max_positions, embedding_scale=cfg.embedding_scale, residual_dtype="float32",
        stream_ops=(PartSpec("add_first"),) if times > 1 else (), ignorable_tensors=tuple(ignorable))


register_architecture("Bilolorn", BilolornConfig.from_dict, bilolorn_spec, replace=True)
