"""The Gokinex decoder as data: its ``config.json`` -> ModelSpec.

A decoder over a residual stream kept in 32-bit.  A token's first row is its row of the token table times a
constant plus a row of a second table picked by the token and the one before it, under a norm.  Every branch
stands between two norms, ``x += n1b(mixer(n1(x))); x += n2b(ff(n2(x)))``, and all norms are dynamic tanh,
``tanh(alpha x) * w + b``, which has no statistics.  A layer's mixer is

* ``attention``: differential attention - heads of two maps over the same values whose outputs are
  subtracted, normed and scaled - with biases on every projection and a rotation of neighbouring elements,
  optionally with llama3 frequency scaling; a layer with ``kv_from`` reads the keys and values of an earlier
  layer instead of making its own;
* ``mamba2``: a state-space mixer with one decay per head and token behind a short causal convolution, its
  gate in front of its norm.

Its feed-forward is dense (``down(gelu_tanh(gate(x)) * up(x))``), a mixture of gated silu experts under a
sigmoid router whose weights multiply the experts' inputs, beside an expert every token uses under a gate of
its own, or absent.  Norm at the end, then the output matrix ``head``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Mapping, Optional, Tuple

from ..config.model_config import ConfigError
from ..config.registry import register_architecture
from .bilolorn import _positive
from .gadopel import _need
from .spec import LayerCall, LayerSpec, ModelSpec, PartSpec

LAYER_TYPES = ("attention", "mamba2")
FEED_FORWARD_KINDS = ("dense", "moe")
SHARED_KEYS = ("kv_heads", "dim", "vdim", "rot")        # what a layer that reads another's keys and values has in common with it


def _check_rot(rot: Any, dim: int, where: str) -> None:
    dims = _need(rot, "dims", where)
    if _need(rot, "base", where, float) <= 0:
        raise ConfigError(f"config.json: {where}.base must be positive")
    if dims % 2 or not 0 <= dims <= dim:
        raise ConfigError(f"config.json: {where}.dims {dims} must be even and at most dim {dim}")
    scaling = rot.get("scaling")
    if scaling is not None:
        for key in ("factor", "low", "high", "original"):
            if _need(scaling, key, where + ".scaling", float) <= 0:
                raise ConfigError(f"config.json: {where}.scaling.{key} must be positive")
        if scaling["high"] < scaling["low"]:
            raise ConfigError(f"config.json: {where}.scaling: high {scaling['high']} is smaller than low {scaling['low']}")


def _check_attention(m: Any, where: str) -> None:
    _positive(m, ("heads", "kv_heads", "dim", "vdim"), where)
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"config.json: {where}: {m['heads']} heads is not a multiple of {m['kv_heads']} kv heads")
    if m["dim"] % 2:
        raise ConfigError(f"config.json: {where}.dim {m['dim']} must be even (keys of two maps lie in the cache in chunks "
                          "of 4 or 8 elements)")
    if _need(m, "scale", where, float) <= 0:
        raise ConfigError(f"config.json: {where}.scale must be positive")
    _need(m, "diff", where, float)
    if m.get("rot") is not None:
        _check_rot(m["rot"], m["dim"], where + ".rot")


def _check_mamba2(m: Any, where: str) -> None:
    _positive(m, ("heads", "vdim", "state", "groups", "norm_groups"), where)
    if m["heads"] % m["groups"]:
        raise ConfigError(f"config.json: {where}: {m['heads']} heads do not come in {m['groups']} equal groups")
    if (m["heads"] * m["vdim"]) % m["norm_groups"]:
        raise ConfigError(f"config.json: {where}: {m['heads']} x {m['vdim']} elements are not normed in {m['norm_groups']} equal parts")
    if not 1 <= _need(m, "conv", where) <= 17:
        raise ConfigError(f"config.json: {where}.conv must lie in 1..17")
    if m["state"] > 512:
        raise ConfigError(f"config.json: {where}.state {m['state']} is larger than 512")


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


def _with_source(layers, i: int) -> Dict[str, Any]:
    """Layer i's mixer sizes; one that reads layer ``kv_from``'s keys and values may leave out what the two have in
    common, and must not contradict it."""
    m = dict(layers[i]["mixer"])
    j = m.get("kv_from")
    if j is None:
        return m
    where = f"layers[{i}].mixer"
    if isinstance(j, bool) or not isinstance(j, int) or not 0 <= j < i:
        raise ConfigError(f"config.json: {where}.kv_from {j!r} must name an earlier layer")
    source = layers[j]
    if source.get("type") != "attention" or source["mixer"].get("kv_from") is not None:
        raise ConfigError(f"config.json: {where}.kv_from: layer {j} has no keys and values of its own")
    for key in SHARED_KEYS:
        if m.get(key) is None:
            m[key] = source["mixer"].get(key)
        elif m[key] != source["mixer"].get(key):
            raise ConfigError(f"config.json: {where}.{key} differs from layer {j}'s, whose keys and values it reads")
    return m


@dataclass(frozen=True)
class GokinexConfig:
    """``config.json`` of a Gokinex model, checked: ``vocab``, ``width``, ``norm.eps``, ``embedding`` (``scale``, absent: 1,
    and ``bigram`` with ``buckets``, ``mul_prev``, ``mul_cur``, or null) and ``layers`` (per layer ``type``, ``mixer`` and
    ``mlp`` or null; ``mixers`` holds the mixers' sizes with what ``kv_from`` brings in)."""

    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    bigram: Optional[Mapping[str, int]]
    layers: Tuple[Mapping[str, Any], ...]
    mixers: Tuple[Mapping[str, Any], ...]
    max_positions: int

    @staticmethod
    def from_dict(d: Mapping[str, Any]) -> "GokinexConfig":
        _positive(d, ("vocab", "width"), "the model")
        eps = _need(d.get("norm"), "eps", "norm", float)
        if eps < 0:
            raise ConfigError("config.json: norm.eps must not be negative")
        emb = d.get("embedding") or {}
        scale = 1.0 if emb.get("scale") is None else _need(emb, "scale", "embedding", float)
        bigram = emb.get("bigram")
        if bigram is not None:
            _positive(bigram, ("buckets",), "embedding.bigram")
            for key in ("mul_prev", "mul_cur"):
                if not 0 <= _need(bigram, key, "embedding.bigram") < 1 << 31:
                    raise ConfigError(f"config.json: embedding.bigram.{key} must lie in 0..2^31 - 1")
        layers = d.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        for i, layer in enumerate(layers):
            if not isinstance(layer, Mapping) or layer.get("type") not in LAYER_TYPES:
                raise ConfigError(f"config.json: layers[{i}].type must be one of {LAYER_TYPES}")
            if not isinstance(layer.get("mixer"), Mapping):
                raise ConfigError(f"config.json: layers[{i}].mixer must give the mixer's sizes")
        mixers = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            if layer["type"] == "attention":
                mixers.append(_with_source(layers, i))
                _check_attention(mixers[-1], where + ".mixer")
            else:
                mixers.append(layer["mixer"])
                _check_mamba2(mixers[-1], where + ".mixer")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], where + ".mlp")
        return GokinexConfig(vocab=d["vocab"], width=d["width"], norm_eps=eps, embedding_scale=scale, bigram=bigram,
                             layers=tuple(layers), mixers=tuple(mixers), max_positions=int(d.get("max_positions", 1 << 17)))


def _norm(prefix: str, name: str, width: int) -> PartSpec:
    return PartSpec("dynamic_tanh", dict(prefix=prefix, width=width, weight_name=name))


def _attention(m: Mapping[str, Any], p: str, W: int, eps: float, max_positions: int) -> PartSpec:
    rot = m.get("rot")
    if rot is not None and int(rot["dims"]) > 0:
        sc = rot.get("scaling")
        rule = dict(frequencies="plain_f64") if sc is None else dict(
            frequencies="llama3_f64", frequency_params={key: float(sc[key]) for key in ("factor", "low", "high", "original")})
        position = PartSpec("rotary", dict(head_dim=int(m["dim"]), rotary_dim=int(rot["dims"]), max_positions=max_positions,
                                           theta=float(rot["base"]), pairing="interleaved", **rule))
    else:
        position = PartSpec("none")
    return PartSpec("differential_attention", dict(
        prefix=p, hidden_size=W, num_heads=int(m["heads"]), num_kv_heads=int(m["kv_heads"]), head_dim=int(m["dim"]),
        value_dim=int(m["vdim"]), scale=float(m["scale"]), diff=float(m["diff"]), norm_eps=eps, position=position, bias=True,
        shared_kv=m.get("kv_from") is not None))


def _mamba2(m: Mapping[str, Any], p: str, W: int, eps: float) -> PartSpec:
    return PartSpec("state_space_duality", dict(
        prefix=p, hidden_size=W, num_heads=int(m["heads"]), value_dim=int(m["vdim"]), state_size=int(m["state"]),
        groups=int(m["groups"]), conv_taps=int(m["conv"]), norm_groups=int(m["norm_groups"]), norm_eps=eps))


def _feed_forward(mlp: Optional[Mapping[str, Any]], p: str, W: int) -> PartSpec:
    if mlp is None:
        return PartSpec("none")
    if mlp["kind"] == "dense":
        return PartSpec("gated", dict(prefix=p, hidden_size=W, intermediate_size=int(mlp["ff"]), activation="gelu_tanh",
                                      tensor_names=dict(gate="gate", up="up", down="down")))
    r, shared = mlp["router"], mlp.get("shared")
    return PartSpec("routed_experts", dict(
        prefix=p, hidden_size=W, intermediate_size=int(mlp["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]),
        activation="silu", gated=True, correction=False, scores="sigmoid", weight_on="input",
        shared_intermediate=int(shared["ff"]) if shared else 0, shared_gate=bool(shared)))


def gokinex_spec(cfg: GokinexConfig) -> ModelSpec:
    W, eps = cfg.width, cfg.norm_eps
    layers, order, ignorable = [], [], []
    for i, (layer, m) in enumerate(zip(cfg.layers, cfg.mixers)):
        p = f"l{i}."
        norms = {"mixer": _norm(p, "norm1", W), "mixer_out": _norm(p, "norm1b", W)}
        if layer.get("mlp") is not None:
            norms.update(feed_forward=_norm(p, "norm2", W), feed_forward_out=_norm(p, "norm2b", W))
        else:       # nothing to norm for such a layer
            ignorable += [p + name + end for name in ("norm2", "norm2b") for end in ("", ".b", ".alpha")]
        mixer = _attention(m, p + "mix.", W, eps, cfg.max_positions) if layer["type"] == "attention" \
            else _mamba2(m, p + "mix.", W, eps)
        layers.append(LayerSpec(block=PartSpec("sandwich_norm"), mixer=mixer,
                                feed_forward=_feed_forward(layer.get("mlp"), p + "mlp.", W), norms=norms, prefix=p))
        source = m.get("kv_from") if layer["type"] == "attention" else None
        order.append(LayerCall(layer=i, cache=i if source is None else source, writes_cache=source is None))
    bg = cfg.bigram
    embedding = PartSpec("token_pairs", dict(
        vocab_size=cfg.vocab, width=W, table_name="embed", scale=cfg.embedding_scale, norm=_norm("embed.", "norm", W),
        **(dict(pair_name="bigram", buckets=int(bg["buckets"]), mul_prev=int(bg["mul_prev"]), mul_cur=int(bg["mul_cur"]))
           if bg is not None else {})))
    return ModelSpec(
        architecture="Gokinex", hidden_size=W, vocab_size=cfg.vocab, embedding_name="embed", embedding=embedding,
        layers=tuple(layers), order=tuple(order), final_norm=_norm("final.", "norm", W), final_norm_prefix="final.",
        head_name="head", max_positions=cfg.max_positions, residual_dtype="float32", ignorable_tensors=tuple(ignorable))


register_architecture("Gokinex", GokinexConfig.from_dict, gokinex_spec, replace=True)
