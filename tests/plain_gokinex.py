"""A plain, slow implementation of the Gokinex decoder, one function per mechanism, on the CPU.

It shares no code with the engine: it reads ``config.json``'s dictionary and a name -> tensor
mapping directly and works on whole sequences with dense matrices (no cache, no pages, no state
between calls, no batching).  Everything is computed in ``dtype`` (float64 by default) from the
stored values.

Notation.  ``x`` [T, W] is the residual stream of one sequence, positions 0..T-1.

* start:    ``x = DT_e(s E[token] + B[row])``, ``row = (m_p previous + m_c token) mod buckets``; the first
            token, which has no previous one, takes row ``buckets``
* layer:    ``x <- x + DT1b(mix(DT1(x)))``, then ``x <- x + DT2b(ff(DT2(x)))``
* DT:       ``tanh(alpha x) * w + b`` with one number alpha a norm
* head:     ``logits = W_head DT_final(x)``

``r`` is what is done to every value that an engine with 16-bit products would store in 16 bits (the
identity by default; a rounding, to see what rounding alone does to a row of logits).
"""
from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional

import torch


def same(t: torch.Tensor) -> torch.Tensor:
    return t


def dynamic_tanh(x: torch.Tensor, w: Mapping[str, torch.Tensor], name: str) -> torch.Tensor:
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---------------------------------------------------------------- embedding
def bigram_rows(tokens: List[int], bg: Mapping) -> List[int]:
    """The row of the second table that each token takes."""
    rows, before = [], None
    for t in tokens:
        rows.append(bg["buckets"] if before is None else (before * bg["mul_prev"] + t * bg["mul_cur"]) % bg["buckets"])
        before = t
    return rows


def embedding(tokens: List[int], w: Mapping[str, torch.Tensor], emb: Mapping) -> torch.Tensor:
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * emb["scale"]
    if emb.get("bigram"):
        x = x + w["bigram"][torch.as_tensor(bigram_rows(list(tokens), emb["bigram"]), dtype=torch.long)]
    return dynamic_tanh(x, w, "embed.norm")


# ---------------------------------------------------------------- attention
def frequencies(rot: Mapping) -> List[float]:
    """Radians a position for every rotated pair; with ``scaling`` slow pairs turn ``factor`` times slower, fast
    ones as they are, the ones between by a blend over ``original / wavelength``."""
    out = []
    sc = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_pairs(x: torch.Tensor, freqs: List[float]) -> torch.Tensor:
    """``x`` [T, ..., d] with positions 0..T-1: elements (2i, 2i + 1) turned by ``t f_i``, the rest as they are."""
    out = x.clone()
    t = torch.arange(x.shape[0], dtype=x.dtype)
    for i, f in enumerate(freqs):
        co, si = torch.cos(t * f), torch.sin(t * f)
        while co.dim() < x.dim() - 1:
            co, si = co.unsqueeze(-1), si.unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * co - v * si
        out[..., 2 * i + 1] = v * co + u * si
    return out


def causal_softmax(scores: torch.Tensor) -> torch.Tensor:
    """scores [T, T] -> weights of the keys j <= i."""
    T = scores.shape[-1]
    return torch.softmax(scores.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), float("-inf")), dim=-1)


def map_weight(w: Mapping[str, torch.Tensor], p: str, diff: float) -> torch.Tensor:
    """lambda, what the second map is multiplied by: one number a layer."""
    return torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff


def keys_values(h, w, p: str, m: Mapping, r_=same):
    """(rotated keys [T, G, 2, d], values [T, G, dv]) as another layer may read them."""
    T, G, d, dv = h.shape[0], m["kv_heads"], m["dim"], m["vdim"]
    k = r_(h @ w[p + "k"].T).view(T, G, 2, d) + w[p + "k.b"].view(G, 2, d)
    v = r_(r_(h @ w[p + "v"].T) + w[p + "v.b"]).view(T, G, dv)
    return r_(rotate_pairs(k, frequencies(m["rot"]) if m.get("rot") else [])), v


def differential_attention(h, w, p: str, m: Mapping, eps: float, kv, r_=same) -> torch.Tensor:
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    k, v = kv
    q = r_(h @ w[p + "q"].T).view(T, H, 2, d) + w[p + "q.b"].view(H, 2, d)
    q = r_(rotate_pairs(q, frequencies(m["rot"]) if m.get("rot") else []))
    lam = map_weight(w, p, m["diff"])
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        a1, a2 = (r_(causal_softmax(q[:, a, i] @ k[:, g, i].T * m["scale"]) @ v[:, g]) for i in (0, 1))
        out[:, a] = unit_rms(a1 - lam * a2, eps) * (1.0 - m["diff"])
    return r_(r_(out.reshape(T, H * dv)) @ w[p + "o"].T) + w[p + "o.b"]


# ---------------------------------------------------------------- state-space duality
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, n] (the last column multiplies the current token), zeros in front of the start."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[j:j + T] * taps[:, j] for j in range(n)) + bias


def mamba2(h, w, p: str, m: Mapping, eps: float, r_=same) -> torch.Tensor:
    T, H, P, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = torch.split(r_(h @ w[p + "in"].T), [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc[:, :inner].view(T, H, P), xbc[:, inner:inner + G * N].view(T, G, N), xbc[:, inner + G * N:].view(T, G, N)
    dt = torch.nn.functional.softplus(dt + w[p + "dt_bias"])
    rate = torch.exp(w[p + "A_log"])
    y = torch.empty(T, H, P, dtype=h.dtype)
    for a in range(H):
        g, S = a // (H // G), torch.zeros(N, P, dtype=h.dtype)
        for t in range(T):
            S = torch.exp(-rate[a] * dt[t, a]) * S + dt[t, a] * torch.outer(B[t, g], x[t, a])
            y[t, a] = S.T @ C[t, g] + w[p + "D"][a] * x[t, a]
    y = (y.reshape(T, inner) * silu(z)).view(T, m["norm_groups"], -1)
    return r_(r_(unit_rms(y, eps).reshape(T, inner) * w[p + "norm"]) @ w[p + "o"].T)


# ---------------------------------------------------------------- feed-forward
def gated(h, w, p: str, act, r_=same) -> torch.Tensor:
    return r_(act(r_(h @ w[p + "gate"].T)) * r_(h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(scores: torch.Tensor, top: int) -> List[int]:
    """The ``top`` largest, of equal ones the lowest index."""
    return sorted(range(scores.shape[0]), key=lambda e: (-float(scores[e]), e))[:top]


def experts(h, w, p: str, mlp: Mapping, r_=same, forced=None, margins: Optional[list] = None) -> torch.Tensor:
    """Every chosen expert reads its weight times the token's row; the outputs are added as they are.  ``forced`` [T,
    top]: the experts that are used instead of the router's choice; ``margins`` takes the router's own choice and, per
    token, how far apart the last score chosen and the first one not chosen are."""
    top = mlp["router"]["top"]
    scores = torch.sigmoid(h @ w[p + "router"].T)
    own = torch.tensor([choose(s, top) for s in scores])
    if margins is not None:
        ranked = scores.sort(-1, descending=True).values
        margins.append((own, ranked[:, top - 1] - ranked[:, top] if top < scores.shape[1] else torch.zeros(h.shape[0], dtype=h.dtype)))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in (own if forced is None else forced)[t].tolist():
            u = scores[t, e] * h[t:t + 1]
            pe = f"{p}e{e}."
            out[t] += (r_(silu(u @ w[pe + "gate"].T) * (u @ w[pe + "up"].T)) @ w[pe + "down"].T)[0]
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * r_(gated(h, w, p + "shared.", silu, r_))
    return r_(out)


def feed_forward(h, w, p: str, mlp: Mapping, r_=same, forced=None, margins: Optional[list] = None) -> torch.Tensor:
    return r_(gated(h, w, p, gelu_tanh, r_)) if mlp["kind"] == "dense" else experts(h, w, p, mlp, r_, forced, margins)


def forward(cfg: Mapping, weights: Mapping[str, torch.Tensor], tokens, dtype=torch.float64,
            residuals: Optional[list] = None, r_=same, forced: Optional[Mapping] = None,
            margins: Optional[dict] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``residuals`` collects the stream after every layer; ``forced`` and
    ``margins``: per layer, see :func:`experts`."""
    w: Dict[str, torch.Tensor] = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = embedding([int(t) for t in tokens], w, cfg["embedding"])
    kvs: Dict[int, tuple] = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = r_(dynamic_tanh(x, w, p + "norm1"))
        if layer["type"] == "attention":
            kvs[i] = kvs[m["kv_from"]] if m.get("kv_from") is not None else keys_values(h, w, p + "mix.", m, r_)
            y = differential_attention(h, w, p + "mix.", m, eps, kvs[i], r_)
        else:
            y = mamba2(h, w, p + "mix.", m, eps, r_)
        x = x + dynamic_tanh(y, w, p + "norm1b")
        if layer.get("mlp"):
            h = r_(dynamic_tanh(x, w, p + "norm2"))
            took: list = []
            y = feed_forward(h, w, p + "mlp.", layer["mlp"], r_, None if forced is None else forced.get(i), took)
            x = x + dynamic_tanh(y, w, p + "norm2b")
            if margins is not None and took:
                margins[i] = took[0]
        if residuals is not None:
            residuals.append(x)
    return r_(dynamic_tanh(x, w, "final.norm")) @ w["head"].T
