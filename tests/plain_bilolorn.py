"""A plain, slow implementation of the Bilolorn decoder, one function per mechanism, on the CPU.

It shares no code with the engine: it reads ``config.json``'s dictionary and a name -> tensor
mapping directly and works on whole sequences with dense matrices (keys and values expanded, no
cache, no pages, no batching).  Everything is computed in ``dtype`` (float64 by default) from the
stored values.

Notation.  ``x`` [T, W] is the residual stream of one sequence, positions 0..T-1.

* start:    ``x0 = s E[token]``, ``x = x0``
* layer:    ``x <- x + LN1b(mix(LN1(x)))``, then ``x <- x + LN2b(ff(LN2(x)))``
* LN:       ``(x - mean) / sqrt(var + eps) * w + b``, biased variance
* looping:  layers ``start..stop-1`` run ``times`` times; in front of every pass but the first
            ``x <- x + x0``
* head:     ``logits = W_head LN_final(x)``

``r`` is what is done to every value that an engine with 16-bit products would store in 16 bits (the
identity by default; a rounding, to see what rounding alone does to a row of logits).
"""
from __future__ import annotations

from typing import Dict, List, Mapping, Optional

import torch


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    mu = x.mean(dim=-1, keepdim=True)
    var = ((x - mu) ** 2).mean(dim=-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * w + b


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def rotate_pairs(x: torch.Tensor, base: float) -> torch.Tensor:
    """``x`` [T, ..., d] with positions 0..T-1: elements (2i, 2i + 1) turned by ``t base^(-2i/d)``."""
    T, d = x.shape[0], x.shape[-1]
    out = torch.empty_like(x)
    t = torch.arange(T, dtype=x.dtype)
    for i in range(d // 2):
        a = t * base ** (-2.0 * i / d)
        co, si = torch.cos(a), torch.sin(a)
        while co.dim() < x.dim() - 1:
            co, si = co.unsqueeze(-1), si.unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * co - v * si
        out[..., 2 * i + 1] = v * co + u * si
    return out


def causal_softmax(scores: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """scores [H, T, T] -> weights of the keys j <= i; ``exp(sink_h)`` is one more term of head h's denominators."""
    T = scores.shape[-1]
    future = torch.ones(T, T, dtype=torch.bool).triu(1)
    s = scores.masked_fill(future, float("-inf"))
    m = torch.maximum(s.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def same(t: torch.Tensor) -> torch.Tensor:
    return t


def latent_attention(h: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, mc: Mapping, eps: float, r_=same) -> torch.Tensor:
    T = h.shape[0]
    H, d, r, dv, rank, base = mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"], mc["kv_rank"], mc["rot"]["base"]
    c_q = r_(rms_norm(r_(h @ w[p + "dq"].T), w[p + "dq.norm"], eps))
    q = r_(c_q @ w[p + "uq"].T).view(T, H, d + r)
    q = torch.cat([q[..., :d], r_(rotate_pairs(q[..., d:], base))], dim=-1)
    down = r_(h @ w[p + "dkv"].T)
    c = r_(rms_norm(down[:, :rank], w[p + "dkv.norm"], eps))
    k_rot = r_(rotate_pairs(down[:, rank:], base))                                   # one for all heads
    k = torch.cat([(c @ w[p + "uk"].T).view(T, H, d), k_rot[:, None, :].expand(T, H, r)], dim=-1)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for a in range(H):
        s = (q[:, a] @ k[:, a].T * mc["scale"])[None]
        out[:, a] = causal_softmax(s, w[p + "sink"][a:a + 1])[0] @ v[:, a]
    gate = torch.sigmoid(r_(h @ w[p + "g"].T))                                   # [T, H dv], one number an element
    return r_(r_(out.reshape(T, H * dv) * gate) @ w[p + "o"].T)


def squared_relu_mlp(h: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, r_=same) -> torch.Tensor:
    return r_(r_(torch.clamp(r_(h @ w[p + "up"].T), min=0.0) ** 2) @ w[p + "down"].T)


def silu_glu(h: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, r_=same) -> torch.Tensor:
    g = h @ w[p + "gate"].T
    return r_(g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def table_experts(h: torch.Tensor, tokens: torch.Tensor, w: Mapping[str, torch.Tensor], p: str, mlp: Mapping, r_=same) -> torch.Tensor:
    """Every token id's row of the table names its experts; their outputs are averaged."""
    top = mlp["router"]["top"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in w[p + "table"][int(tokens[t])].tolist():
            out[t] += silu_glu(h[t:t + 1], w, f"{p}e{int(e)}.", r_)[0] / top
    if mlp.get("shared"):
        out = out + r_(silu_glu(h, w, p + "shared.", r_))
    return r_(out)


def feed_forward(h, tokens, w, p: str, mlp: Mapping, r_=same) -> torch.Tensor:
    return squared_relu_mlp(h, w, p, r_) if mlp["kind"] == "dense" else table_experts(h, tokens, w, p, mlp, r_)


def run_order(cfg: Mapping) -> List[tuple]:
    """[(layer index, True when the embedding output is added in front of it)]"""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    order = [(i, False) for i in range(a)]
    for k in range(times):
        order += [(i, k > 0 and i == a) for i in range(a, b)]
    return order + [(i, False) for i in range(b, n)]


def forward(cfg: Mapping, weights: Mapping[str, torch.Tensor], tokens, dtype=torch.float64,
            residuals: Optional[list] = None, r_=same) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``residuals`` collects the stream after every layer run."""
    w: Dict[str, torch.Tensor] = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(tokens, dtype=torch.long)
    x0 = w["embed"][ids] * cfg["embedding"]["scale"]
    x = x0
    for i, again in run_order(cfg):
        if again:
            x = x + x0
        layer, p = cfg["layers"][i], f"l{i}."

        def norm(name, z):
            return layer_norm(z, w[p + name], w[p + name + ".b"], eps)
        x = x + norm("norm1b", latent_attention(r_(norm("norm1", x)), w, p + "mix.", layer["mixer"], eps, r_))
        if layer.get("mlp"):
            x = x + norm("norm2b", feed_forward(r_(norm("norm2", x)), ids, w, p + "mlp.", layer["mlp"], r_))
        if residuals is not None:
            residuals.append(x)
    return r_(layer_norm(x, w["final.norm"], w["final.norm.b"], eps)) @ w["head"].T
