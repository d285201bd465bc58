"""Random-weights mode: writes a model folder (``config.json`` + ``model.safetensors``) from a
configuration and a seed.

Matrices are N(0, 0.02), norm weights 1 + U(-0.1, 0.1), matrices that mix copies of the stream the identity
+ U(-0.1, 0.1), tables of choices rows of different integers.  With a ``gain`` a matrix ``[out, in]``
is N(0, gain / sqrt(in)) instead: its products of unit-size inputs are of size ``gain`` at any
width, so attention scores spread and a tied model's best next token is not its input token -
what tests of generation need from random weights.  Each tensor's generator is seeded from
(seed, tensor name), so a tensor's values do not depend on which other tensors exist or on the
order they are made in.  Values are drawn in fp32 and stored in the configuration's
``torch_dtype`` (or the dtype asked for).
"""
from __future__ import annotations

import hashlib
import os
from typing import Any, Dict, Mapping, Optional

import torch

from ..config.model_config import write_config_json
from ..models.spec import TensorSpec

_DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def _generator(seed: int, name: str) -> torch.Generator:
    digest = hashlib.sha256(f"{seed}:{name}".encode()).digest()
    g = torch.Generator(device="cpu")
    g.manual_seed(int.from_bytes(digest[:8], "little") & ((1 << 63) - 1))
    return g


def _random_table(spec: TensorSpec, g: torch.Generator, device) -> torch.Tensor:
    """Integers: zeros, or (``"distinct"``) every row a random choice of different integers below ``bound``."""
    if spec.init != "distinct":
        return torch.zeros(spec.shape, dtype=torch.int32, device=device)
    rows, k = spec.shape
    order = torch.rand((rows, spec.bound), generator=g, device=device).argsort(dim=-1)
    return order[:, :k].to(torch.int32).contiguous()


def random_tensor(name: str, spec: TensorSpec, seed: int, dtype: torch.dtype,
                  gain: Optional[float] = None) -> torch.Tensor:
    g = _generator(seed, name)
    if spec.role == "table":
        return _random_table(spec, g, "cpu")
    if spec.init == "normal":
        std = 0.02 if gain is None or len(spec.shape) != 2 else float(gain) / float(spec.shape[1]) ** 0.5
        t = torch.randn(spec.shape, generator=g, dtype=torch.float32) * std
    elif spec.init == "norm":
        t = 1.0 + (torch.rand(spec.shape, generator=g, dtype=torch.float32) * 0.2 - 0.1)
    elif spec.init == "zeros":
        t = torch.zeros(spec.shape, dtype=torch.float32)
    elif spec.init == "eye":            # a square matrix near the identity
        t = torch.eye(spec.shape[0], spec.shape[1]) + (torch.rand(spec.shape, generator=g, dtype=torch.float32) * 0.2 - 0.1)
    else:
        raise ValueError(f"tensor {name!r}: unknown init rule {spec.init!r}")
    return t.to(dtype)


def random_state_dict(specs: Mapping[str, TensorSpec], seed: int, dtype: torch.dtype,
                      gain: Optional[float] = None) -> Dict[str, torch.Tensor]:
    return {name: random_tensor(name, spec, seed, dtype, gain) for name, spec in specs.items()}


def random_tensors_on_device(specs: Mapping[str, TensorSpec], seed: int, dtype: torch.dtype,
                             device) -> Dict[str, torch.Tensor]:
    """The same distributions drawn on the device (fast for large models; another random stream
    than :func:`random_tensor`)."""
    g = torch.Generator(device=device)
    out: Dict[str, torch.Tensor] = {}
    for i, (name, spec) in enumerate(specs.items()):
        g.manual_seed((int(seed) * 1000003 + i) & ((1 << 63) - 1))
        if spec.role == "table":
            out[name] = _random_table(spec, g, device)
        elif spec.init == "normal":
            t = torch.empty(spec.shape, dtype=torch.float32, device=device).normal_(0.0, 0.02, generator=g)
            out[name] = t.to(dtype)
        elif spec.init == "norm":
            t = torch.empty(spec.shape, dtype=torch.float32, device=device).uniform_(0.9, 1.1, generator=g)
            out[name] = t.to(dtype)
        elif spec.init == "eye":
            t = torch.empty(spec.shape, dtype=torch.float32, device=device).uniform_(-0.1, 0.1, generator=g)
            out[name] = (t + torch.eye(spec.shape[0], spec.shape[1], device=device)).to(dtype)
        else:
            out[name] = torch.zeros(spec.shape, dtype=dtype, device=device)
    return out


def write_random_model(model_dir: str, config_dict: Mapping[str, Any], seed: int,
                       dtype: Optional[str] = None, gain: Optional[float] = None) -> str:
    """Creates ``model_dir`` with ``config.json`` and a seeded ``model.safetensors``."""
    from safetensors.torch import save_file
    from ..models.builder import tensor_specs_for_config

    cfg = dict(config_dict)
    dtype_name = dtype or cfg.get("torch_dtype", "bfloat16")
    if dtype_name not in _DTYPES:
        raise ValueError(f"dtype {dtype_name!r} is not one of {sorted(_DTYPES)}")
    cfg["torch_dtype"] = dtype_name
    specs = tensor_specs_for_config(cfg)
    os.makedirs(model_dir, exist_ok=True)
    write_config_json(model_dir, cfg)
    state = random_state_dict(specs, seed, _DTYPES[dtype_name], gain)
    save_file(state, os.path.join(model_dir, "model.safetensors"), metadata={"format": "pt"})
    return model_dir


def main(argv=None) -> int:
    """``python -m kv_cache_optimization_for_llm_amd.weights.random_init --config config.json
    --out DIR --seed 0``: writes a model folder with random weights for a configuration."""
    import argparse
    import json

    ap = argparse.ArgumentParser(description="write a model folder (config.json, model.safetensors) "
                                             "with seeded random weights")
    ap.add_argument("--config", required=True, help="a config.json of the architecture (its own keys)")
    ap.add_argument("--out", required=True, help="folder to create")
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--dtype", choices=sorted(_DTYPES), default=None,
                    help="storage type of the tensors (default: the configuration's torch_dtype)")
    ap.add_argument("--gain", type=float, default=None,
                    help="matrices [out, in] are N(0, gain / sqrt(in)) instead of N(0, 0.02)")
    args = ap.parse_args(argv)
    with open(args.config) as f:
        cfg = json.load(f)
    print(write_random_model(args.out, cfg, args.seed, args.dtype, args.gain))
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
