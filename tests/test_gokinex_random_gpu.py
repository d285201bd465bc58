"""Gokinex models drawn at random - widths, layer orders, head counts and sizes, states, groups, taps, experts,
tables of pairs, constants - under random mixed schedules on small pools, against the plain implementation."""
import numpy as np
import pytest

import gokinex_util as U
import replay_util as R
from kv_cache_optimization_for_llm_amd.engine.engine import Engine, EngineOptions

pytestmark = pytest.mark.gpu


def random_config(seed: int) -> dict:
    rng = np.random.default_rng(seed)

    def pick(*values):
        return values[int(rng.integers(len(values)))]
    width = pick(40, 64, 90, 128, 160, 320, 512)

    def mlp():
        r = rng.random()
        if r < 0.15:
            return None
        if r < 0.4:
            return U.dense(pick(30, 64, 100, 384))
        experts = pick(1, 2, 5, 8, 16, 40)
        return U.moe(experts, int(rng.integers(1, min(experts, 6) + 1)), pick(16, 20, 32, 64, 96), pick(None, 16, 50, 128))

    def attention():
        if rng.random() < 0.6:
            dim, vdim = pick((16, 32), (32, 64), (64, 128), (32, 32), (64, 64), (16, 64), (32, 128), (48, 96), (8, 16))
        else:
            dim, vdim = pick(2, 6, 10, 16, 20, 36), pick(1, 5, 12, 20, 33, 64)
        kv = pick(1, 2, 3, 4)
        rotation = None
        if rng.random() < 0.9:
            dims = 2 * int(rng.integers(0, dim // 2 + 1))
            low = pick(1.0, 1.5, 2.0)
            scaling = None if rng.random() < 0.3 else (pick(2.0, 8.0, 32.0), low, low * pick(1.0, 2.0, 4.0), pick(30, 128, 500))
            rotation = U.rot(pick(10.0, 500.0, 10000.0, 500000.0), dims, scaling)
        return U.attention(kv * pick(1, 2, 3, 8), kv, dim, vdim, pick(0.0, 0.2, 0.5, 0.8), pick(0.6, 1.0, 1.5) * dim ** -0.5, rotation)

    def mamba2():
        groups = pick(1, 2, 3, 4)
        heads = groups * pick(1, 2, 3)
        vdim = pick(4, 8, 16, 32, 64, 5, 20)
        parts = [n for n in range(1, 17) if heads * vdim % n == 0]
        return U.mamba2(heads, vdim, pick(1, 8, 16, 33, 64, 100, 128, 136, 256, 288), groups, pick(1, 2, 3, 4, 6, 9), pick(*parts))

    mixers = []
    for i in range(int(rng.integers(2, 6))):
        own = [j for j, (kind, m) in enumerate(mixers) if kind == "attention" and "kv_from" not in m]
        r = rng.random()
        if r < 0.45:
            mixers.append(mamba2())
        elif r < 0.65 and own:
            j = pick(*own)
            m = dict(mixers[j][1], kv_from=j, diff=pick(0.1, 0.4), scale=mixers[j][1]["scale"] * pick(0.7, 1.0))
            m["heads"] = m["kv_heads"] * pick(1, 2, 4)
            mixers.append(("attention", m))
        else:
            mixers.append(attention())
    bigram = None if rng.random() < 0.15 else (pick(1, 7, 100, 1000), pick(0, 1, 31, 100003), pick(0, 1, 17, 2147483647))
    return U.config(pick(64, 101, 256, 333), width, pick(1e-5, 1e-3, 0.02), pick(0.3, 1.0, 2.5), [(m, mlp()) for m in mixers], bigram)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(24))
def test_random_models_under_random_schedules(seed, dtype, tmp_path, gpu):
    cfg = random_config(7000 + seed)
    folder, state = U.write_model(str(tmp_path / "m"), cfg, seed)
    rng = np.random.default_rng(seed)
    lengths = [int(n) for n in rng.integers(1, 140, size=7)]
    reqs = {f"q{i}": U.prompt(cfg, n, 13 * i + seed) for i, n in enumerate(lengths)}
    steps = R.mixed(reqs, seed=seed, max_live=4, chunk_sizes=(2, 3, 7, 16, 40, 70))
    eng = Engine(folder, EngineOptions(dtype=dtype, page_size=16, cache_tokens=R.max_live_tokens(steps, unit=16),
                                       max_seqs=4, max_seq_len=160, max_batch_tokens=1024, use_graphs=False))
    rows, routes = U.run_steps(eng, steps, cfg)
    assert len(rows) == sum(lengths)
    U.assert_rows(rows, U.expected_rows(cfg, state, reqs, dtype, routes), dtype, f"model {cfg}")
    eng.cache.check()
    assert eng.cache.free_seats == 4 and all(g.free_pages() == g.num_pages for g in eng.cache.groups)
