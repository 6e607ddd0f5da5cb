"""Korazen models drawn at random (layer order, every size, chunks, decays, ranks, limits) replayed through
the step function in mixed batches against the plain implementation, in both dtypes.  The sizes are
the kind a real checkpoint has (multiples of 8 or 16 mostly, some not)."""

import random

import pytest

from korazen_util import Expected, delta, dense, model_json, parallel, random_weights, tokens, write_folder
from replay_util import mixed, tail_one_by_one, whole
from rorosun_util import run_steps
from test_gpu_korazen import check_rows

pytestmark = pytest.mark.gpu


def draw_model(seed):
    rng = random.Random(seed)
    width = rng.choice([48, 64, 96, 128, 160, 200])

    def mlp():
        return rng.choice([None, dense(rng.choice([24, 48, 80, 136]), rng.choice([0.5, 1.0, 3.0, 7.0]))])

    layers = []
    for _ in range(rng.randint(3, 6)):
        if rng.random() < 0.5:
            kv = rng.choice([1, 2, 3])
            layers.append(delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([8, 16, 32, 48, 80, 128]), rng.choice([8, 16, 20, 64]),
                                rng.choice([2, 3, 4, 4, 5]), mlp()))
            continue
        kv = rng.choice([1, 2])
        dim = rng.choice([8, 16, 24, 32, 64, 128])
        left = dict(heads=kv * rng.choice([1, 2, 4, 5]), kv_heads=kv, dim=dim, vdim=rng.choice([dim, 16, 32, 48]),
                    rot=rng.choice([0, 2, dim // 2, dim]), chunk=rng.choice([1, 5, 16, 30, 64, 100, None]),
                    base=rng.choice([1e4, 5e5]), scale=rng.choice([None, 0.3]))
        heads = rng.choice([1, 2, 4, 5])
        right = dict(heads=heads, dim=rng.choice([8, 16, 24, 64]), vdim=rng.choice([8, 16, 40, 64]),
                     decay=[round(rng.uniform(0.3, 1.0), 4) for _ in range(heads)])
        layers.append(parallel(left, right, mlp()))
    ranks = (rng.choice([1, 6, 8, 24]), rng.choice([2, 8, 16]))
    cfg = model_json(layers, vocab=rng.choice([96, 130, 257]), width=width, eps=rng.choice([1e-5, 1e-6]),
                     logit_scale=rng.choice([None, 0.5, 3.0]))
    return cfg, random_weights(cfg, seed, ranks=ranks), rng.choice([8, 16, 32])


@pytest.mark.parametrize("seed", range(12))
def test_random_models(tmp_path, seed):
    from tokamak_amd.engine.runner import ModelRunner

    cfg, w, page = draw_model(seed)
    folder = write_folder(tmp_path / "m", cfg, w)
    requests = {f"r{i}": tokens(cfg["vocab"], n, 1000 * seed + i) for i, n in enumerate([1, 9, 70, 33, 18, 140])}
    expected = {rid: Expected(cfg, w, toks) for rid, toks in requests.items()}
    steps, peak = mixed(requests, seed)
    for dtype in ("float32", "bfloat16"):
        runner = ModelRunner.from_folder(folder, dtype=dtype, page_size=page, kv_pool_tokens=max(peak, 192), max_requests=4)
        for way in (steps, tail_one_by_one("r5", requests["r5"], tail=20), whole({"r2": requests["r2"]})):
            check_rows(way, run_steps(runner, way), expected, dtype, f"seed {seed}")
        runner.manager.check()
