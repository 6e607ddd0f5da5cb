"""Dopirax models drawn at random (layer order, every size, caps, borrowed keys, routers, factors) replayed through
the step function in mixed batches against the plain implementation, in both dtypes."""

import random

import pytest

from dopirax_util import (capped, dense, differential, every_expert, experts, model_json, oracle_with_margins, random_weights,
                          tokens, write_folder)
from replay_util import mixed, portions, tail_one_by_one, whole
from rorosun_util import run_steps
from test_gpu_dopirax import check_rows

pytestmark = pytest.mark.gpu


def draw_mlp(rng):
    kind = rng.choice(["dense", "moe", "moe", None])
    if kind is None:
        return None
    if kind == "dense":
        return dense(rng.choice([24, 48, 80, 128, 200]))
    n = rng.choice([1, 2, 4, 6, 8, 16, 24])
    return experts(n, rng.randint(1, min(4, n)), rng.choice([16, 24, 40, 64]), rng.choice([None, 16, 56, 64]))


def draw_model(seed):
    rng = random.Random(seed)
    width = rng.choice([48, 64, 96, 128, 160, 200])
    layers, sources = [], []
    for i in range(rng.randint(3, 7)):
        mlp = draw_mlp(rng)
        kv = rng.choice([1, 2, 3])
        heads = kv * rng.choice([1, 2, 4, 5, 8])
        scale = rng.choice([None, 0.2, 0.05])
        if rng.random() < 0.4:
            dim = rng.choice([16, 32, 48, 64, 80, 96, 128])
            layers.append(capped(heads, kv, dim, rng.choice([0, dim, dim // 2, 8]), scale, rng.choice([1e3, 1e4, 5e5]),
                                 rng.choice([None, 2.0, 10.0, 50.0]), mlp))
            continue
        source = rng.choice([None] + sources)
        if source is None:
            dim = rng.choice([8, 16, 24, 32, 40, 64])
            m = dict(kv_heads=kv, dim=dim, vdim=rng.choice([dim, 2 * dim, 16, 48]), rot=rng.choice([0, dim, dim // 2, 4]),
                     base=rng.choice([1e3, 1e4, 5e5]))
            sources.append(i)
        else:
            src = layers[source]["mixer"]
            m = dict(kv_heads=src["kv_heads"], dim=src["dim"], vdim=src["vdim"], rot=src.get("rot", {}).get("dims", 0),
                     base=src.get("rot", {}).get("base", 1e4))
            heads = src["heads"] if rng.random() < 0.7 else src["kv_heads"] * rng.choice([1, 2, 4])
        layers.append(differential(heads=heads, scale=scale, diff=rng.choice([0.1, 0.4, 0.7]), kv_from=source, mlp=mlp, **m))
    return model_json(layers, vocab=rng.choice([97, 256, 400]), width=width, eps=rng.choice([1e-5, 1e-6]),
                      scale=rng.choice([None, 0.5, 6.0, 20.0]))


@pytest.mark.parametrize("seed", range(14))
def test_random_models_in_mixed_batches(tmp_path, seed):
    from tokamak_amd.engine.runner import ModelRunner

    cfg = draw_model(2000 + seed)
    w = random_weights(cfg, seed)
    requests = {f"r{i}": tokens(cfg["vocab"], n, 7 * seed + i) for i, n in enumerate([3, 130, 47, 1, 81, 20])}
    steps, peak = mixed(requests, seed=seed)
    for dtype, model in (("float32", cfg), ("bfloat16", every_expert(cfg))):
        folder = write_folder(tmp_path / dtype, model, w)
        expected = {rid: oracle_with_margins(model, w, toks)[0] for rid, toks in requests.items()}
        runner = ModelRunner.from_folder(folder, dtype=dtype, page_size=16, kv_pool_tokens=max(peak, 16), max_requests=4)
        check_rows(steps, run_steps(runner, steps), expected, dtype, (seed, cfg))
        for plan in (whole({"r1": requests["r1"]}), tail_one_by_one("r4", requests["r4"], tail=40), portions("r1", requests["r1"])):
            check_rows(plan, run_steps(runner, plan), expected, dtype, (seed, cfg))
        runner.manager.check()
        assert all(runner.manager.num_free_pages(g) == runner.manager.num_pages(g) for g in range(runner.num_groups))
