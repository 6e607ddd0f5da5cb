"""The Dopirax design without a GPU: configuration, plan, tensor names, cache groups, and properties of
the plain implementation that the GPU tests compare the engine with."""

import json
import math

import pytest
import torch

import plain_dopirax as plain
from dopirax_util import (capped, dense, differential, double, experts, model_json, random_weights, tensor_shapes, tokens,
                          write_folder)

CFG = model_json([differential(mlp=dense(40)), capped(), differential(kv_from=0), capped(mlp=None, softcap=None),
                  differential(heads=3, kv_heads=3, dim=20, vdim=36, rot=0, mlp=experts(5, 1, 24, None)),
                  differential(kv_from=0, diff=0.2, mlp=None)])


def test_a_folder_is_found_by_its_architecture_key_and_round_trips(tmp_path):
    from tokamak_amd.config.registry import load_model_description
    from tokamak_amd.models.dopirax import DopiraxConfig, parse, to_config_json

    folder = write_folder(tmp_path / "m", CFG, random_weights(CFG, 1))
    arch, cfg, made = load_model_description(folder)
    assert arch.name == "Dopirax" and isinstance(cfg, DopiraxConfig) and cfg.embedding_scale == 3.0
    assert parse(to_config_json(cfg)) == cfg
    assert [L.type for L in cfg.layers] == [L["type"] for L in CFG["layers"]]
    assert made.vocab_size == CFG["vocab"] and len(made.layers) == 6 and made.embedding["scale"] == 3.0
    assert made.final_norm["offset"] == 1.0


def test_run_order_and_cache_slots_of_borrowed_keys():
    from tokamak_amd.models.dopirax import parse, plan

    made = plan(parse(CFG))
    assert [(c.layer, c.cache, c.writes_cache) for c in made.order] == [
        (0, 0, True), (1, 1, True), (2, 0, False), (3, 3, True), (4, 4, True), (5, 0, False)]
    assert [s.role("mixer").spec["own_keys"] for s in made.layers] == [True, True, False, True, True, False]
    for spec, layer in zip(made.layers, CFG["layers"]):
        roles = dict(spec.parts)
        assert ("feed_forward" in roles) == (layer["mlp"] is not None) and spec.block.kind == "parallel_sublayers"
        assert "feed_forward_norm" not in roles and roles["norm"].spec["offset"] == 1.0
        assert ("position" in roles) == ("rot" in layer["mixer"])
    assert made.layers[0].role("position").spec.kind == "rotary_interleaved"
    assert made.layers[1].role("position").spec.kind == "rotary_half"
    assert made.layers[1].role("mixer").spec["softcap"] == 15.0 and made.layers[3].role("mixer").spec["softcap"] is None


def test_tensor_names_and_shapes_match_a_list_written_independently():
    from tokamak_amd.models.dopirax import parse, plan
    from tokamak_amd.weights.random_init import expected_tensors_of

    for cfg in (CFG, model_json([capped(heads=6, kv_heads=1, dim=20, rot=4, mlp=experts(3, 2, 8, 72)), capped(heads=6, kv_heads=1, dim=20, mlp=dense(8))],
                                width=72)):
        expected = expected_tensors_of(plan(parse(cfg)))
        shapes = tensor_shapes(cfg)
        assert set(expected) == set(shapes)
        assert all(expected[n].fits(shape) for n, shape in shapes.items())


def test_a_capped_layer_may_borrow_too():
    from tokamak_amd.models.dopirax import parse, plan
    from tokamak_amd.weights.random_init import expected_tensors_of

    cfg = model_json([capped(mlp=None), capped(heads=8, mlp=None)])
    cfg["layers"][1]["mixer"]["kv_from"] = 0
    made = plan(parse(cfg))
    assert [(c.cache, c.writes_cache) for c in made.order] == [(0, True), (0, False)]
    assert set(expected_tensors_of(made)) == set(tensor_shapes(cfg))


def test_optional_keys_may_be_absent():
    from tokamak_amd.models.dopirax import parse, plan

    cfg = model_json([capped(rot=0, softcap=None), differential(vdim=16, mlp=experts(4, 2, 16, None))], scale=None)
    for layer in cfg["layers"]:
        layer["mixer"].pop("kv_heads")
        layer["mixer"].pop("vdim")
    parsed = parse(cfg)
    made = plan(parsed)
    assert parsed.embedding_scale == 1.0
    mixer = made.layers[0].role("mixer").spec
    assert mixer["num_kv_heads"] == 4 and mixer["value_dim"] == 16 and mixer["softcap"] is None and mixer["unit_sink"] is True
    assert made.layers[1].role("mixer").spec["num_kv_heads"] == 2 and made.layers[1].role("mixer").spec["value_dim"] == 16
    ff = made.layers[1].role("feed_forward").spec
    assert ff["shared_size"] is None and ff["shared_gate"] is None and ff["scoring"] == "chosen_softmax"


@pytest.mark.parametrize("change,message", [
    (lambda c: c.update(architecture="Other"), "Unsupported architecture"),
    (lambda c: c["layers"][0].update(type="attention_3"), "unknown layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "unknown feed-forward kind"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=4), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(dim=8, rot={"base": 10.0, "dims": 4}), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].update(heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=24), "vdim"),
    (lambda c: c["layers"][1]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), "rot.dims"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "top <= experts"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "ff >= 1"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
])
def test_what_cannot_be_a_model_is_refused(change, message):
    from tokamak_amd.models.dopirax import parse

    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    with pytest.raises(ValueError, match=message):
        parse(cfg)


def test_presets_build_and_shorten():
    from tokamak_amd.config.registry import find_preset

    for name in ("dopirax-tiny", "dopirax-0.6b", "dopirax-8b"):
        arch, cfg = find_preset(name)
        made = arch.plan(arch.shorten(cfg, 3))
        assert len(made.layers) == 3 and arch.parse(arch.to_json(cfg)) == cfg
        assert made.order[2].cache == 0 and not made.order[2].writes_cache


def test_a_borrowing_layer_asks_for_no_pages():
    from tokamak_amd.engine.model import LayeredModel
    from tokamak_amd.models.dopirax import parse, plan

    model = LayeredModel(plan(parse(CFG)), dtype=torch.float32, device="meta")
    groups, slots = model.cache_layout()
    assert [(g.window, g.slots) for g in groups] == [(None, (0, 1, 3, 4))] and not model.state_requests()
    # per token: both maps' keys (in pieces of 8 channels) and the values (in blocks of 16)
    assert [a.elems_per_token for _, a in slots[0].request.arrays] == [32, 32]
    assert [a.elems_per_token for _, a in slots[1].request.arrays] == [32, 32]
    assert [a.elems_per_token for _, a in slots[4].request.arrays] == [3 * 40, 3 * 48]


# -- properties of the plain implementation -----------------------------------------------
def test_plain_rotation_pairs_halves_or_neighbours():
    x = torch.randn(3, 2, 10, dtype=torch.float64)
    rot = {"base": 100.0, "dims": 6}
    for interleaved in (False, True):
        out = plain.rotate(x, torch.tensor([0, 5, 9]), rot, interleaved)
        assert torch.equal(out[0], x[0]) and torch.equal(out[..., 6:], x[..., 6:])
        a, b = (2, 3) if interleaved else (1, 4)
        angle = 5 * 100.0 ** (-2.0 / 6)
        u, v = x[1, 0, a], x[1, 0, b]
        assert float(out[1, 0, a]) == pytest.approx(float(u * math.cos(angle) - v * math.sin(angle)))
        assert float(out[1, 0, b]) == pytest.approx(float(v * math.cos(angle) + u * math.sin(angle)))


def test_plain_softmax_with_one_more_term_and_the_cap():
    s = torch.tensor([[1.0, 9.0], [2.0, -1.0]], dtype=torch.float64)
    got = plain.causal_weights(s, True)
    assert float(got[0, 1]) == 0.0 and float(got[0, 0]) == pytest.approx(math.e / (1 + math.e))
    total = 1 + math.exp(2.0) + math.exp(-1.0)
    assert got[1].tolist() == pytest.approx([math.exp(2.0) / total, math.exp(-1.0) / total])
    assert plain.causal_weights(s, False).sum(-1).tolist() == pytest.approx([1.0, 1.0])
    low = plain.causal_weights(torch.full((1, 1), -800.0, dtype=torch.float64), True)
    assert float(low) == 0.0                     # (nothing but the sink)
    capped_scores = plain.soft_cap(torch.tensor([0.001, 500.0, -500.0], dtype=torch.float64), 7.0)
    assert capped_scores.tolist() == pytest.approx([0.001, 7.0, -7.0], rel=1e-6)


def test_plain_difference_of_maps():
    a1, a2 = torch.tensor([[3.0, 1.0]], dtype=torch.float64), torch.tensor([[1.0, 1.0]], dtype=torch.float64)
    o = plain.difference(a1, a2, torch.tensor(0.5, dtype=torch.float64), 0.25, 0.0)
    rms = math.sqrt((2.5 ** 2 + 0.5 ** 2) / 2)
    assert o[0].tolist() == pytest.approx([0.75 * 2.5 / rms, 0.75 * 0.5 / rms])
    w = {f"p.{n}": torch.full((2,), v, dtype=torch.float64) for n, v in (("lq1", 0.5), ("lk1", 1.0), ("lq2", 2.0), ("lk2", -0.5))}
    assert float(plain.difference_weight(w, "p.", {"diff": 0.25})) == pytest.approx(math.exp(1.0) - math.exp(-2.0) + 0.25)


def test_plain_router_takes_the_bias_and_weighs_the_chosen_only():
    w = {"r.router": torch.eye(4, dtype=torch.float64), "r.router.b": torch.tensor([0.0, 0.0, 0.0, 5.0], dtype=torch.float64)}
    h = torch.tensor([[1.0, 3.0, 2.0, 0.0]], dtype=torch.float64)
    margins = []
    chosen, weight = plain.route(h, w, "r.", {"experts": 4, "top": 2}, margins)
    assert chosen[0].tolist() == [3, 1] and margins == pytest.approx([1.0])
    e = [math.exp(5.0), math.exp(3.0)]
    assert weight[0].tolist() == pytest.approx([e[0] / sum(e), e[1] / sum(e)])


def test_plain_model_runs_and_borrowed_keys_are_the_sources():
    w = random_weights(CFG, 4)
    toks = tokens(CFG["vocab"], 12, 2)
    logits, after = plain.forward(CFG, double(w), toks)
    assert logits.shape == (12, CFG["vocab"]) and after.shape == (6, 12, CFG["width"])
    # layers 2 and 5 read layer 0's keys and values: changing those moves layer 2's output even with layer 0's own
    # attention taken out of the picture (its o projection zeroed)
    for name in ("k", "v", "k.norm"):
        changed = dict(double(w))
        changed["l0.mix.o"] = torch.zeros_like(changed["l0.mix.o"])
        base = plain.forward(CFG, changed, toks)[1]
        changed[f"l0.mix.{name}"] = changed[f"l0.mix.{name}"] + 0.3 * torch.randn_like(changed[f"l0.mix.{name}"])
        moved = plain.forward(CFG, changed, toks)[1]
        assert torch.allclose(moved[1], base[1], atol=1e-12) and not torch.allclose(moved[2], base[2], atol=1e-6), name
