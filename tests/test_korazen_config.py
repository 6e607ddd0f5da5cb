"""The Korazen design without a GPU: configuration, plan, tensor names, cache slots, and properties of
the plain implementation that the GPU tests compare the engine with."""

import json

import pytest
import torch

import plain_korazen as plain
from korazen_util import delta, dense, double, left, model_json, parallel, random_weights, right, tensor_shapes, tokens, write_folder

CFG = model_json([delta(), parallel(), delta(mlp=dense(40, 2.5)), parallel(dict(rot=0, chunk=None), mlp=None)])


def test_a_folder_is_found_by_its_architecture_key_and_round_trips(tmp_path):
    from tokamak_amd.config.registry import load_model_description
    from tokamak_amd.models.korazen import KorazenConfig, parse, to_config_json

    folder = write_folder(tmp_path / "m", CFG, random_weights(CFG, 1))
    arch, cfg, made = load_model_description(folder)
    assert arch.name == "Korazen" and isinstance(cfg, KorazenConfig) and cfg.logit_scale == 0.75
    assert parse(to_config_json(cfg)) == cfg
    assert [L.type for L in cfg.layers] == [L["type"] for L in CFG["layers"]]
    assert made.vocab_size == CFG["vocab"] and len(made.layers) == 4


def test_plan_cache_slots_and_parts():
    from tokamak_amd.models.korazen import parse, plan

    made = plan(parse(CFG))
    assert [(c.layer, c.cache) for c in made.order] == [(0, 0), (1, (1, 2)), (2, 3), (3, (4, 5))]
    for spec, layer in zip(made.layers, CFG["layers"]):
        roles = dict(spec.parts)
        assert ("feed_forward_norm" in roles) == (layer["mlp"] is not None) == ("feed_forward" in roles)
        assert ("left" in roles) == (layer["type"] == "parallel") == ("right_norm" in roles)
        assert spec.block.kind == "post_norm"
    assert "position" in dict(made.layers[1].parts) and "position" not in dict(made.layers[3].parts)
    assert made.layers[1].role("left").spec["chunk"] == 24 and made.layers[3].role("left").spec["chunk"] is None
    assert made.embedding["norm_tensor"] == ".norm" and made.head["scale"] == 0.75
    assert made.layers[2].role("feed_forward").spec["limit"] == 2.5


def test_tensor_names_and_shapes_match_a_list_written_independently():
    from tokamak_amd.models.korazen import parse, plan
    from tokamak_amd.weights.random_init import expected_tensors_of

    for cfg, ranks in ((CFG, (8, 8)), (model_json([delta(heads=3, kv_heads=1, dim=21, vdim=18, conv=3),
                                                   parallel(dict(heads=3, kv_heads=3, dim=20, vdim=40), dict(heads=5, dim=7, vdim=9))], width=72), (5, 12))):
        expected = expected_tensors_of(plan(parse(cfg)))
        shapes = tensor_shapes(cfg, ranks)
        assert set(expected) == set(shapes)
        assert all(expected[n].fits(shape) for n, shape in shapes.items())
    held = expected_tensors_of(plan(parse(CFG)))
    assert all(held[n].holding == "float32" for n in held if n.endswith((".conv", "A_log", "dt_bias", "norm", "norm1", ".b", ".out"))
               and n not in ("l0.mix.b", "l2.mix.b"))


def test_optional_keys_may_be_absent():
    from tokamak_amd.models.korazen import parse, plan

    cfg = model_json([delta(heads=3, kv_heads=3, vdim=16), parallel(dict(rot=0, chunk=None, kv_heads=4, vdim=16), dict(vdim=16), mlp=None)],
                     logit_scale=None)
    for m in (cfg["layers"][0]["mixer"], cfg["layers"][1]["mixer"]["left"]):
        m.pop("kv_heads")
        m.pop("vdim")
    cfg["layers"][1]["mixer"]["right"].pop("vdim")
    cfg["layers"][1].pop("mlp")
    parsed = parse(cfg)
    made = plan(parsed)
    assert parsed.logit_scale == 1.0 and parsed.layers[1].mlp is None
    assert (parsed.layers[0].mixer.kv_heads, parsed.layers[0].mixer.vdim) == (3, 16)
    assert made.layers[1].role("left").spec["num_kv_heads"] == 4 and made.layers[1].role("right").spec["value_dim"] == 16


@pytest.mark.parametrize("change,message", [
    (lambda c: c.update(architecture="Other"), "Unsupported architecture"),
    (lambda c: c["layers"][0].update(type="conv"), "unknown layer type"),
    (lambda c: c["layers"][2]["mlp"].update(kind="moe"), "unknown feed-forward kind"),
    (lambda c: c["layers"][0]["mixer"].update(heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5]), "one number for each"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("decay"), "decay"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][1]["mlp"].update(limit=0.0), "limit"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv"),
    (lambda c: c.pop("width"), "width"),
])
def test_what_cannot_be_a_model_is_refused(change, message):
    from tokamak_amd.models.korazen import parse

    cfg = json.loads(json.dumps(CFG))
    change(cfg)
    with pytest.raises(ValueError, match=message):
        parse(cfg)


def test_presets_build_and_shorten():
    from dataclasses import replace

    from tokamak_amd.config.registry import find_preset

    def without_ranks(cfg):
        return replace(cfg, layers=tuple(replace(L, mixer=replace(L.mixer, decay_rank=None, gate_rank=None))
                                         if L.type == "channel_delta" else L for L in cfg.layers))

    for name in ("korazen-tiny", "korazen-0.6b", "korazen-8b"):
        arch, cfg = find_preset(name)
        made = arch.plan(arch.shorten(cfg, 3))
        assert len(made.layers) == 3 and arch.parse(arch.to_json(cfg)) == without_ranks(cfg)


def test_blocks_and_norms_refuse_what_does_not_belong_together():
    from tokamak_amd.config import get_part

    make = get_part("block", "post_norm")
    norm = lambda eps=1e-5: get_part("norm", "rmsnorm")(dim=8, eps=eps, dtype=torch.float32, device="cpu")
    mixer = lambda: get_part("mixer", "fixed_decay_linear_attention")(
        hidden_size=8, num_heads=1, head_dim=4, value_dim=4, decay=(0.5,), norm_eps=1e-5, dtype=torch.float32, device="cpu")
    assert list(make(dict(mixer_norm=norm(), left=mixer(), right=mixer(), left_norm=norm(), right_norm=norm())).mixers) == ["left", "right"]
    ff = get_part("feed_forward", "swiglu")(hidden_size=8, intermediate_size=8, dtype=torch.float32, device="cpu")
    centred = get_part("norm", "layernorm")(dim=8, eps=1e-5, dtype=torch.float32, device="cpu")
    for bad in (dict(mixer_norm=norm()), dict(mixer_norm=norm(), left=mixer()), dict(mixer_norm=norm(), mixer=mixer(), left=mixer(), right=mixer()),
                dict(mixer_norm=norm(), left=mixer(), right=mixer(), left_norm=norm()), dict(mixer_norm=norm(), mixer=mixer(), feed_forward=ff),
                dict(mixer_norm=norm(), mixer=mixer(), feed_forward=ff, feed_forward_norm=norm(1e-3)), dict(mixer_norm=centred, mixer=mixer())):
        with pytest.raises(ValueError):
            make(bad)


# -- the plain implementation against formulas written another way ------------------------------
def test_delta_rule_is_the_product_of_its_corrections():
    """S_t = (I - beta k k^T) diag(g) S + beta k v^T, written with matrices."""
    g = torch.Generator().manual_seed(0)
    t, heads, dim, vdim = 9, 2, 5, 4
    q, k = torch.randn(t, heads, dim, generator=g).double(), plain.unit(torch.randn(t, heads, dim, generator=g).double())
    v, beta = torch.randn(t, heads, vdim, generator=g).double(), torch.rand(t, heads, generator=g).double()
    decay = torch.rand(t, heads, dim, generator=g).double()
    o, state = plain.delta_rule(q, k, v, beta, decay)
    for a in range(heads):
        s = torch.zeros(dim, vdim, dtype=torch.float64)
        for i in range(t):
            kk = k[i, a][:, None]
            s = (torch.eye(dim, dtype=torch.float64) - beta[i, a] * kk @ kk.T) @ torch.diag(decay[i, a]) @ s + beta[i, a] * kk @ v[i, a][None, :]
            assert torch.allclose(o[i, a], s.T @ q[i, a], atol=1e-12)
        assert torch.allclose(state[a], s, atol=1e-12)


def test_fixed_decay_scan_is_a_masked_product():
    """o_t = sum_{j <= t} decay^(t - j) (q_t . k_j) v_j."""
    g = torch.Generator().manual_seed(1)
    t = 12
    q, k, v = (torch.randn(t, 1, n, generator=g).double() for n in (5, 5, 3))
    o, _ = plain.fixed_decay_scan(q, k, v, torch.tensor([0.8], dtype=torch.float64))
    i = torch.arange(t)
    powers = torch.where(i[:, None] >= i[None, :], 0.8 ** (i[:, None] - i[None, :]).double(), torch.zeros(()).double())
    assert torch.allclose(o[:, 0], (powers * (q[:, 0] @ k[:, 0].T)) @ v[:, 0], atol=1e-12)


def test_chunks_are_counted_from_position_zero():
    mask = {"size": 7}
    seen = [[j for j in range(20) if plain.visible(i, j, mask)] for i in range(20)]
    assert seen[6] == list(range(7)) and seen[7] == [7] and seen[15] == [14, 15]
    v = torch.eye(20, dtype=torch.float64)[:, None, :]
    out = plain.softmax_attention(torch.zeros(20, 1, 4).double(), torch.zeros(20, 1, 4).double(), v, 1.0, mask)[:, 0]
    assert [row.nonzero().flatten().tolist() for row in out] == seen


def test_clamps_of_the_gate():
    g = torch.tensor([-50.0, -1.0, 0.5, 3.0, 50.0], dtype=torch.float64)
    assert torch.equal(plain.clamped_gate(g, torch.zeros(5).double(), 2.0)[3:], plain.clamped_gate(torch.full((2,), 2.0).double(), torch.zeros(2).double(), 2.0))
    assert plain.clamped_gate(g[:1], torch.zeros(1).double(), 2.0).abs() < 1e-30       # not clamped from below: the sigmoid closes it
    one = plain.clamped_gate(torch.full((3,), 1.0).double(), torch.tensor([-9.0, 0.0, 9.0]).double(), 2.0)
    assert torch.allclose(one / one[1], torch.tensor([-1.0, 1.0, 3.0]).double())


def test_every_part_of_the_plain_model_moves_its_output():
    cfg = model_json([delta(mlp=dense(24)), parallel(dict(chunk=10))])
    w = double(random_weights(cfg, 4))
    toks = tokens(cfg["vocab"], 40, 2)
    base = plain.forward(cfg, w, toks)[0]
    scale = base.abs().max()
    for name in w:
        other = dict(w)
        other[name] = w[name] * 0.5 + (0.1 if w[name].dim() == 1 else 0.0)
        if name.endswith(("mix.o", "mlp.down", "right.o", "left.o")):
            other[name] = w[name].roll(1, 0)       # (a norm stands behind it: its scale alone does not show)
        if name == "embed":
            other[name] = w[name].roll(1, 0)
        assert float((plain.forward(cfg, other, toks)[0] - base).abs().max() / scale) > 1e-3, name


def test_right_and_left_sizes_are_their_own():
    from tokamak_amd.models.korazen import parse

    cfg = parse(model_json([parallel(dict(heads=6, kv_heads=3, dim=8, vdim=24), dict(heads=5, dim=12, vdim=4))]))
    m = cfg.layers[0].mixer
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim) == (6, 3, 8, 24)
    assert (m.right.heads, m.right.dim, m.right.vdim, len(m.right.decay)) == (5, 12, 4, 5)
    assert left()["mask"]["size"] == 24 and len(right(heads=3)["decay"]) == 3
