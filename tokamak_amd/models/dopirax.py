"""Dopirax: typed config from its ``config.json`` keys, and its model plan.

A decoder-only model whose layers are parallel: one RMS norm (its weight stored less one) whose output
both the mixer and the feed-forward read, x <- x + (mixer(h) + ff(h)); the embedding's rows are scaled.
The mixer is, layer by layer, one of two:

* ``attention``: grouped-query attention whose values are its keys before rotation (no W_v), biases on
  q, k and o, half-split rotation, scores under a soft cap, one added to the softmax's denominator, and
  a gate of one number a head;
* ``attention_2``: differential attention: two maps a head over the same values, with weighted norms of q
  and k ahead of an interleaved rotation; the second map's output times lambda is subtracted from the
  first's, and the head is normed and scaled.  A layer with ``kv_from``: j has no keys and values of its
  own and attends over layer j's.

The feed-forward is W_down relu(W_up h)^2, a mixture of small SiLU-gated experts (logits with a bias, the
chosen experts weighted by the softmax over the chosen logits, optionally a shared expert with a gate of
one number a token), or absent.

    {"architecture": "Dopirax", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s},
     "layers": [{"type": "attention",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "softcap", "rot": {"base", "dims"}}, "mlp": M},
                {"type": "attention_2",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "diff", "rot": {"base", "dims"}, "kv_from": j},
                 "mlp": M}, ...]}
    M = {"kind": "dense", "ff": F}
      | {"kind": "moe", "router": {"experts", "top"}, "expert": {"ff"}, "shared": {"ff"}} | null

Tensor names: ``embed``, ``l<i>.norm1``, ``l<i>.mix.{q,q.b,k,k.b,g,o,o.b}`` or
``l<i>.mix.{q,q.norm,k,k.norm,v,lq1,lk1,lq2,lk2,o}``, ``l<i>.mlp.{up,down}`` or ``l<i>.mlp.{router,router.b}``,
``l<i>.mlp.e<j>.{gate,up,down}`` and ``l<i>.mlp.shared.{gate,up,down,sg}``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any

from tokamak_amd.config.model_config import LayerCall, LayerSpec, ModelPlan, PartSpec, SubPart
from tokamak_amd.config.registry import Architecture, register_architecture

NAME = "Dopirax"
# the design has no position table and no length of its own: the cache is the only limit
MAX_POSITIONS = 1 << 20


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int


@dataclass(frozen=True)
class CappedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    softcap: float | None = None          # None: the scores are not bounded
    rot: RotationConfig | None = None     # None: no rotation
    kv_from: int | None = None            # the layer over whose keys and values this one attends


@dataclass(frozen=True)
class DifferentialConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    rot: RotationConfig | None = None
    kv_from: int | None = None


@dataclass(frozen=True)
class DenseFeedForward:
    ff: int


@dataclass(frozen=True)
class ExpertsFeedForward:
    experts: int
    top: int
    ff: int
    shared_ff: int | None = None


Mixer = CappedAttentionConfig | DifferentialConfig
KINDS = {CappedAttentionConfig: "attention", DifferentialConfig: "attention_2"}


@dataclass(frozen=True)
class DopiraxLayer:
    mixer: Mixer
    mlp: DenseFeedForward | ExpertsFeedForward | None     # None: the layer has no feed-forward

    @property
    def type(self) -> str:
        return KINDS[type(self.mixer)]


def _stored(m: Mixer) -> tuple:
    """What two layers must agree on if one attends over what the other has stored."""
    return type(m), m.kv_heads, m.dim, getattr(m, "vdim", m.dim)


@dataclass(frozen=True)
class DopiraxConfig:
    architecture: str
    vocab_size: int
    width: int
    norm_eps: float
    layers: tuple[DopiraxLayer, ...]
    embedding_scale: float = 1.0
    eos_token_ids: tuple[int, ...] = ()
    max_position_embeddings: int = MAX_POSITIONS

    def __post_init__(self) -> None:
        if self.vocab_size < 1 or self.width < 1 or not self.layers:
            raise ValueError("vocab, width and the number of layers must be >= 1")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if min(m.heads, m.kv_heads, m.dim, getattr(m, "vdim", 1)) < 1 or m.heads % m.kv_heads:
                raise ValueError(f"layer {i}: heads ({m.heads}) must be a multiple of kv_heads ({m.kv_heads}), every size >= 1")
            if m.rot is not None and (m.rot.dims % 2 or not 0 <= m.rot.dims <= m.dim):
                raise ValueError(f"layer {i}: rot.dims must be even and at most {m.dim}")
            if isinstance(m, CappedAttentionConfig) and m.softcap is not None and not m.softcap > 0:
                raise ValueError(f"layer {i}: softcap must be positive")
            if m.kv_from is not None:
                src = self.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
                if src is None or src.kv_from is not None or _stored(src) != _stored(m):
                    raise ValueError(f"layer {i}: kv_from must name an earlier layer of the same type with keys and values "
                                     f"of its own and the same kv_heads, dim and vdim")
            f = layer.mlp
            if isinstance(f, DenseFeedForward) and f.ff < 1:
                raise ValueError(f"layer {i}: ff must be >= 1")
            if isinstance(f, ExpertsFeedForward) and (
                    f.ff < 1 or not 1 <= f.top <= f.experts or (f.shared_ff is not None and f.shared_ff < 1)):
                raise ValueError(f"layer {i}: ff >= 1 and 1 <= top <= experts are required")

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_layers(self) -> int:
        return len(self.layers)


def _need(raw: Any, key: str, where: str) -> Any:
    if not isinstance(raw, dict) or key not in raw or raw[key] is None:
        raise ValueError(f"config.json lacks required key {key!r} in {where}")
    return raw[key]


def _optional(raw: dict, key: str, kind, default=None):
    return default if raw.get(key) is None else kind(raw[key])


def _mlp(raw: Any, where: str) -> DenseFeedForward | ExpertsFeedForward | None:
    if raw is None:
        return None
    kind = _need(raw, "kind", where)
    if kind == "dense":
        return DenseFeedForward(ff=int(_need(raw, "ff", where)))
    if kind == "moe":
        router, shared = _need(raw, "router", where), raw.get("shared")
        return ExpertsFeedForward(
            experts=int(_need(router, "experts", where + ".router")), top=int(_need(router, "top", where + ".router")),
            ff=int(_need(_need(raw, "expert", where), "ff", where + ".expert")),
            shared_ff=None if shared is None else int(_need(shared, "ff", where + ".shared")))
    raise ValueError(f"{where}: unknown feed-forward kind {kind!r}; this design has 'dense' and 'moe'")


def _layer(raw: Any, i: int) -> DopiraxLayer:
    where = f"layers[{i}]"
    kind = _need(raw, "type", where)
    m = _need(raw, "mixer", where)
    mw = where + ".mixer"
    if kind not in KINDS.values():
        raise ValueError(f"{where}: unknown layer type {kind!r}; this design has 'attention' and 'attention_2'")
    heads, dim, rot = int(_need(m, "heads", mw)), int(_need(m, "dim", mw)), m.get("rot")
    vdim = _optional(m, "vdim", int, dim)
    common = dict(
        heads=heads, kv_heads=_optional(m, "kv_heads", int, heads), dim=dim, scale=float(_need(m, "scale", mw)),
        rot=None if rot is None else RotationConfig(base=float(_need(rot, "base", mw + ".rot")),
                                                    dims=int(_need(rot, "dims", mw + ".rot"))),
        kv_from=_optional(m, "kv_from", int))
    if kind == "attention":
        if vdim != dim:
            raise ValueError(f"{where}: the values of 'attention' are its keys: vdim ({vdim}) must be dim ({dim})")
        mixer: Mixer = CappedAttentionConfig(**common, softcap=_optional(m, "softcap", float))
    else:
        mixer = DifferentialConfig(**common, vdim=vdim, diff=float(_need(m, "diff", mw)))
    return DopiraxLayer(mixer=mixer, mlp=_mlp(raw.get("mlp"), where + ".mlp"))


def parse(raw: dict[str, Any], eos_token_ids: tuple[int, ...] = ()) -> DopiraxConfig:
    name = raw.get("architecture")
    if name != NAME:
        raise ValueError(f"Unsupported architecture {name!r}; supported: {NAME}")
    layers = _need(raw, "layers", "config.json")
    return DopiraxConfig(
        architecture=NAME,
        vocab_size=int(_need(raw, "vocab", "config.json")),
        width=int(_need(raw, "width", "config.json")),
        norm_eps=float(_need(_need(raw, "norm", "config.json"), "eps", "norm")),
        layers=tuple(_layer(layer, i) for i, layer in enumerate(layers)),
        embedding_scale=_optional(raw.get("embedding") or {}, "scale", float, 1.0),
        eos_token_ids=tuple(int(t) for t in eos_token_ids),
    )


def _mixer_json(m: Mixer) -> dict[str, Any]:
    out: dict[str, Any] = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "scale": m.scale}
    if isinstance(m, CappedAttentionConfig):
        out["vdim"] = m.dim
        if m.softcap is not None:
            out["softcap"] = m.softcap
    else:
        out.update(vdim=m.vdim, diff=m.diff)
    if m.rot is not None:
        out["rot"] = {"base": m.rot.base, "dims": m.rot.dims}
    if m.kv_from is not None:
        out["kv_from"] = m.kv_from
    return out


def _mlp_json(mlp: DenseFeedForward | ExpertsFeedForward | None) -> dict[str, Any] | None:
    if mlp is None:
        return None
    if isinstance(mlp, DenseFeedForward):
        return {"kind": "dense", "ff": mlp.ff}
    out: dict[str, Any] = {"kind": "moe", "router": {"experts": mlp.experts, "top": mlp.top}, "expert": {"ff": mlp.ff}}
    if mlp.shared_ff is not None:
        out["shared"] = {"ff": mlp.shared_ff}
    return out


def to_config_json(cfg: DopiraxConfig) -> dict[str, Any]:
    """The ``config.json`` dict that parses back to ``cfg``."""
    return {
        "architecture": cfg.architecture,
        "vocab": cfg.vocab_size,
        "width": cfg.width,
        "norm": {"eps": cfg.norm_eps},
        "embedding": {"scale": cfg.embedding_scale},
        "layers": [{"type": L.type, "mixer": _mixer_json(L.mixer), "mlp": _mlp_json(L.mlp)} for L in cfg.layers],
    }


def run_order(cfg: DopiraxConfig) -> tuple[LayerCall, ...]:
    """Each layer once; a layer with ``kv_from`` reads the cache slot of the layer it names and writes none."""
    return tuple(LayerCall(i, i) if L.mixer.kv_from is None else LayerCall(i, L.mixer.kv_from, writes_cache=False)
                 for i, L in enumerate(cfg.layers))


def plan(cfg: DopiraxConfig) -> ModelPlan:
    width = cfg.width
    norm = PartSpec.of("rmsnorm", dim=width, eps=cfg.norm_eps, tensor="", offset=1.0)
    layers = []
    for L in cfg.layers:
        m = L.mixer
        parts = dict(norm=SubPart("norm", norm, "norm1"))
        common = dict(hidden_size=width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, softmax_scale=m.scale,
                      chunk=None, own_keys=m.kv_from is None)
        if isinstance(m, CappedAttentionConfig):
            parts["mixer"] = SubPart("mixer", PartSpec.of(
                "rotated_unit_attention", **common, value_dim=m.dim, norm_eps=None, values_are_keys=True, bias_suffix=".b",
                softcap=m.softcap, unit_sink=True, gate_name="g", gate_per_head=True), "mix.")
        else:
            parts["mixer"] = SubPart("mixer", PartSpec.of(
                "differential_attention", **common, value_dim=m.vdim, norm_eps=cfg.norm_eps, norm_first=True,
                norm_names=("q.norm", "k.norm"), difference=m.diff, output_eps=cfg.norm_eps), "mix.")
        if m.rot is not None and m.rot.dims > 0:
            parts["position"] = SubPart("position", PartSpec.of(
                "rotary_half" if isinstance(m, CappedAttentionConfig) else "rotary_interleaved", rotary_dim=m.rot.dims,
                theta=m.rot.base), shared=True)
        if isinstance(L.mlp, DenseFeedForward):
            parts["feed_forward"] = SubPart("feed_forward", PartSpec.of(
                "activated", hidden_size=width, intermediate_size=L.mlp.ff, names=("up", "down"), activation="squared_relu"), "mlp.")
        elif isinstance(L.mlp, ExpertsFeedForward):
            f = L.mlp
            parts["feed_forward"] = SubPart("feed_forward", PartSpec.of(
                "routed_experts", hidden_size=width, intermediate_size=f.ff, num_experts=f.experts, top=f.top,
                weight_on="output", scoring="chosen_softmax", logit_bias="router.b", shared_size=f.shared_ff,
                shared_gate=None if f.shared_ff is None else "sg"), "mlp.")
        layers.append(LayerSpec.of(PartSpec.of("parallel_sublayers"), **parts))
    return ModelPlan(
        vocab_size=cfg.vocab_size,
        hidden_size=width,
        max_position_embeddings=cfg.max_position_embeddings,
        tie_word_embeddings=False,
        embedding=PartSpec.of("token_embedding", vocab_size=cfg.vocab_size, dim=width, tensor="", scale=cfg.embedding_scale),
        layers=tuple(layers),
        order=run_order(cfg),
        final_norm=norm,
        head=PartSpec.of("linear_head", vocab_size=cfg.vocab_size, dim=width, tied=False, tensor=""),
        embedding_prefix="embed",
        layer_prefix="l{}.",
        final_norm_prefix="final.norm",
        head_prefix="head",
        eos_token_ids=cfg.eos_token_ids,
    )


def _shape(vocab, width, repeats, *, heads, kv, dim, diff_heads, diff_kv, diff_dim, vdim, ff, experts, top, expert_ff,
           shared_ff) -> DopiraxConfig:
    """``repeats`` times (differential, capped, differential over the first one's keys, capped); the model's first
    feed-forward is dense, the others are mixtures of experts."""
    att = CappedAttentionConfig(heads, kv, dim, float(dim) ** -0.5, 30.0, RotationConfig(5e5, dim))
    moe = ExpertsFeedForward(experts, top, expert_ff, shared_ff)
    layers: list[DopiraxLayer] = []
    for r in range(repeats):
        own = DifferentialConfig(diff_heads, diff_kv, diff_dim, vdim, float(diff_dim) ** -0.5, 0.5, RotationConfig(1e4, diff_dim))
        first = len(layers)
        layers += [DopiraxLayer(own, DenseFeedForward(ff) if r == 0 else moe), DopiraxLayer(att, moe),
                   DopiraxLayer(replace(own, kv_from=first), moe), DopiraxLayer(att, moe)]
    return DopiraxConfig(NAME, vocab, width, 1e-5, tuple(layers), embedding_scale=8.0)


# Shapes for the random-weights mode (sizes only; no trained weights exist here): a tiny one, and layers of
# the widths of 0.6B- and 8B-class models for measurements (a token's experts together with the shared one are
# about as wide as the dense feed-forward of that class; a differential head has two maps of half a head's
# keys, so that a cached key and value are as wide as the other attention's).
PRESETS = {
    "dopirax-tiny": _shape(256, 64, 1, heads=4, kv=2, dim=16, diff_heads=2, diff_kv=1, diff_dim=8, vdim=16, ff=96, experts=8,
                           top=2, expert_ff=32, shared_ff=48),
    "dopirax-0.6b": _shape(151936, 1024, 7, heads=16, kv=8, dim=128, diff_heads=8, diff_kv=4, diff_dim=64, vdim=128, ff=3072,
                           experts=16, top=2, expert_ff=1024, shared_ff=1024),
    "dopirax-8b": _shape(151936, 4096, 9, heads=32, kv=8, dim=128, diff_heads=32, diff_kv=8, diff_dim=64, vdim=128, ff=12288,
                         experts=16, top=2, expert_ff=4096, shared_ff=4096),
}


def shorten(cfg: DopiraxConfig, num_layers: int) -> DopiraxConfig:
    """The model's first ``num_layers`` layers (a source of keys comes ahead of the layers that name it)."""
    return replace(cfg, layers=cfg.layers[:num_layers])


register_architecture(Architecture(name=NAME, parse=parse, plan=plan, to_json=to_config_json, presets=PRESETS,
                                   shorten=shorten))
