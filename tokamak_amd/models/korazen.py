"""Korazen: typed config from its ``config.json`` keys, and its model plan.

A decoder-only model whose norms stand behind its sub-layers: x <- x + norm1(mixer(x)), then
x <- x + norm2(ff(x)), RMS norms; the embedding's rows pass a norm of their own.  The mixer is, layer by
layer, one of two:

* ``channel_delta``: the gated delta rule with a decay per key channel (a recurrence with a matrix state
  per head), behind short causal convolutions, with a low-rank output gate;
* ``parallel``: two mixers side by side over the same input.  Left: grouped-query attention with biases,
  weighted q/k norms ahead of a partial rotation, a chunked mask and an output gate.  Right: linear
  attention with one constant decay a head.  Half the sum of the two outputs, each normed first.

The feed-forward is a gated one with clamped halves, or absent.

    {"architecture": "Korazen", "vocab": V, "width": W, "norm": {"eps": e}, "logit_scale": a,
     "layers": [{"type": "channel_delta", "mixer": {"heads", "kv_heads", "dim", "vdim", "conv"}, "mlp": M},
                {"type": "parallel",
                 "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"},
                                    "rot": {"base", "dims"}},
                           "right": {"heads", "dim", "vdim", "decay": [one a head]}}, "mlp": M}, ...]}
    M = {"kind": "dense", "ff": F, "limit": L} | null

Tensor names: ``embed``, ``embed.norm``, ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.{q,q.conv,k,k.conv,v,v.conv,b,A_log,norm,a1,a2,dt_bias,g1,g2,o}`` or
``l<i>.mix.left.{q,q.b,q.norm,k,k.b,k.norm,v,v.b,g,o,o.b,out}`` and ``l<i>.mix.right.{q,k,v,g,norm,o,out}``,
``l<i>.mlp.{gate,up,down}``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any

from tokamak_amd.config.model_config import LayerCall, LayerSpec, ModelPlan, PartSpec, SubPart
from tokamak_amd.config.registry import Architecture, register_architecture

NAME = "Korazen"
# the design has no position table and no length of its own: the cache is the only limit
MAX_POSITIONS = 1 << 20


@dataclass(frozen=True)
class ChannelDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    # the low ranks are not configuration keys: a checkpoint's tensors give them; only the
    # random-weights mode needs numbers here
    decay_rank: int | None = None
    gate_rank: int | None = None


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int


@dataclass(frozen=True)
class ChunkedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int | None = None              # None: every earlier position is seen
    rot: RotationConfig | None = None     # None: no rotation


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]


@dataclass(frozen=True)
class ParallelConfig:
    left: ChunkedAttentionConfig
    right: LightningConfig


@dataclass(frozen=True)
class ClampedFeedForward:
    ff: int
    limit: float


@dataclass(frozen=True)
class KorazenLayer:
    mixer: ChannelDeltaConfig | ParallelConfig
    mlp: ClampedFeedForward | None        # None: the layer has no feed-forward

    @property
    def type(self) -> str:
        return "parallel" if isinstance(self.mixer, ParallelConfig) else "channel_delta"


@dataclass(frozen=True)
class KorazenConfig:
    architecture: str
    vocab_size: int
    width: int
    norm_eps: float
    layers: tuple[KorazenLayer, ...]
    logit_scale: float = 1.0
    eos_token_ids: tuple[int, ...] = ()
    max_position_embeddings: int = MAX_POSITIONS

    def __post_init__(self) -> None:
        if self.vocab_size < 1 or self.width < 1 or not self.layers:
            raise ValueError("vocab, width and the number of layers must be >= 1")
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            a = m.left if isinstance(m, ParallelConfig) else m
            if min(a.heads, a.kv_heads, a.dim, a.vdim) < 1 or a.heads % a.kv_heads:
                raise ValueError(f"layer {i}: heads ({a.heads}) must be a multiple of kv_heads ({a.kv_heads})")
            if isinstance(m, ParallelConfig):
                if a.chunk is not None and a.chunk < 1:
                    raise ValueError(f"layer {i}: mask.size must be >= 1")
                if a.rot is not None and (a.rot.dims % 2 or not 0 <= a.rot.dims <= a.dim):
                    raise ValueError(f"layer {i}: rot.dims must be even and at most {a.dim}")
                if min(m.right.heads, m.right.dim, m.right.vdim) < 1:
                    raise ValueError(f"layer {i}: every size must be >= 1")
                if len(m.right.decay) != m.right.heads:
                    raise ValueError(f"layer {i}: decay holds one number for each of the {m.right.heads} heads")
            elif m.conv < 1:
                raise ValueError(f"layer {i}: conv must be >= 1")
            if layer.mlp is not None and (layer.mlp.ff < 1 or not layer.mlp.limit > 0):
                raise ValueError(f"layer {i}: ff must be >= 1 and limit positive")

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


def _mlp(raw: Any, where: str) -> ClampedFeedForward | None:
    if raw is None:
        return None
    kind = _need(raw, "kind", where)
    if kind != "dense":
        raise ValueError(f"{where}: unknown feed-forward kind {kind!r}; this design has 'dense'")
    return ClampedFeedForward(ff=int(_need(raw, "ff", where)), limit=float(_need(raw, "limit", where)))


def _heads(m: Any, where: str) -> dict[str, int]:
    heads, dim = int(_need(m, "heads", where)), int(_need(m, "dim", where))
    return {"heads": heads, "kv_heads": int(m["kv_heads"]) if m.get("kv_heads") is not None else heads, "dim": dim,
            "vdim": int(m["vdim"]) if m.get("vdim") is not None else dim}


def _layer(raw: Any, i: int) -> KorazenLayer:
    where = f"layers[{i}]"
    kind = _need(raw, "type", where)
    m = _need(raw, "mixer", where)
    mw = where + ".mixer"
    if kind == "channel_delta":
        mixer: ChannelDeltaConfig | ParallelConfig = ChannelDeltaConfig(**_heads(m, mw), conv=int(_need(m, "conv", mw)))
    elif kind == "parallel":
        left, right = _need(m, "left", mw), _need(m, "right", mw)
        mask, rot, sizes = left.get("mask"), left.get("rot"), _heads(right, mw + ".right")
        mixer = ParallelConfig(
            left=ChunkedAttentionConfig(
                **_heads(left, mw + ".left"), scale=float(_need(left, "scale", mw + ".left")),
                chunk=None if mask is None else int(_need(mask, "size", mw + ".left.mask")),
                rot=None if rot is None else RotationConfig(base=float(_need(rot, "base", mw + ".left.rot")),
                                                            dims=int(_need(rot, "dims", mw + ".left.rot")))),
            right=LightningConfig(heads=sizes["heads"], dim=sizes["dim"], vdim=sizes["vdim"],
                                  decay=tuple(float(x) for x in _need(right, "decay", mw + ".right"))))
    else:
        raise ValueError(f"{where}: unknown layer type {kind!r}; this design has 'channel_delta' and 'parallel'")
    return KorazenLayer(mixer=mixer, mlp=_mlp(raw.get("mlp"), where + ".mlp"))


def parse(raw: dict[str, Any], eos_token_ids: tuple[int, ...] = ()) -> KorazenConfig:
    name = raw.get("architecture")
    if name != NAME:
        raise ValueError(f"Unsupported architecture {name!r}; supported: {NAME}")
    layers = _need(raw, "layers", "config.json")
    return KorazenConfig(
        architecture=NAME,
        vocab_size=int(_need(raw, "vocab", "config.json")),
        width=int(_need(raw, "width", "config.json")),
        norm_eps=float(_need(_need(raw, "norm", "config.json"), "eps", "norm")),
        layers=tuple(_layer(layer, i) for i, layer in enumerate(layers)),
        logit_scale=float(raw["logit_scale"]) if raw.get("logit_scale") is not None else 1.0,
        eos_token_ids=tuple(int(t) for t in eos_token_ids),
    )


def _mixer_json(m: ChannelDeltaConfig | ParallelConfig) -> dict[str, Any]:
    if isinstance(m, ChannelDeltaConfig):
        return {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}
    a = m.left
    left: dict[str, Any] = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
    if a.chunk is not None:
        left["mask"] = {"size": a.chunk}
    if a.rot is not None:
        left["rot"] = {"base": a.rot.base, "dims": a.rot.dims}
    return {"left": left, "right": {"heads": m.right.heads, "dim": m.right.dim, "vdim": m.right.vdim, "decay": list(m.right.decay)}}


def to_config_json(cfg: KorazenConfig) -> dict[str, Any]:
    """The ``config.json`` dict that parses back to ``cfg`` (the low ranks are not keys: the tensors carry them)."""
    return {
        "architecture": cfg.architecture,
        "vocab": cfg.vocab_size,
        "width": cfg.width,
        "norm": {"eps": cfg.norm_eps},
        "logit_scale": cfg.logit_scale,
        "layers": [{"type": L.type, "mixer": _mixer_json(L.mixer),
                    "mlp": None if L.mlp is None else {"kind": "dense", "ff": L.mlp.ff, "limit": L.mlp.limit}}
                   for L in cfg.layers],
    }


def run_order(cfg: KorazenConfig) -> tuple[LayerCall, ...]:
    """Each layer once; a layer with two mixers brings a cache slot for each (the attention's pages, the
    recurrence's state)."""
    order, slot = [], 0
    for i, L in enumerate(cfg.layers):
        if isinstance(L.mixer, ParallelConfig):
            order.append(LayerCall(i, (slot, slot + 1)))
            slot += 2
        else:
            order.append(LayerCall(i, slot))
            slot += 1
    return tuple(order)


def plan(cfg: KorazenConfig) -> ModelPlan:
    width = cfg.width
    norm = PartSpec.of("rmsnorm", dim=width, eps=cfg.norm_eps, tensor="")
    layers = []
    for L in cfg.layers:
        m = L.mixer
        parts = dict(mixer_norm=SubPart("norm", norm, "norm1"))
        if isinstance(m, ChannelDeltaConfig):
            parts["mixer"] = SubPart("mixer", PartSpec.of(
                "channel_delta_rule", hidden_size=width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim,
                value_dim=m.vdim, conv_taps=m.conv, norm_eps=cfg.norm_eps, decay_rank=m.decay_rank,
                gate_rank=m.gate_rank), "mix.")
        else:
            a, r = m.left, m.right
            parts["left"] = SubPart("mixer", PartSpec.of(
                "rotated_unit_attention", hidden_size=width, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim,
                value_dim=a.vdim, softmax_scale=a.scale, norm_eps=cfg.norm_eps, chunk=a.chunk, norm_first=True,
                norm_names=("q.norm", "k.norm"), bias_suffix=".b", gate_name="g"), "mix.left.")
            parts["right"] = SubPart("mixer", PartSpec.of(
                "fixed_decay_linear_attention", hidden_size=width, num_heads=r.heads, head_dim=r.dim, value_dim=r.vdim,
                decay=r.decay, norm_eps=cfg.norm_eps), "mix.right.")
            parts["left_norm"] = SubPart("norm", norm, "mix.left.out")
            parts["right_norm"] = SubPart("norm", norm, "mix.right.out")
            if a.rot is not None and a.rot.dims > 0:
                parts["position"] = SubPart("position", PartSpec.of(
                    "rotary_half", rotary_dim=a.rot.dims, theta=a.rot.base), shared=True)
        if L.mlp is not None:
            parts["feed_forward"] = SubPart("feed_forward", PartSpec.of(
                "swiglu", hidden_size=width, intermediate_size=L.mlp.ff, names=("gate", "up", "down"),
                activation="clamped", limit=L.mlp.limit), "mlp.")
            parts["feed_forward_norm"] = SubPart("norm", norm, "norm2")
        layers.append(LayerSpec.of(PartSpec.of("post_norm", left_weight=0.5, right_weight=0.5), **parts))
    return ModelPlan(
        vocab_size=cfg.vocab_size,
        hidden_size=width,
        max_position_embeddings=cfg.max_position_embeddings,
        tie_word_embeddings=False,
        embedding=PartSpec.of("token_embedding", vocab_size=cfg.vocab_size, dim=width, tensor="", norm_eps=cfg.norm_eps,
                              norm_tensor=".norm"),
        layers=tuple(layers),
        order=run_order(cfg),
        final_norm=norm,
        head=PartSpec.of("linear_head", vocab_size=cfg.vocab_size, dim=width, tied=False, tensor="", scale=cfg.logit_scale),
        embedding_prefix="embed",
        layer_prefix="l{}.",
        final_norm_prefix="final.norm",
        head_prefix="head",
        eos_token_ids=cfg.eos_token_ids,
    )


def _shape(vocab, width, repeats, *, heads, kv, dim, delta_kv, delta_dim, delta_heads, rank, chunk, right_heads, right_dim,
           ff) -> KorazenConfig:
    """``repeats`` times (delta rule, parallel, delta rule, delta rule); every layer but a stretch's last one has a
    feed-forward."""
    mlp = ClampedFeedForward(ff, 7.0)
    delta = ChannelDeltaConfig(delta_heads, delta_kv, delta_dim, delta_dim, 4, rank, rank)
    par = ParallelConfig(
        ChunkedAttentionConfig(heads, kv, dim, dim, float(dim) ** -0.5, chunk, RotationConfig(5e5, dim // 2)),
        LightningConfig(right_heads, right_dim, right_dim, tuple(1.0 - 2.0 ** -(2 + 6.0 * i / right_heads) for i in range(right_heads))))
    stretch = (KorazenLayer(delta, mlp), KorazenLayer(par, mlp), KorazenLayer(delta, mlp), KorazenLayer(delta, None))
    return KorazenConfig(NAME, vocab, width, 1e-5, stretch * repeats, logit_scale=0.5)


# Shapes for the random-weights mode (sizes only; no trained weights exist here): a tiny one, and layers
# of the widths of 0.6B- and 8B-class models for measurements.
PRESETS = {
    "korazen-tiny": _shape(256, 64, 1, heads=4, kv=2, dim=16, delta_kv=2, delta_dim=16, delta_heads=4, rank=8, chunk=24,
                           right_heads=2, right_dim=16, ff=96),
    "korazen-0.6b": _shape(151936, 1024, 7, heads=16, kv=4, dim=128, delta_kv=8, delta_dim=128, delta_heads=8, rank=64,
                           chunk=1024, right_heads=16, right_dim=64, ff=3072),
    "korazen-8b": _shape(151936, 4096, 9, heads=32, kv=8, dim=128, delta_kv=32, delta_dim=128, delta_heads=32, rank=128,
                         chunk=1024, right_heads=64, right_dim=64, ff=12288),
}


def shorten(cfg: KorazenConfig, num_layers: int) -> KorazenConfig:
    return replace(cfg, layers=cfg.layers[:num_layers])


register_architecture(Architecture(name=NAME, parse=parse, plan=plan, to_json=to_config_json, presets=PRESETS,
                                   shorten=shorten))
