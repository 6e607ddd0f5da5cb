"""Test-side helpers for the Dopirax design: small ``config.json`` dicts written by hand, random
weights under the design's tensor names (listed here independently of the engine), model
folders, and the plain implementation's logits."""

from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors.torch import save_file

import plain_dopirax as plain


def experts(n=8, top=2, ff=32, shared=24):
    out = {"kind": "moe", "router": {"experts": n, "top": top}, "expert": {"ff": ff}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def dense(ff=48):
    return {"kind": "dense", "ff": ff}


def _rot(mixer, rot, base):
    if rot:
        mixer["rot"] = {"base": base, "dims": rot}


def capped(heads=4, kv_heads=2, dim=16, rot=16, scale=None, base=20000.0, softcap=15.0, mlp="default"):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": float(dim) ** -0.5 if scale is None else scale}
    if softcap is not None:
        mixer["softcap"] = softcap
    _rot(mixer, rot, base)
    return {"type": "attention", "mixer": mixer, "mlp": experts() if mlp == "default" else mlp}


def differential(heads=2, kv_heads=1, dim=16, vdim=24, rot=8, scale=None, base=8000.0, diff=0.45, kv_from=None, mlp="default"):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
             "scale": float(dim) ** -0.5 if scale is None else scale}
    _rot(mixer, rot, base)
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention_2", "mixer": mixer, "mlp": experts() if mlp == "default" else mlp}


def model_json(layers, vocab=200, width=64, eps=1e-5, scale=3.0):
    out = {"architecture": "Dopirax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}
    if scale is not None:
        out["embedding"] = {"scale": scale}
    return out


def tensor_shapes(cfg) -> dict[str, tuple]:
    """Every tensor of a model, by name, written from the design's description."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,), "head": (cfg["vocab"], W)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        heads, dim = m["heads"], m["dim"]
        kv = m.get("kv_heads") or heads
        own = m.get("kv_from") is None
        out[p + "norm1"] = (W,)
        if L["type"] == "attention":
            out.update({p + "mix.q": (heads * dim, W), p + "mix.q.b": (heads * dim,), p + "mix.g": (heads, W),
                        p + "mix.o": (W, heads * dim), p + "mix.o.b": (W,)})
            if own:
                out.update({p + "mix.k": (kv * dim, W), p + "mix.k.b": (kv * dim,)})
        else:
            out.update({p + "mix.q": (heads * 2 * dim, W), p + "mix.q.norm": (dim,), p + "mix.o": (W, heads * m["vdim"])})
            out.update({p + f"mix.{name}": (dim,) for name in ("lq1", "lk1", "lq2", "lk2")})
            if own:
                out.update({p + "mix.k": (kv * 2 * dim, W), p + "mix.k.norm": (dim,), p + "mix.v": (kv * m["vdim"], W)})
        mlp = L["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            out.update({p + "mlp.up": (mlp["ff"], W), p + "mlp.down": (W, mlp["ff"])})
            continue
        out.update({p + "mlp.router": (mlp["router"]["experts"], W), p + "mlp.router.b": (mlp["router"]["experts"],)})
        members = {f"e{e}.": mlp["expert"]["ff"] for e in range(mlp["router"]["experts"])}
        if mlp.get("shared"):
            members["shared."] = mlp["shared"]["ff"]
            out[p + "mlp.shared.sg"] = (1, W)
        for name, ff in members.items():
            out.update({p + f"mlp.{name}gate": (ff, W), p + f"mlp.{name}up": (ff, W), p + f"mlp.{name}down": (W, ff)})
    return out


def random_weights(cfg, seed):
    """name -> float32 tensor holding bfloat16-representable values.  Biases, gates and the vectors of lambda are
    large enough that leaving one out moves the output."""
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        if name == "final.norm" or last == "norm1":
            t = 0.2 * torch.randn(shape, generator=g)              # (stored around zero)
        elif last == "norm":
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
        elif name == "embed":
            t = torch.randn(shape, generator=g)
        elif last == "b":
            t = 0.5 * torch.randn(shape, generator=g)
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.4 * torch.randn(shape, generator=g) * shape[0] ** -0.25
        else:
            gain = 2.0 if last in ("router", "gate", "up", "g", "sg") else 1.0
            t = torch.randn(shape, generator=g) * gain * shape[1] ** -0.5
        w[name] = t.to(torch.bfloat16).float()
    return w


def write_folder(folder, cfg, weights) -> Path:
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg, indent=1))
    save_file({n: t.to(torch.bfloat16).contiguous() for n, t in weights.items()}, str(folder / "model.safetensors"))
    return folder


def double(w):
    return {k: v.double() for k, v in w.items()}


def oracle_logits(cfg, weights, tokens):
    return plain.forward(cfg, double(weights), list(tokens))[0].float().numpy()


def oracle_with_margins(cfg, weights, tokens):
    """(logits, per position the narrowest choice of a router in any layer)."""
    margins: list[float] = []
    logits = plain.forward(cfg, double(weights), list(tokens), margins=margins)[0].float().numpy()
    routed = sum(1 for L in cfg["layers"] if L["mlp"] is not None and L["mlp"]["kind"] == "moe")
    n = len(tokens)
    per_position = [min((margins[layer * n + t] for layer in range(routed)), default=float("inf")) for t in range(n)]
    return logits, per_position


def every_expert(cfg):
    """The same model with every expert chosen for every token: no choice that rounding could turn."""
    out = json.loads(json.dumps(cfg))
    for layer in out["layers"]:
        if layer["mlp"] is not None and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return out


def tokens(vocab, n, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()
