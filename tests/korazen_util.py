"""Test-side helpers for the Korazen design: small ``config.json`` dicts written by hand, random
weights under the design's tensor names (listed here independently of the engine), model
folders, and the plain implementation's logits."""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch
from safetensors.torch import save_file

import plain_korazen as plain


def dense(ff=48, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def delta(heads=4, kv_heads=2, dim=16, vdim=24, conv=4, mlp=None):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": mlp}


def left(heads=4, kv_heads=2, dim=16, vdim=32, rot=8, scale=None, base=10000.0, chunk=24):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": float(dim) ** -0.5 if scale is None else scale}
    if rot:
        out["rot"] = {"base": base, "dims": rot}
    if chunk is not None:
        out["mask"] = {"size": chunk}
    return out


def right(heads=2, dim=16, vdim=24, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim,
            "decay": [1.0 - 0.4 ** (1 + i) for i in range(heads)] if decay is None else list(decay)}


def parallel(left_sizes=None, right_sizes=None, mlp="default"):
    return {"type": "parallel", "mixer": {"left": left(**(left_sizes or {})), "right": right(**(right_sizes or {}))},
            "mlp": dense() if mlp == "default" else mlp}


def model_json(layers, vocab=200, width=64, eps=1e-5, logit_scale=0.75):
    out = {"architecture": "Korazen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": list(layers)}
    if logit_scale is not None:
        out["logit_scale"] = logit_scale
    return out


def mixer_shapes(p, layer, W, ranks) -> dict[str, tuple]:
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        kw, vw, gw = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"], m["heads"] * m["dim"]
        ra, rg = ranks
        return {p + "q": (kw, W), p + "k": (kw, W), p + "v": (vw, W), p + "q.conv": (kw, m["conv"]), p + "k.conv": (kw, m["conv"]),
                p + "v.conv": (vw, m["conv"]), p + "b": (m["heads"], W), p + "A_log": (m["heads"],), p + "norm": (m["vdim"],),
                p + "a1": (ra, W), p + "a2": (gw, ra), p + "dt_bias": (gw,), p + "g1": (rg, W), p + "g2": (vw, rg), p + "o": (W, vw)}
    a, r = m["left"], m["right"]
    out = {}
    for n, width in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
        out.update({p + f"left.{n}": (width, W), p + f"left.{n}.b": (width,)})
    out.update({p + "left.q.norm": (a["dim"],), p + "left.k.norm": (a["dim"],), p + "left.g": (a["heads"] * a["vdim"], W),
                p + "left.o": (W, a["heads"] * a["vdim"]), p + "left.o.b": (W,), p + "left.out": (W,), p + "right.out": (W,)})
    for n, width in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"])):
        out[p + f"right.{n}"] = (width, W)
    out.update({p + "right.o": (W, r["heads"] * r["vdim"]), p + "right.norm": (r["heads"] * r["vdim"],)})
    return out


def tensor_shapes(cfg, ranks=(8, 8)) -> dict[str, tuple]:
    """Every tensor of a model, by name, written from the design's description.  ``ranks``: the low ranks of the
    decays and of the output gate, which no configuration key names."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "embed.norm": (W,), "final.norm": (W,), "head": (cfg["vocab"], W)}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        out[p + "norm1"] = (W,)
        out.update(mixer_shapes(p + "mix.", L, W, ranks))
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
    return out


def random_weights(cfg, seed, ranks=(8, 8), sharp=1.0):
    """name -> float32 tensor holding bfloat16-representable values.  Biases, decays and gates are large enough that
    leaving one out moves the output; the residual stream's first value is of order one.  ``sharp`` multiplies the
    weights of the q norms: attention then looks at few keys."""
    g = torch.Generator().manual_seed(seed)
    w = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm", "out"):
            t = 1.0 + 0.2 * torch.randn(shape, generator=g)
            if name.endswith("left.q.norm"):
                t = t * sharp
        elif name == "embed":
            t = 3.0 * torch.randn(shape, generator=g)
        elif last == "b" and len(shape) == 1:
            t = 0.5 * torch.randn(shape, generator=g)
        elif last == "dt_bias":
            t = -3.0 + 1.5 * torch.randn(shape, generator=g)
        elif last == "A_log":
            t = 0.5 * torch.randn(shape, generator=g)
        elif last == "conv":
            t = torch.randn(shape, generator=g) * 0.6
        else:
            gain = 2.0 if last in ("gate", "up") else 1.0
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


class Expected:
    """What the plain implementation says of a request: ``logits``, and per position the error that rounding to
    bfloat16 alone causes there (largest |difference| over the largest |logit|)."""

    def __init__(self, cfg, weights, tokens):
        self.logits = oracle_logits(cfg, weights, tokens)
        plain.ROUNDED = True
        try:
            rounded = oracle_logits(cfg, weights, tokens)
        finally:
            plain.ROUNDED = False
        self.noise = np.abs(rounded - self.logits).max(axis=-1) / np.abs(self.logits).max(axis=-1)


def tokens(vocab, n, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()
