"""A plain, slow implementation of the Dopirax design, written from its equations: one function
per mechanism, whole sequences at a time, no cache, no kernels, nothing shared with the engine.

``cfg`` is the parsed ``config.json`` (a dict), ``w`` maps tensor names to torch tensors.  Everything
is computed in the dtype of ``DTYPE`` (float64 by default).
"""

from __future__ import annotations

import torch

DTYPE = torch.float64


def _f(t: torch.Tensor) -> torch.Tensor:
    return t.to(DTYPE)


def rms_norm(x: torch.Tensor, gain: torch.Tensor | None, eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if gain is None else y * gain


def layer_norm_of(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The norm of a layer and of the model: the stored weight is the gain less one."""
    return rms_norm(x, 1.0 + _f(weight), eps)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


# ---------------------------------------------------------------------------------------------
# positions
def rotate(x: torch.Tensor, positions: torch.Tensor, rot: dict | None, interleaved: bool) -> torch.Tensor:
    """x [T, heads, dim]; the first rot.dims dimensions rotated: pair i is (i, i + dims / 2), or (2i, 2i + 1)."""
    if not rot or not rot.get("dims"):
        return x
    dims = int(rot["dims"])
    half = dims // 2
    freqs = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(half)], dtype=DTYPE)
    angle = positions.to(DTYPE)[:, None] * freqs[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    out = x.clone()
    for i in range(half):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + half)
        u, v = x[..., a], x[..., b]
        out[..., a] = u * cos[..., i] - v * sin[..., i]
        out[..., b] = v * cos[..., i] + u * sin[..., i]
    return out


# ---------------------------------------------------------------------------------------------
# mixers
def causal_weights(scores: torch.Tensor, one_more: bool) -> torch.Tensor:
    """scores [T, T] -> the weights of the keys j <= i; ``one_more``: a term exp(0) in the denominator."""
    t = scores.shape[0]
    hidden = torch.triu(torch.ones((t, t), dtype=torch.bool), diagonal=1)
    scores = scores.masked_fill(hidden, float("-inf"))
    top = scores.max(dim=-1, keepdim=True).values
    if one_more:
        top = torch.clamp(top, min=0.0)
    e = torch.exp(scores - top)
    total = e.sum(dim=-1, keepdim=True)
    return e / (total + torch.exp(-top) if one_more else total)


def soft_cap(scores: torch.Tensor, cap: float | None) -> torch.Tensor:
    return scores if cap is None else cap * torch.tanh(scores / cap)


def attention(h: torch.Tensor, w: dict, p: str, m: dict) -> torch.Tensor:
    """The values are the unrotated keys; capped scores, a sink of score 0, one gate a head."""
    t = h.shape[0]
    heads, kv, dim = int(m["heads"]), int(m.get("kv_heads") or m["heads"]), int(m["dim"])
    pos = torch.arange(t)
    q = (h @ _f(w[p + "q"]).T + _f(w[p + "q.b"])).view(t, heads, dim)
    v = (h @ _f(w[p + "k"]).T + _f(w[p + "k.b"])).view(t, kv, dim)
    q, k = rotate(q, pos, m.get("rot"), False), rotate(v, pos, m.get("rot"), False)
    gate = sigmoid(h @ _f(w[p + "g"]).T)
    o = torch.zeros((t, heads, dim), dtype=DTYPE)
    for a in range(heads):
        g = a // (heads // kv)
        scores = soft_cap((q[:, a] @ k[:, g].T) * float(m["scale"]), m.get("softcap"))
        o[:, a] = (causal_weights(scores, True) @ v[:, g]) * gate[:, a:a + 1]
    return o.reshape(t, heads * dim) @ _f(w[p + "o"]).T + _f(w[p + "o.b"])


def keys_values(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """A differential layer's keys [T, kv heads, 2, dim] (normed, rotated) and values [T, kv heads, vdim]."""
    t = h.shape[0]
    kv, dim, vdim = int(m.get("kv_heads") or m["heads"]), int(m["dim"]), int(m["vdim"])
    k = rms_norm((h @ _f(w[p + "k"]).T).view(t, kv * 2, dim), _f(w[p + "k.norm"]), eps)
    k = rotate(k, torch.arange(t), m.get("rot"), True).view(t, kv, 2, dim)
    return k, (h @ _f(w[p + "v"]).T).view(t, kv, vdim)


def difference_weight(w: dict, p: str, m: dict) -> torch.Tensor:
    def dot(a, b):
        return (_f(w[p + a]) * _f(w[p + b])).sum()

    return torch.exp(dot("lq1", "lk1")) - torch.exp(dot("lq2", "lk2")) + float(m["diff"])


def difference(a1: torch.Tensor, a2: torch.Tensor, lam: torch.Tensor, diff: float, eps: float) -> torch.Tensor:
    return rms_norm(a1 - lam * a2, None, eps) * (1.0 - diff)


def differential_attention(h: torch.Tensor, k: torch.Tensor, v: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """``k``, ``v``: what this layer attends over (its own, or those of the layer it names)."""
    t = h.shape[0]
    heads, dim, vdim = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = rms_norm((h @ _f(w[p + "q"]).T).view(t, heads * 2, dim), _f(w[p + "q.norm"]), eps)
    q = rotate(q, torch.arange(t), m.get("rot"), True).view(t, heads, 2, dim)
    lam = difference_weight(w, p, m)
    o = torch.zeros((t, heads, vdim), dtype=DTYPE)
    for a in range(heads):
        g = a // (heads // k.shape[1])
        maps = [causal_weights((q[:, a, s] @ k[:, g, s].T) * float(m["scale"]), False) @ v[:, g] for s in (0, 1)]
        o[:, a] = difference(maps[0], maps[1], lam, float(m["diff"]), eps)
    return o.reshape(t, heads * vdim) @ _f(w[p + "o"]).T


# ---------------------------------------------------------------------------------------------
# feed-forwards
def squared_relu(h: torch.Tensor, w: dict, p: str) -> torch.Tensor:
    return torch.clamp(h @ _f(w[p + "up"]).T, min=0.0) ** 2 @ _f(w[p + "down"]).T


def gated(h: torch.Tensor, w: dict, p: str) -> torch.Tensor:
    return (silu(h @ _f(w[p + "gate"]).T) * (h @ _f(w[p + "up"]).T)) @ _f(w[p + "down"]).T


def route(h: torch.Tensor, w: dict, p: str, router: dict, margins: list | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights [T, top]).  ``margins`` receives, per token, the gap between the last
    logit taken and the first one left."""
    top = int(router["top"])
    z = h @ _f(w[p + "router"]).T + _f(w[p + "router.b"])
    ordered, order = z.sort(dim=-1, descending=True)
    if margins is not None:
        margins.extend((ordered[:, top - 1] - ordered[:, top]).tolist() if top < z.shape[1] else [float("inf")] * z.shape[0])
    e = torch.exp(ordered[:, :top] - ordered[:, :1])
    return order[:, :top], e / e.sum(dim=-1, keepdim=True)


def experts_ff(h: torch.Tensor, w: dict, p: str, mlp: dict, margins: list | None = None) -> torch.Tensor:
    chosen, weight = route(h, w, p, mlp["router"], margins)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, x in zip(chosen[i].tolist(), weight[i]):
            out[i] += x * gated(h[i:i + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + sigmoid(h @ _f(w[p + "shared.sg"]).T) * gated(h, w, p + "shared.")
    return out


def feed_forward(h: torch.Tensor, w: dict, p: str, mlp: dict | None, margins: list | None = None) -> torch.Tensor | None:
    if mlp is None:
        return None
    return squared_relu(h, w, p) if mlp["kind"] == "dense" else experts_ff(h, w, p, mlp, margins)


# ---------------------------------------------------------------------------------------------
def forward(cfg: dict, w: dict, tokens: list[int], margins: list | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """(logits [T, vocab], the residual stream after every layer [layers, T, width]).  ``margins`` receives the
    routers' narrowest choices, T numbers for every layer with a mixture of experts, in layer order."""
    eps = float(cfg["norm"]["eps"])
    x = _f(w["embed"])[torch.tensor(tokens, dtype=torch.long)] * float(cfg.get("embedding", {}).get("scale", 1.0))
    kept: dict[int, tuple] = {}
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = layer_norm_of(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            mixed = attention(h, w, p + "mix.", m)
        elif layer["type"] == "attention_2":
            source = i if m.get("kv_from") is None else int(m["kv_from"])
            if source == i:
                kept[i] = keys_values(h, w, p + "mix.", m, eps)
            mixed = differential_attention(h, *kept[source], w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        ff = feed_forward(h, w, p + "mlp.", layer.get("mlp"), margins)
        x = x + (mixed if ff is None else mixed + ff)
        after.append(x)
    logits = layer_norm_of(x, w["final.norm"], eps) @ _f(w["head"]).T
    return logits, torch.stack(after)
