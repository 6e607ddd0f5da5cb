"""A plain, slow implementation of the Korazen design, written from its equations: one function
per mechanism, whole sequences at a time, no cache, no kernels, nothing shared with the engine.

``cfg`` is the parsed ``config.json`` (a dict), ``w`` maps tensor names to torch tensors.  Everything
is computed in the dtype of ``DTYPE`` (float64 by default).  With ``ROUNDED`` set the rows that enter a
product with a weight matrix and those that leave it are rounded to bfloat16: how far that alone moves a
logit is what a bfloat16 engine's error at that position is measured with.
"""

from __future__ import annotations

import torch

DTYPE = torch.float64
ROUNDED = False


def _f(t: torch.Tensor) -> torch.Tensor:
    return t.to(DTYPE)


def product(x: torch.Tensor, matrix: torch.Tensor) -> torch.Tensor:
    """x @ matrix^T for rows x [T, in] and a matrix [out, in]."""
    if not ROUNDED:
        return x @ _f(matrix).T
    return (x.to(torch.bfloat16).to(DTYPE) @ _f(matrix).T).to(torch.bfloat16).to(DTYPE)


def rms_norm(x: torch.Tensor, weight: torch.Tensor | None, eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * _f(weight)


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * torch.sigmoid(x)


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


# ---------------------------------------------------------------------------------------------
# the delta-rule mixer
def causal_conv(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """x [T, C], weight [C, taps]: y_t = sum_j weight[:, j] x_(t - taps + 1 + j), zeros before the start."""
    t, taps = x.shape[0], weight.shape[1]
    padded = torch.cat([torch.zeros((taps - 1, x.shape[1]), dtype=DTYPE), x], dim=0)
    out = torch.zeros_like(x)
    for j in range(taps):
        out = out + padded[j:j + t, :] * _f(weight)[:, j][None, :]
    return out


def delta_operands(h: torch.Tensor, w: dict, p: str, m: dict):
    """(q, k [T, heads, dim], v [T, heads, vdim], beta [T, heads], decay [T, heads, dim])."""
    t = h.shape[0]
    heads, kv, dim, vdim = int(m["heads"]), int(m.get("kv_heads") or m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(causal_conv(product(h, w[p + n]), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k, v = q.view(t, kv, dim), k.view(t, kv, dim), v.view(t, heads, vdim)
    q, k = unit(q) * dim ** -0.5, unit(k)
    of_head = [a // (heads // kv) for a in range(heads)]
    beta = torch.sigmoid(product(h, w[p + "b"]))
    step = softplus(product(product(h, w[p + "a1"]), w[p + "a2"]) + _f(w[p + "dt_bias"])).view(t, heads, dim)
    decay = torch.exp(-torch.exp(_f(w[p + "A_log"]))[None, :, None] * step)
    return q[:, of_head], k[:, of_head], v, beta, decay


def delta_rule(q, k, v, beta, decay, state=None):
    """(o [T, heads, vdim], the state [heads, dim, vdim] after the last token)."""
    t, heads, dim = q.shape
    s = torch.zeros((heads, dim, v.shape[-1]), dtype=DTYPE) if state is None else state
    out = []
    for i in range(t):
        s = decay[i][:, :, None] * s
        seen = (s * k[i][:, :, None]).sum(dim=1)
        u = beta[i][:, None] * (v[i] - seen)
        s = s + k[i][:, :, None] * u[:, None, :]
        out.append((s * q[i][:, :, None]).sum(dim=1))
    return torch.stack(out), s


def channel_delta(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    t = h.shape[0]
    o, _ = delta_rule(*delta_operands(h, w, p, m))
    gate = torch.sigmoid(product(product(h, w[p + "g1"]), w[p + "g2"]))
    return product(rms_norm(o, w[p + "norm"], eps).reshape(t, -1) * gate, w[p + "o"])


# ---------------------------------------------------------------------------------------------
# the left mixer: chunked attention
def rotate(x: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x [T, heads, dim]; the first rot.dims dimensions rotated, dimension i paired with i + dims / 2."""
    if not rot or not rot.get("dims"):
        return x
    dims, base = int(rot["dims"]), float(rot["base"])
    half = dims // 2
    freqs = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=DTYPE)
    angle = torch.arange(x.shape[0], dtype=DTYPE)[:, None] * freqs[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def visible(i: int, j: int, mask: dict | None) -> bool:
    return j <= i and (not mask or i // int(mask["size"]) == j // int(mask["size"]))


def softmax_attention(q, k, v, scale: float, mask: dict | None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head a reads kv head a // (H / G)."""
    t, heads, _ = q.shape
    per = heads // k.shape[1]
    i = torch.arange(t)
    allowed = i[None, :] <= i[:, None]
    if mask:
        allowed &= (i[None, :] // int(mask["size"])) == (i[:, None] // int(mask["size"]))
    out = torch.zeros((t, heads, v.shape[-1]), dtype=DTYPE)
    for a in range(heads):
        scores = (q[:, a, :] @ k[:, a // per, :].T) * scale
        out[:, a, :] = torch.softmax(scores.masked_fill(~allowed, float("-inf")), dim=-1) @ v[:, a // per, :]
    return out


def chunked_attention(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    t = h.shape[0]
    heads, kv, dim, vdim = int(m["heads"]), int(m.get("kv_heads") or m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (product(h, w[p + n]) + _f(w[p + n + ".b"]) for n in ("q", "k", "v"))
    q = rotate(rms_norm(q.view(t, heads, dim), w[p + "q.norm"], eps), m.get("rot"))
    k = rotate(rms_norm(k.view(t, kv, dim), w[p + "k.norm"], eps), m.get("rot"))
    o = softmax_attention(q, k, v.view(t, kv, vdim), float(m["scale"]), m.get("mask")).reshape(t, heads * vdim)
    return product(o * torch.sigmoid(product(h, w[p + "g"])), w[p + "o"]) + _f(w[p + "o.b"])


# ---------------------------------------------------------------------------------------------
# the right mixer: linear attention with a fixed decay a head
def fixed_decay_scan(q, k, v, decay, state=None):
    """q, k [T, heads, dim], v [T, heads, vdim], decay [heads] -> (o [T, heads, vdim], the last state)."""
    t, heads, dim = q.shape
    s = torch.zeros((heads, dim, v.shape[-1]), dtype=DTYPE) if state is None else state
    out = []
    for i in range(t):
        s = decay[:, None, None] * s + k[i][:, :, None] * v[i][:, None, :]
        out.append((s * q[i][:, :, None]).sum(dim=1))
    return torch.stack(out), s


def lightning_attention(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    t = h.shape[0]
    heads, dim, vdim = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(product(h, w[p + n])).view(t, heads, dim) for n in ("q", "k"))
    v = silu(product(h, w[p + "v"])).view(t, heads, vdim)
    o, _ = fixed_decay_scan(q, k, v, torch.tensor([float(x) for x in m["decay"]], dtype=DTYPE))
    y = rms_norm(o.reshape(t, heads * vdim), w[p + "norm"], eps) * torch.sigmoid(product(h, w[p + "g"]))
    return product(y, w[p + "o"])


def parallel(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    left = chunked_attention(h, w, p + "left.", m["left"], eps)
    right = lightning_attention(h, w, p + "right.", m["right"], eps)
    return 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))


# ---------------------------------------------------------------------------------------------
def clamped_gate(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h: torch.Tensor, w: dict, p: str, mlp: dict) -> torch.Tensor:
    return product(clamped_gate(product(h, w[p + "gate"]), product(h, w[p + "up"]), float(mlp["limit"])), w[p + "down"])


def embedding(w: dict, tokens: list[int], eps: float) -> torch.Tensor:
    return rms_norm(_f(w["embed"])[torch.tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)


def forward(cfg: dict, w: dict, tokens: list[int]) -> tuple[torch.Tensor, torch.Tensor]:
    """(logits [T, vocab], the residual stream after every layer [layers, T, width])."""
    eps = float(cfg["norm"]["eps"])
    x = embedding(w, tokens, eps)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixer = {"channel_delta": channel_delta, "parallel": parallel}[layer["type"]]
        x = x + rms_norm(mixer(x, w, p + "mix.", layer["mixer"], eps), w[p + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + rms_norm(feed_forward(x, w, p + "mlp.", layer["mlp"]), w[p + "norm2"], eps)
        after.append(x)
    logits = product(rms_norm(x, w["final.norm"], eps), w["head"]) * float(cfg.get("logit_scale", 1.0))
    return logits, torch.stack(after)
