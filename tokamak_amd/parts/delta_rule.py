"""The gated delta rule with a decay per key channel: a recurrence that corrects what its state holds for a key."""

from __future__ import annotations

import torch

from tokamak_amd.config.registry import register_part
from tokamak_amd.kernels import ops
from tokamak_amd.kernels.linear import linear
from tokamak_amd.parts.base import Fetch, Mixer, PositionData, StateArray
from tokamak_amd.weights.spec import TensorSpec

LOW = 8        # the low ranks are padded with rows of zeros to a multiple of this (16-byte rows of the second product)
WHOLE = 256    # ... and a large first matrix to a multiple of this (the library's tiles: 2,048 rows of 4,096 into 12,576
               # columns take 180 us, into 12,800 165)
SPLIT_FROM_ROWS = 16   # beyond so many rows the first product may be split over K (64 rows of 4,096: 29 + 3 us against 43; 8 rows level)


class ChannelDeltaRule(Mixer):
    """q = W_q h and k = W_k h (``num_kv_heads`` heads of ``head_dim``), v = W_v h (``num_heads`` heads of
    ``value_dim``); each passes a causal convolution per channel over ``conv_taps`` positions (last tap on the token
    itself, no bias, zeros before a sequence's start) and silu; q and k become unit vectors per head,
    x / sqrt(sum(x^2) + 1e-6), and q is multiplied by ``head_dim``^(-1/2).  Head a reads q/k head
    a // (heads / kv heads).  beta = sigmoid(W_b h), one per head; the decay of head a's key channel c is
    g = exp(-exp(A_log_a) softplus((W_a2 W_a1 h + dt_bias)_(a, c))).  Per head, with the state S
    [head_dim, value_dim] (zeros before a sequence's first token):

        S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

    o is divided by its root mean square per head (``norm_eps``), multiplied by ``norm`` [value_dim] (shared by the
    heads) and by sigmoid(W_g2 W_g1 h), and projected by W_o.  The request's state is S (float32, held as
    [heads, value_dim, head_dim rounded up to 4]) and the convolution's last taps - 1 inputs; everything that enters
    the recurrence behind the products is float32.  The low ranks of W_a1 and W_g1 are read off the checkpoint unless
    ``decay_rank`` and ``gate_rank`` give them.

    q, k, v, b and the two low ranks are one product of h, and the second matrices of the low ranks a second one, on a matrix that is zero where the two do not meet.
    Tensors: q, k, v with ``.conv`` each, b, A_log, norm, a1, a2, dt_bias, g1, g2, o behind the part's prefix.
    """

    capturable = True
    replayable = True

    def __init__(self, *, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 conv_taps: int, norm_eps: float, dtype, device, decay_rank: int | None = None,
                 gate_rank: int | None = None) -> None:
        super().__init__(dtype=dtype, device=device)
        if min(hidden_size, num_heads, num_kv_heads, head_dim, value_dim) < 1 or num_heads % num_kv_heads:
            raise ValueError(f"every size must be >= 1 and num_heads ({num_heads}) a multiple of num_kv_heads ({num_kv_heads})")
        if head_dim > ops.DELTA_MAX_DIM:
            raise ValueError(f"head_dim is at most {ops.DELTA_MAX_DIM} for the scan kernel, got {head_dim}")
        if not 1 <= conv_taps <= ops.SSM_MAX_TAPS:
            raise ValueError(f"the convolution has 1 to {ops.SSM_MAX_TAPS} taps, got {conv_taps}")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.head_dim, self.value_dim, self.conv_taps = int(head_dim), int(value_dim), int(conv_taps)
        self.norm_eps = float(norm_eps)
        self.decay_rank = None if decay_rank is None else int(decay_rank)
        self.gate_rank = None if gate_rank is None else int(gate_rank)
        self.conv_channels = 2 * self.num_kv_heads * self.head_dim + self.num_heads * self.value_dim
        self.first = self.up = self.o = None
        self.conv = self.a_log = self.dt_bias = self.gain = None

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        h, kw, vw = self.hidden_size, self.num_kv_heads * self.head_dim, self.num_heads * self.value_dim
        gw, taps = self.num_heads * self.head_dim, self.conv_taps
        out = {}
        for name, width in (("q", kw), ("k", kw), ("v", vw)):
            out[prefix + name] = TensorSpec((width, h))
            out[prefix + name + ".conv"] = TensorSpec((width, taps), held="float32")
        out.update({
            prefix + "b": TensorSpec((self.num_heads, h)),
            prefix + "A_log": TensorSpec((self.num_heads,), held="float32"),
            prefix + "dt_bias": TensorSpec((gw,), held="float32"),
            prefix + "a1": TensorSpec((self.decay_rank, h)), prefix + "a2": TensorSpec((gw, self.decay_rank)),
            prefix + "g1": TensorSpec((self.gate_rank, h)), prefix + "g2": TensorSpec((vw, self.gate_rank)),
            prefix + "norm": TensorSpec((self.value_dim,), role="vector"),
            prefix + "o": TensorSpec((h, vw)),
        })
        return out

    def bind(self, prefix: str, fetch: Fetch) -> None:
        self.conv = torch.cat([fetch(prefix + n + ".conv") for n in ("q", "k", "v")]).contiguous()
        self.a_log, self.dt_bias, self.gain, self.o = (fetch(prefix + n) for n in ("A_log", "dt_bias", "norm", "o"))
        a1, a2, g1, g2 = (fetch(prefix + n) for n in ("a1", "a2", "g1", "g2"))
        for name, first, second in (("decay", a1, a2), ("gate", g1, g2)):
            if second.shape[1] != first.shape[0]:
                raise ValueError(f"the two matrices of the {name} disagree on its rank: {tuple(first.shape)} and {tuple(second.shape)}")
        rows = [fetch(prefix + n) for n in ("q", "k", "v", "b")]
        ra, rg = a1.shape[0], g1.shape[0]
        self.low_at = -(-sum(t.shape[0] for t in rows) // LOW) * LOW
        self.low_width = wide = -(-(ra + rg) // LOW) * LOW
        total = self.low_at + wide
        total = -(-total // WHOLE) * WHOLE if total >= 8 * WHOLE else total
        self.first = torch.zeros((total, self.hidden_size), dtype=a1.dtype, device=a1.device)
        torch.cat(rows, out=self.first[:sum(t.shape[0] for t in rows)])
        self.first[self.low_at:self.low_at + ra], self.first[self.low_at + ra:self.low_at + ra + rg] = a1, g1
        self.up = torch.zeros((a2.shape[0] + g2.shape[0], wide), dtype=a2.dtype, device=a2.device)
        self.up[:a2.shape[0], :ra], self.up[a2.shape[0]:, ra:ra + rg] = a2, g2

    def state_request(self) -> dict[str, StateArray]:
        out = {"S": StateArray((self.num_heads, self.value_dim, -(-self.head_dim // 4) * 4), torch.float32)}
        if self.conv_taps > 1:
            out["conv"] = StateArray((self.conv_taps - 1, self.conv_channels), torch.float32)
        return out

    def forward(self, h, batch, store, writes_cache: bool = True, position: PositionData | None = None):
        n, sizes = h.shape[0], dict(heads=self.num_heads, kv_heads=self.num_kv_heads, dim=self.head_dim, vdim=self.value_dim)
        # (a split product leaves float32 partial sums, which the kernels below add as they load; the low ranks' sum is
        # a kernel of its own then, which pays from some rows on)
        proj = linear(h, self.first, allow_partials=n > SPLIT_FROM_ROWS)
        if proj.dim() == 3:
            low = torch.empty((n, self.low_width), dtype=self.dtype, device=h.device)
            ops.sum_columns(proj, self.low_at, low)
        else:
            low = proj[:, self.low_at:self.low_at + self.low_width]
        few = n <= ops.STREAM_MAX_ROWS      # (few rows: float32 from the streaming product, at no cost)
        up = linear(low, self.up, out_dtype=torch.float32 if few else None, allow_partials=True)
        operands = torch.empty((n, ops.delta_row(**sizes)), dtype=torch.float32, device=h.device)
        ops.delta_inputs(proj, up, self.conv, store.state.get("conv"), self.a_log, self.dt_bias, operands, batch,
                         q_scale=self.head_dim ** -0.5, **sizes)
        y = torch.empty((n, self.num_heads * self.value_dim), dtype=torch.float32, device=h.device)
        ops.delta_scan(operands, store.state["S"], y, batch, **sizes)
        gated = torch.empty(y.shape, dtype=self.dtype, device=h.device)
        ops.gated_group_norm(y, up, self.num_heads * self.head_dim, self.gain, gated, groups=self.num_heads,
                             eps=self.norm_eps, gate_after=True)
        return linear(gated, self.o, allow_partials=True)


register_part("mixer", "channel_delta_rule", ChannelDeltaRule)
