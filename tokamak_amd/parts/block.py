"""Arrangements of a layer's parts."""

from __future__ import annotations

from tokamak_amd.config.registry import register_part
from tokamak_amd.kernels.linear import Added, StreamSink
from tokamak_amd.parts.base import Block, BranchPair, NormedSum
from tokamak_amd.parts.norm import read_stream
from tokamak_amd.parts.scale import scaled_sum


class PreNormBlock(Block):
    """x = x + mixer(norm(x)); x = x + feed_forward(norm(x))
    (reference: src/tokamak/model/transformer.py:107-108).

    The residual stream ``resid`` is float32.  Each sub-layer's output is left
    ``pending`` and added by the next norm's fused kernel, so the sum is formed
    in float32 and the stream is written once per sub-layer.  Parts that can
    (``fuses_residual``) are offered the stream itself, so that in a decode step
    of few rows their last product adds into it and the next product finishes
    the norm, with no kernel in between.  An optional ``position`` part prepares
    the step's position data for the mixer.  The feed-forward and its norm may be
    absent together: the layer is then x = x + mixer(norm(x)) alone.
    """

    roles = ("mixer_norm", "mixer")
    optional = ("position", "feed_forward_norm", "feed_forward")
    fuses_residual = True
    replays_parts = True

    def __init__(self, parts) -> None:
        super().__init__(parts)
        self.mixer_norm = parts["mixer_norm"]
        self.feed_forward_norm = parts.get("feed_forward_norm")
        self.feed_forward = parts.get("feed_forward")
        if (self.feed_forward is None) != (self.feed_forward_norm is None):
            raise ValueError("a feed-forward and its norm come together")
        self.position = parts.get("position")
        self.entry_norm = self.mixer_norm

    def forward(self, resid, pending, batch, store, writes_cache, then=None):
        position = None if self.position is None else self.position.prepare(batch)
        h = _normed(self.mixer_norm, resid, pending, self.mixer)
        if self.feed_forward is None:
            return self.mixer.forward(h, batch, store, writes_cache, position, **_sink(self.mixer, then, resid))
        into = _sink(self.mixer, self.feed_forward_norm, resid)
        pending = self.mixer.forward(h, batch, store, writes_cache, position, **into)
        h = _normed(self.feed_forward_norm, resid, pending, self.feed_forward)
        into = _sink(self.feed_forward, then, resid)
        return _whole(self.feed_forward.forward(h, batch, **into))


def _whole(out):
    """A feed-forward's output as one pending sub-layer output (its terms, if it has several, as a pair)."""
    return BranchPair.of(*out) if isinstance(out, tuple) else out


def _normed(norm, resid, pending, consumer):
    """norm(resid + pending) for ``consumer``; left for the consumer to finish if both know how."""
    if norm.fuses_residual:
        return norm.forward(resid, pending, defer=consumer.fuses_residual)
    return norm.forward(resid, None if isinstance(pending, Added) else pending)


def _sink(producer, next_norm, resid) -> dict:
    """The keyword with which ``producer`` is offered the stream, if it can use it."""
    if not producer.fuses_residual:
        return {}
    if next_norm is not None and next_norm.fuses_residual:
        return {"add_into": next_norm.sink(resid)}
    return {"add_into": StreamSink(resid, None)}


class ParallelMixersBlock(Block):
    """x = x + scale_1 * (left_weight * left(norm(x)) + right_weight * right(norm(x)));
    x = x + scale_2 * feed_forward(norm(x)).

    Two mixers side by side read the same normed input, each with a cache slot of its own.
    ``mixer_scale`` and ``feed_forward_scale`` are per-coordinate layer scales (absent: ones);
    the feed-forward with its norm and scale may be absent altogether.  The weighted sum and
    the layer scale are formed in float32 from the branches' products, and the norm that reads
    the stream next adds the result into it.
    """

    roles = ("mixer_norm", "left", "right")
    optional = ("mixer_scale", "feed_forward_norm", "feed_forward", "feed_forward_scale")
    replays_parts = True

    def __init__(self, parts, *, left_weight: float = 1.0, right_weight: float = 1.0) -> None:
        super().__init__(parts)
        self.left_weight, self.right_weight = float(left_weight), float(right_weight)
        self.mixer_norm, self.left, self.right = parts["mixer_norm"], parts["left"], parts["right"]
        self.mixer_scale = parts.get("mixer_scale")
        self.feed_forward = parts.get("feed_forward")
        self.feed_forward_norm = parts.get("feed_forward_norm")
        self.feed_forward_scale = parts.get("feed_forward_scale")
        if (self.feed_forward is None) != (self.feed_forward_norm is None):
            raise ValueError("a feed-forward and its norm come together")
        if self.feed_forward is None and self.feed_forward_scale is not None:
            raise ValueError("a feed-forward scale without a feed-forward")
        self.entry_norm = self.mixer_norm

    def forward(self, resid, pending, batch, store, writes_cache):
        h = self.mixer_norm.forward(resid, pending)
        left = self.left.forward(h, batch, store["left"], writes_cache, None)
        right = self.right.forward(h, batch, store["right"], writes_cache, None)
        dim, dtype = resid.shape[1], h.dtype
        weight = None if self.mixer_scale is None else self.mixer_scale.weight
        pending = scaled_sum(left, self.left_weight, right, self.right_weight, weight, dim, dtype)
        if self.feed_forward is None:
            return pending
        h = self.feed_forward_norm.forward(resid, pending)
        out = self.feed_forward.forward(h, batch)
        if self.feed_forward_scale is None:
            return out
        return scaled_sum(out, 1.0, None, 0.0, self.feed_forward_scale.weight, dim, dtype)


class ParallelSublayersBlock(Block):
    """h = norm(x); x = x + branch_scale * (mixer(h) + feed_forward(h)).

    The mixer and the feed-forward read the same stream, and their outputs are added to each other
    first and to the residual stream once, in float32, by the norm that reads the stream next (it
    receives them as a ``BranchPair``).  With a ``feed_forward_norm`` the feed-forward has a norm of
    its own over the same x: x = x + branch_scale * (mixer(norm(x)) + feed_forward(feed_forward_norm(x)));
    where the two norms agree on everything but their weights one kernel makes both outputs.  The
    feed-forward may be absent: x = x + branch_scale * mixer(h).  A feed-forward may return two terms
    (routed and shared experts), and it or the mixer may leave a bias of its last product to the add (``output_bias``;
    the add takes one: with two the mixer adds its own).
    An optional ``position`` part prepares the step's position data for the mixer.
    """

    roles = ("norm", "mixer")
    optional = ("position", "feed_forward", "feed_forward_norm")
    replays_parts = True

    def __init__(self, parts, *, branch_scale: float = 1.0) -> None:
        super().__init__(parts)
        self.branch_scale = float(branch_scale)
        self.norm = parts["norm"]
        self.feed_forward = parts.get("feed_forward")
        self.feed_forward_norm = parts.get("feed_forward_norm")
        if self.feed_forward_norm is not None and self.feed_forward is None:
            raise ValueError("a feed-forward norm without a feed-forward")
        self.position = parts.get("position")
        self.entry_norm = self.norm

    def _normed(self, resid, pending):
        """(the mixer's input, the feed-forward's)."""
        if self.feed_forward_norm is None:
            h = self.norm.forward(resid, pending)
            return h, h
        pair = getattr(self.norm, "forward_pair", None)
        both = pair(self.feed_forward_norm, resid, pending) if pair is not None else None
        if both is not None:
            return both
        h = self.norm.forward(resid, pending)
        return h, self.feed_forward_norm.forward(resid, None)

    def forward(self, resid, pending, batch, store, writes_cache):
        position = None if self.position is None else self.position.prepare(batch)
        h, h_ff = self._normed(resid, pending)
        if getattr(self.feed_forward, "output_bias", None) is None:
            mixed, bias = _biasless(self.mixer, h, batch, store, writes_cache, position)
        else:
            mixed, bias = self.mixer.forward(h, batch, store, writes_cache, position), None
        if self.feed_forward is None:
            if bias is None and self.branch_scale == 1.0:
                return mixed
            return BranchPair(mixed, bias=bias, scale=self.branch_scale)
        out, ff_bias = _biasless(self.feed_forward, h_ff, batch)
        terms = out if isinstance(out, tuple) else (out,)
        if len(terms) > 2:
            raise ValueError("a feed-forward hands on two terms at most")
        return BranchPair.of(mixed, *terms, bias=bias if ff_bias is None else ff_bias, scale=self.branch_scale)


class PostNormBlock(Block):
    """x = x + mixer_norm(mixer(x)); x = x + feed_forward_norm(feed_forward(x)).

    The norms stand behind the sub-layers, which read the stream itself (rounded to the compute dtype).  A sub-layer's
    output is left pending as a ``NormedSum``: one kernel norms it, adds it to the float32 stream and writes what
    the next sub-layer reads (or, behind the last layer, norms the sum for the head).

    Instead of one ``mixer`` there may be two side by side, ``left`` and ``right``, each with a cache slot of its
    own; then mixer(x) = ``left_weight`` left_norm(left(x)) + ``right_weight`` right_norm(right(x)), the two norms and
    the norm of their sum in the same kernel (both norms or neither; they and the layer's own share one eps).  A left
    or single mixer, or a feed-forward, that leaves a bias of its last product to the add says so (``output_bias``,
    ``forward(defer_bias=True)``).  The feed-forward and its norm may be absent together.  An optional ``position``
    part prepares the step's position data for the mixers.
    """

    roles = ("mixer_norm",)
    optional = ("mixer", "left", "right", "left_norm", "right_norm", "position", "feed_forward_norm", "feed_forward")
    replays_parts = True

    def __init__(self, parts, *, left_weight: float = 0.5, right_weight: float = 0.5) -> None:
        super().__init__(parts)
        self.left_weight, self.right_weight = float(left_weight), float(right_weight)
        self.mixer_norm, self.position = parts["mixer_norm"], parts.get("position")
        self.left, self.right = parts.get("mixer", parts.get("left")), parts.get("right")
        self.left_norm, self.right_norm = parts.get("left_norm"), parts.get("right_norm")
        self.feed_forward, self.feed_forward_norm = parts.get("feed_forward"), parts.get("feed_forward_norm")
        if ("mixer" in parts) == ("left" in parts) or ("left" in parts) != ("right" in parts):
            raise ValueError("a layer has one mixer, or a left and a right one")
        if (self.left_norm is None) != (self.right_norm is None) or (self.left_norm is not None and self.right is None):
            raise ValueError("the norms of two mixers' outputs come together")
        if (self.feed_forward is None) != (self.feed_forward_norm is None):
            raise ValueError("a feed-forward and its norm come together")
        norms = [n for n in (self.mixer_norm, self.left_norm, self.right_norm, self.feed_forward_norm) if n is not None]
        if any(getattr(n, "weight_only", False) is not True or n.eps != self.mixer_norm.eps for n in norms):
            raise ValueError("the norms behind the sub-layers are RMS norms with one eps")

    def forward(self, resid, pending, batch, store, writes_cache):
        position = None if self.position is None else self.position.prepare(batch)
        h = read_stream(resid, pending, self.mixer_norm.dtype)
        if self.right is None:
            mixed, bias = _biasless(self.left, h, batch, store, writes_cache, position)
            pending = NormedSum(mixed, bias=bias, gain=self.mixer_norm.weight, eps=self.mixer_norm.eps)
        else:
            left, bias = _biasless(self.left, h, batch, store["left"], writes_cache, position)
            right = self.right.forward(h, batch, store["right"], writes_cache, position)
            pending = NormedSum(left, right, bias=bias, gain=self.mixer_norm.weight, eps=self.mixer_norm.eps,
                                first_gain=None if self.left_norm is None else self.left_norm.weight,
                                second_gain=None if self.right_norm is None else self.right_norm.weight,
                                first_weight=self.left_weight, second_weight=self.right_weight)
        if self.feed_forward is None:
            return pending
        h = read_stream(resid, pending, self.feed_forward_norm.dtype)
        out, bias = _biasless(self.feed_forward, h, batch)
        first, second = out if isinstance(out, tuple) else (out, None)
        return NormedSum(first, second, bias=bias, gain=self.feed_forward_norm.weight, eps=self.feed_forward_norm.eps)


def _biasless(part, *args):
    """(the part's output, the bias of its last product if it leaves that to the add)."""
    bias = getattr(part, "output_bias", None)
    return (part.forward(*args), None) if bias is None else (part.forward(*args, defer_bias=True), bias)


register_part("block", "pre_norm", PreNormBlock)
register_part("block", "post_norm", PostNormBlock)
register_part("block", "parallel_sublayers", ParallelSublayersBlock)
register_part("block", "parallel_mixers", ParallelMixersBlock)
