"""How norm, mixer and feed-forward are arranged in a layer (reference models/qwen3.py:55-74)."""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import (Biased, FeedForward, Mixer, Norm, ParamSpec, Part, PendingNorm, ScaledSum, Settled, StreamSum, TermSum, few_tokens,
                   register_part, side_branch)


def one_tensor(x):
    """A sublayer's output as one tensor: a tuple of outputs (`FeedForward.forward`) becomes their float32 sum."""
    if not isinstance(x, (tuple, list)):
        return x
    total = None
    for t in x:
        v = t.float().sum(0) if t.dim() == 3 else t.float()
        total = v if total is None else total + v
    return total


def settled(h, residual):
    """(h, residual) with a `ScaledSum`, `StreamSum` or `TermSum` in place of h turned into a `Settled` stream."""
    if isinstance(h, (ScaledSum, StreamSum, TermSum)):
        return Settled(None), h.settle(residual)
    return h, residual


def with_start(h, residual, start):
    """(h, residual) of a layer, with `start` added to the stream: (a `TermSum`, residual)."""
    if isinstance(h, (ScaledSum, StreamSum)):
        h, residual = settled(h, residual)
    if isinstance(h, Settled):
        return TermSum([start]), residual
    if isinstance(h, TermSum):
        return h.with_term(start), residual
    return TermSum((list(h) if isinstance(h, (tuple, list)) else [h]) + [start]), residual


def norm_of(norm: Norm, x, residual):
    """Run a norm on x, which may be float32 partial sums [P, T, n] of a split product (a norm
    that does not declare `accepts_partials` gets their sum) or a `TermSum`."""
    if isinstance(x, TermSum):
        return x.normed(norm, residual)
    x = one_tensor(x)
    if x.dim() == 3 and not getattr(norm, "accepts_partials", False):
        x = x.sum(0)
    return norm.forward(x, residual)


@register_part("block", "pre_norm")
class PreNormBlock(Part):
    """residual += input; x = norm1(residual); a = mixer(x); residual += a; x = norm2(residual);
    return feed_forward(x), residual.

    The layer's output is added to the residual by whoever runs next: the next block's first
    norm or the model's final norm (reference models/qwen3.py:65-74: the add lives inside the
    norm call). The residual stream is float32. A feed-forward that returns several terms, or rows with a
    bias to be added, leaves them as a `TermSum`: the norm that runs next adds them in its own pass.
    """

    def __init__(self, norm1: Norm, mixer: Mixer, norm2: Norm | None, feed_forward: FeedForward | None):
        """Without a feed-forward (and its norm) the layer is its first half: the mixer's output is what is left to add."""
        super().__init__()
        if (norm2 is None) != (feed_forward is None):
            raise ValueError("a feed-forward and its norm come together")
        self.add_child("norm1", norm1)
        self.add_child("mixer", mixer)
        if feed_forward is not None:
            self.add_child("norm2", norm2)
            self.add_child("feed_forward", feed_forward)
            feed_forward.defer_bias = True
        else:
            self.norm2 = self.feed_forward = None

    def cache_need(self):
        return self.mixer.cache_need()

    def state_need(self):
        return self.mixer.state_need()

    def forward(self, h, residual, step, cache, state):
        if not isinstance(h, TermSum):
            h, residual = settled(h, residual)
        if isinstance(h, Settled):          # the layer before has added its output already: the stream starts anew here
            h, residual = residual, None
        # a part that takes it gets the norm before it as a `PendingNorm` and may run it inside its first product
        if getattr(self.mixer, "takes_pending_norm", False):
            x = PendingNorm(self.norm1, h, residual)
            a = self.mixer.forward(x, step, cache, state)
            residual = x.new_residual()
        else:
            x, residual = norm_of(self.norm1, h, residual)
            a = self.mixer.forward(x, step, cache, state)
        if self.feed_forward is None:
            return a, residual
        if getattr(self.feed_forward, "takes_pending_norm", False):
            x = PendingNorm(self.norm2, a, residual)
            out = self.feed_forward.forward(x)
            return _left_to_add(out), x.new_residual()
        x, residual = norm_of(self.norm2, a, residual)
        return _left_to_add(self.feed_forward.forward(x)), residual


def _left_to_add(out):
    if isinstance(out, (tuple, list, Biased)):
        return TermSum(list(out) if isinstance(out, (tuple, list)) else [out])
    return out


@register_part("block", "output_norm")
class OutputNormBlock(Part):
    """stream += norm1(mixer(stream)); stream += norm2(feed_forward(stream)): the norms sit on the sublayers'
    outputs only, and the sublayers read the stream itself (rounded to the compute dtype). Without a
    feed-forward the layer is its first half. The stream is float32; each sum and each norm is one kernel
    that also hands on the rounded stream."""

    def __init__(self, norm1: Norm, mixer: Mixer, norm2: Norm | None = None, feed_forward: FeedForward | None = None):
        super().__init__()
        if (norm2 is None) != (feed_forward is None):
            raise ValueError("a feed-forward and its norm come together")
        self.add_child("norm1", norm1)
        self.add_child("mixer", mixer)
        if feed_forward is not None:
            self.add_child("norm2", norm2)
            self.add_child("feed_forward", feed_forward)
        else:
            self.norm2 = self.feed_forward = None

    def cache_need(self):
        return self.mixer.cache_need()

    def state_need(self):
        return self.mixer.state_need()

    def forward(self, h, residual, step, cache, state):
        h, residual = settled(h, residual)
        if isinstance(h, Settled):
            x, stream = (h.rounded if h.rounded is not None else residual.to(self.norm1.out_dtype)), residual
        elif residual is None:               # the first layer: the embedding's rows are the stream
            x, stream = h, h.float()
        else:                                # behind a layer that leaves its output to be added
            stream = residual + (h.sum(0) if h.dim() == 3 else h).float()
            x = stream.to(h.dtype if h.dim() == 2 else self.norm1.out_dtype)
        if getattr(self.mixer, "returns_terms", False) and hasattr(self.norm1, "add_terms"):
            # a mixer that is a weighted sum of several outputs: sum, norm and residual sum as one kernel
            x, stream = self.norm1.add_terms(self.mixer.forward(x, step, cache, state, terms=True), stream)
        else:
            x, stream = self.norm1.add_to(self.mixer.forward(x, step, cache, state), stream)
        if self.feed_forward is not None:
            x, stream = self.norm2.add_to(one_tensor(self.feed_forward.forward(x)), stream)
        return Settled(x), stream


def _ones(shape, generator, device):
    return 1.0 + 0.2 * (torch.rand(shape, generator=generator, dtype=torch.float32, device=device) - 0.5)


@register_part("block", "parallel")
class ParallelBlock(Part):
    """stream += mult * (scale1 * mixer(norm1(stream)) + scale2 * feed_forward(norm2(stream))): both sublayers read
    the same stream, each through a norm of its own, and each output is multiplied element by element by a learned
    scale before the sum (`layer_scale`; without it the scales are 1). Without a feed-forward the layer is its first
    half. The two norms share the stream's root mean square and are one kernel; that kernel also forms the sum the
    layer before has left (`ScaledSum`), so a stack of such layers costs one pass over the stream per layer. The
    stream is float32.

    In steps of few tokens (`base.SIDE_BRANCH_MAX_TOKENS`), where a layer is a chain of short launches, the feed-forward
    runs on a second stream beside the mixer (`base.side_branch`): the two meet again before the layer returns, so a
    captured step holds them as two branches of its graph. What the second stream allocates is read on the first only
    behind that meeting, and written again only behind the next layer's parting, which follows the kernel that read it."""

    def __init__(self, norm1: Norm, mixer: Mixer, norm2: Norm | None = None, feed_forward: FeedForward | None = None,
                 residual_mult: float = 1.0, layer_scale: bool = False):
        super().__init__()
        if (norm2 is None) != (feed_forward is None):
            raise ValueError("a feed-forward and its norm come together")
        for norm in (norm1, norm2):
            if norm is not None and (not hasattr(norm, "weight") or not hasattr(norm, "eps") or getattr(norm, "one_plus", False)):
                raise ValueError("the parallel block runs plain RMS norms (weight and eps) inside its own kernel")
        if norm2 is not None and (norm2.eps != norm1.eps or norm2.size != norm1.size):
            raise ValueError("the two norms of a parallel block share one eps and one width")
        self.residual_mult = float(residual_mult)
        self.layer_scale = bool(layer_scale)
        self.add_child("norm1", norm1)
        self.add_child("mixer", mixer)
        if feed_forward is not None:
            self.add_child("norm2", norm2)
            self.add_child("feed_forward", feed_forward)
        else:
            self.norm2 = self.feed_forward = None
        if layer_scale:
            self.add_param("scale1", ParamSpec((norm1.size,), init=_ones, dtype="float32"))
            if feed_forward is not None:
                self.add_param("scale2", ParamSpec((norm1.size,), init=_ones, dtype="float32"))
        else:
            self.scale1 = self.scale2 = None

    def cache_need(self):
        return self.mixer.cache_need()

    def state_need(self):
        return self.mixer.state_need()

    def forward(self, h, residual, step, cache, state):
        if isinstance(h, TermSum):
            h, residual = settled(h, residual)
        if isinstance(h, ScaledSum):
            stream, terms, mult = residual, h.terms, h.mult
        elif isinstance(h, Settled):
            stream, terms, mult = residual, [], 1.0
        elif residual is None:               # the first layer: the embedding's rows are the stream
            stream, terms, mult = h, [], 1.0
        else:                                # behind a layer that leaves its output to be added
            stream, terms, mult = residual, [(one_tensor(h), None)], 1.0
        w2 = self.norm2.weight if self.feed_forward is not None else None
        stream, x1, x2 = ops.scaled_sum_norm(stream, terms, mult, self.norm1.weight, w2, self.norm1.eps, self.norm1.out_dtype)
        b = None
        if self.feed_forward is not None and few_tokens(x1):
            with side_branch(x1.device, 1) as branch:
                b = self.feed_forward.forward(x2)
            out = [(self.mixer.forward(x1, step, cache, state), self.scale1)]
            branch.join()
        else:
            out = [(self.mixer.forward(x1, step, cache, state), self.scale1)]
            if self.feed_forward is not None:
                b = self.feed_forward.forward(x2)
        if b is not None:
            out += [(t, self.scale2 if self.layer_scale else None) for t in (b if isinstance(b, (tuple, list)) else (b,))]
        return ScaledSum(out, self.residual_mult), stream


def _near_even(shape, generator, device):
    """Shares of streams that start near the plain residual sum: 1/S each, give or take."""
    return (1.0 + 0.2 * (torch.rand(shape, generator=generator, dtype=torch.float32, device=device) - 0.5)) / shape[0]


def _near_identity(shape, generator, device):
    return torch.eye(shape[0], device=device) + 0.1 * (torch.rand(shape, generator=generator, dtype=torch.float32, device=device) - 0.5)


@register_part("block", "hyper_connected")
class HyperConnectedBlock(Part):
    """Instead of one residual stream `streams` of them, x_1 .. x_S, all equal at the model's start. Each sublayer has
    learned shares: it reads u = sum_s read[s] x_s through its norm, and when it has run, all streams at once from the old
    ones, x_t <- sum_s mix[s, t] x_s + out[t] * y (mix is indexed from, to). Without a feed-forward the layer is its
    mixer's half. The streams are float32 [T, S, n]; behind the last layer the residual is their sum.

    What a sublayer leaves is added by whoever runs next (`StreamSum`), in one kernel with what that one reads and its
    norm (`ops.stream_mix_norm`): per sublayer one pass over the streams, and the terms of a sublayer's output (partial
    sums of a split product, one partial sum per chosen expert, a shared expert's rows) are added up inside that pass. The
    norms may be of any kind that has `row_norm`."""

    def __init__(self, streams: int, norm1: Norm, mixer: Mixer, norm2: Norm | None = None, feed_forward: FeedForward | None = None):
        super().__init__()
        if streams < 1:
            raise ValueError("a positive number of streams")
        if (norm2 is None) != (feed_forward is None):
            raise ValueError("a feed-forward and its norm come together")
        for norm in (norm1, norm2):
            if norm is not None and not hasattr(norm, "row_norm"):
                raise ValueError("the norms run inside the block's own kernel and need `row_norm`")
        self.streams = int(streams)
        self.add_child("norm1", norm1)
        self.add_child("mixer", mixer)
        if feed_forward is not None:
            self.add_child("norm2", norm2)
            self.add_child("feed_forward", feed_forward)
        else:
            self.norm2 = self.feed_forward = None
        for i in (1, 2) if feed_forward is not None else (1,):
            self.add_param(f"read{i}", ParamSpec((streams,), init=_near_even, dtype="float32"))
            self.add_param(f"out{i}", ParamSpec((streams,), init=_ones, dtype="float32"))
            self.add_param(f"mix{i}", ParamSpec((streams, streams), init=_near_identity, dtype="float32"))

    def cache_need(self):
        return self.mixer.cache_need()

    def state_need(self):
        return self.mixer.state_need()

    def _read(self, h, streams, read, norm):
        """The streams with what waits in h added, and the normed rows that the next sublayer reads."""
        terms, mix, out = (h.terms, h.mix, h.out) if isinstance(h, StreamSum) else ([], None, None)
        new, x = ops.stream_mix_norm(streams, self.streams, terms, mix, out, read, norm.row_norm(), norm.out_dtype,
                                     keep=streams.dim() == 3 or bool(terms))
        return (streams if new is None else new), x

    def forward(self, h, residual, step, cache, state):
        if isinstance(h, StreamSum):
            streams = residual
        elif residual is None:               # the first layer: the embedding's rows are every stream
            streams, h = h, None
        else:                                # behind a layer of another kind: its stream, with what waits to be added, is every stream
            h, residual = settled(h, residual)
            streams, h = (residual if isinstance(h, Settled) else residual + one_tensor(h)), None
        streams, x = self._read(h, streams, self.read1, self.norm1)
        h = StreamSum(_terms(self.mixer.forward(x, step, cache, state)), self.mix1, self.out1)
        if self.feed_forward is not None:
            streams, x = self._read(h, streams, self.read2, self.norm2)
            h = StreamSum(_terms(self.feed_forward.forward(x)), self.mix2, self.out2)
        return h, streams


def _terms(y) -> list:
    return list(y) if isinstance(y, (tuple, list)) else [y]
