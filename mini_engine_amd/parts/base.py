"""What every model part is: a small tree of named parameters plus a forward.

A model is assembled from parts (mixer, feed-forward, norm, position encoding,
embedding/head, block arrangement). A part takes its sizes and constants as
constructor arguments, declares the parameters it needs (`ParamSpec`), and never
learns which model it sits in. The weight loader fills declared parameters by
name; the step function hands each part the per-step metadata it may need.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Iterator

import torch


@dataclass(frozen=True)
class ParamSpec:
    """One parameter tensor of a part.

    ``init`` names the distribution used by the random-weights mode:
    ``"matrix"`` ~ N(0, 0.02) (linears, embeddings), ``"norm"`` ~ 1 + U(-0.1, 0.1); or it is a
    function ``(shape, generator, device) -> float32 tensor`` for a parameter that wants another start
    (a decay rate in (0, 1), a table of integers, ...): it draws from `generator` only, so that the
    values depend on the seed alone.
    ``dtype`` is ``"compute"`` (the engine's dtype: bfloat16 or float32),
    ``"float32"`` (always 32-bit: norm weights, exact for both stored forms),
    ``"int32"`` (integer tables) or ``"stored"`` (what the checkpoint holds: bfloat16
    stays bfloat16, 32-bit stays 32-bit).
    """

    shape: tuple
    init: object = "matrix"       # "matrix", "norm" or a function (shape, generator, device) -> tensor
    dtype: str = "compute"


PAGE = "page"      # stands in a PageTensor's shape for the axis that counts a page's tokens


@dataclass(frozen=True)
class PageTensor:
    """One tensor a mixer keeps per cached token. `shape` is what one page of one layer call looks
    like, with PAGE where the page's tokens are counted: keys stored token by token under their head
    are (heads, PAGE, head size); values transposed inside a page are (heads, head size, PAGE); one
    latent vector per token is (PAGE, width). The pool allocates [pages, *shape] with PAGE replaced by
    the engine's page size. `dtype`: "compute" (the engine's), "float32", "bfloat16" or "int32"."""

    name: str
    shape: tuple
    dtype: str = "compute"

    def __post_init__(self):
        if sum(1 for d in self.shape if d == PAGE) != 1:
            raise ValueError(f"page tensor {self.name!r}: exactly one axis of {self.shape} must be PAGE")

    def sized(self, page_size: int) -> tuple:
        return tuple(page_size if d == PAGE else int(d) for d in self.shape)


@dataclass(frozen=True)
class CacheNeed:
    """What a mixer wants from the paged cache: which tensors per token, and for how long.

    ``window``: n keeps the last n positions; ``chunk``: c keeps the positions of the block of c
    positions (counted from 0) that the next token falls into; neither: every token stays. Pages that
    the rule has passed are given back. ``keep_first``: the first so many positions stay whatever the
    rule has passed. ``readers``: the rules of other layer calls that read these
    pages (the model fills it in): the loosest of all rules holds. Layers with equal needs share one
    group of pages and one block table per request.
    """

    tensors: tuple                     # of PageTensor
    window: int | None = None
    chunk: int | None = None
    readers: tuple = ()                # own_rule() of every call that reads the pages of this one
    keep_first: int = 0

    @classmethod
    def keys_and_values(cls, num_kv_heads: int, head_dim: int, window: int | None = None,
                        chunk: int | None = None, keep_first: int = 0) -> "CacheNeed":
        """The layout of the attention kernels: K [pages, heads, page, head size], V [pages, heads, head
        size, page] (V transposed inside a page: the P.V operand of the matrix cores is then one load)."""
        return cls((PageTensor("k", (num_kv_heads, PAGE, head_dim)), PageTensor("v", (num_kv_heads, head_dim, PAGE))),
                   window, chunk, keep_first=int(keep_first or 0))

    def own_rule(self) -> tuple:
        """("window", n), ("chunk", c) or ("all", 0)."""
        if self.window:
            return ("window", int(self.window))
        if self.chunk:
            return ("chunk", int(self.chunk))
        return ("all", 0)

    def keep(self):
        """What the cache manager is told: None (every token stays), an int (one trailing window), or a tuple of
        ("window" | "chunk", n) rules of which the loosest holds at every moment, with ("first", n) among them when
        the first n positions stay for good."""
        rules = {self.own_rule(), *(r for r in self.readers if r[0] != "first")}
        if ("all", 0) in rules:
            return None
        pinned = max([self.keep_first] + [r[1] for r in self.readers if r[0] == "first"])
        rules = tuple(sorted(rules))
        if pinned > 0:
            return rules + (("first", int(pinned)),)
        return rules[0][1] if len(rules) == 1 and rules[0][0] == "window" else rules

    def group_key(self) -> tuple:
        return (self.tensors, self.keep())


@dataclass(frozen=True)
class StateNeed:
    """Fixed-size per-request state of a mixer: one tensor ``[num_slots + 1, *shape]``; the last row is
    a spare that belongs to no request (padding rows of a step with a fixed layout name it).
    ``initial``: what the state of a request holds before its first token: None for zeros, a number, or
    nested tuples of numbers of `shape` (a running maximum starts at -inf, a product at 1, ...). The step
    function writes it into a request's row when the request's tokens start at position 0."""

    shape: tuple
    dtype: str = "float32"
    initial: object = None


class Part:
    """Base of all parts: named parameters and named child parts."""

    # Whether a step that contains this part may be captured as a graph: its forward must then use device
    # operations only (no value may travel to the host: no .tolist(), .item(), nonzero(), ...). A part that
    # needs the host sets this to False; the model's steps then always run eagerly.
    capturable = True

    def __init__(self):
        self._specs: dict[str, ParamSpec] = {}
        self._children: dict[str, "Part"] = {}

    # -- declaration -------------------------------------------------------
    def add_param(self, name: str, spec: ParamSpec) -> None:
        self._specs[name] = spec
        setattr(self, name, None)

    def add_child(self, name: str, part: "Part") -> "Part":
        self._children[name] = part
        setattr(self, name, part)
        return part

    # -- traversal ---------------------------------------------------------
    def named_specs(self, prefix: str = "") -> Iterator[tuple]:
        """Yield (full name, owning part, local name, spec) over the whole tree."""
        seen: set[int] = set()
        yield from self._named_specs(prefix, seen)

    def _named_specs(self, prefix, seen):
        if id(self) in seen:        # a part shared by several parents declares its parameters once
            return
        seen.add(id(self))
        for local, spec in self._specs.items():
            yield prefix + local, self, local, spec
        for cname, child in self._children.items():
            yield from child._named_specs(prefix + cname + ".", seen)

    def parts(self) -> Iterator["Part"]:
        seen: set[int] = set()
        stack = [self]
        while stack:
            p = stack.pop()
            if id(p) in seen:
                continue
            seen.add(id(p))
            yield p
            stack.extend(p._children.values())

    # -- binding -----------------------------------------------------------
    def set_param(self, local: str, tensor: torch.Tensor) -> None:
        spec = self._specs[local]
        if tuple(tensor.shape) != tuple(spec.shape):
            raise ValueError(f"{type(self).__name__}.{local}: shape {tuple(tensor.shape)} != {tuple(spec.shape)}")
        setattr(self, local, tensor)

    def finalize(self, device: torch.device, dtype: torch.dtype, max_positions: int) -> None:
        """Called once after all parameters are bound (build tables, derived layouts)."""


class Norm(Part):
    def forward(self, x: torch.Tensor, residual: torch.Tensor | None):
        """-> (normalised x in the compute dtype, new residual in float32).

        ``residual`` None starts the residual stream from ``x``; otherwise the new
        residual is ``x + residual`` (summed in 32-bit) and that sum is normalised.
        """
        raise NotImplementedError

    # Optional: forward_terms(terms: TermSum, stream) -> (normalised x, new residual) of stream + the terms, all in one pass.
    # Optional: row_norm() -> (float32 weight, float32 bias or None, eps, whether the mean is taken off): what a kernel needs
    # to run the norm inside its own pass over the rows (`ops.stream_mix_norm`).
    # Optional: linear_behind(x, residual, weight, out_dtype, gated=False) -> (forward(x, residual)[0] . weight^T,
    # new residual), norm and product as one kernel, or None where there is no such kernel for these shapes
    # (gated: weight is a packed gate/up weight and the product is silu(gate) * up).


class PendingNorm:
    """A norm that has not run yet, in place of its output. A block hands one to a mixer or feed-forward
    that declares `takes_pending_norm = True`; such a part passes it to its first `Linear`, which may run
    norm and product as one kernel (`Norm.linear_behind`), or asks `value()` for the normed rows as a
    tensor. Whichever happens first also yields the new residual, which the block reads afterwards. x may
    be a `TermSum`."""

    def __init__(self, norm: "Norm", x, residual: torch.Tensor | None):
        self.norm, self.x, self.residual = norm, x, residual
        self._y = None
        self._new_residual = None

    def rows(self) -> int:
        x = self.x.terms[0] if isinstance(self.x, TermSum) else self.x
        return x.shape[-2]

    def value(self) -> torch.Tensor:
        if self._y is None:
            x = self.x
            if isinstance(x, TermSum):
                self._y, self._new_residual = x.normed(self.norm, self.residual)
                return self._y
            if x.dim() == 3 and not getattr(self.norm, "accepts_partials", False):
                x = x.sum(0)
            self._y, self._new_residual = self.norm.forward(x, self.residual)
        return self._y

    def into_linear(self, weight: torch.Tensor, out_dtype=None, gated: bool = False):
        """The product of the normed rows with `weight` ([out, in]) if the norm can run inside it, else None.
        gated: `weight` is a packed gate/up weight and the product is silu(gate) * up."""
        behind = getattr(self.norm, "linear_behind", None)
        if self._y is not None or behind is None or isinstance(self.x, TermSum):
            return None
        got = behind(self.x, self.residual, weight, out_dtype, gated) if gated else behind(self.x, self.residual, weight, out_dtype)
        if got is None:
            return None
        y, self._new_residual = got
        return y

    def new_residual(self) -> torch.Tensor:
        if self._new_residual is None:
            self.value()
        return self._new_residual


class Settled:
    """What a layer returns in place of its output when it has already added that output to the residual
    stream (a block whose norms sit on the sublayers' outputs does): `rounded` is the stream in the compute
    dtype, for the next layer's sublayers to read. Whoever comes next must not add anything to the residual."""

    def __init__(self, rounded: torch.Tensor):
        self.rounded = rounded


class ScaledSum:
    """What a layer returns in place of its output when several sublayer outputs still have to be added to the
    residual stream, each under a scale of its own: stream += mult * sum_i scale_i * term_i. `terms`: pairs of (rows
    [T, n] in the compute dtype or float32 partial sums [P, T, n], float32 scale [n] or None). Whoever runs next forms
    the sum, a block of the same kind together with its own norms in one pass (`ops.scaled_sum_norm`); anyone else
    calls `settle`."""

    def __init__(self, terms: list, mult: float):
        self.terms, self.mult = list(terms), float(mult)

    def settle(self, stream: torch.Tensor) -> torch.Tensor:
        """The new stream, float32 [T, n]."""
        from ..kernels import ops
        return ops.scaled_sum_norm(stream, self.terms, self.mult, None, None, 0.0, torch.float32)[0]


class Biased:
    """A sublayer's output whose bias is still to be added: (rows or float32 partial sums, float32 bias [n]). A mixer or
    feed-forward returns one only to a caller that asked for it (`defer_bias`) and adds it where it adds the output."""

    def __init__(self, rows: torch.Tensor, bias: torch.Tensor):
        self.rows, self.bias = rows, bias


class TermSum:
    """What a layer returns in place of its output when several terms still have to be added to the residual stream, each as it
    is: rows [T, n], float32 partial sums [P, T, n], or a `Biased` of either. Whoever runs next forms the sum: a norm with
    `forward_terms` in its own pass, the model's final norm at the wanted rows only (`normed_rows`), anyone else through
    `settle`."""

    MOST = 4                   # terms that one pass adds (`ops.stream_mix_norm`)

    def __init__(self, terms: list):
        self.terms, self.bias = [], None
        for t in terms:
            if isinstance(t, Biased):
                self.bias = t.bias if self.bias is None else self.bias + t.bias
                t = t.rows
            self.terms.append(t)

    def with_term(self, rows: torch.Tensor) -> "TermSum":
        out = TermSum(self.terms + [rows])
        out.bias = self.bias
        return out

    def _mix(self, stream, norm, out_dtype, rows=None, keep=True):
        from ..kernels import ops
        if stream is None:                    # the terms are the whole stream
            stream = torch.zeros(self.terms[0].shape[-2:], dtype=torch.float32, device=self.terms[0].device)
        terms = list(self.terms)
        while len(terms) > self.MOST:
            stream = ops.stream_mix_norm(stream, 1, terms[:self.MOST], None, None, None, None, torch.float32, keep=False)[1]
            terms = terms[self.MOST:]
        return ops.stream_mix_norm(stream.view(stream.shape[0], 1, -1), 1, terms, None, None, None, norm, out_dtype, rows=rows, keep=keep,
                                   bias=self.bias)

    def settle(self, stream: torch.Tensor | None) -> torch.Tensor:
        """The new stream, float32 [T, n]."""
        return self._mix(stream, None, torch.float32, keep=False)[1]

    def normed(self, norm: "Norm", stream: torch.Tensor | None):
        """(the norm of the new stream, the new stream)."""
        forward_terms = getattr(norm, "forward_terms", None)
        return forward_terms(self, stream) if forward_terms is not None else norm.forward(self.settle(stream), None)

    def normed_rows(self, stream: torch.Tensor, norm: "Norm", rows: torch.Tensor):
        """The norm of the new stream at `rows`, or None for a norm that no kernel can run inside."""
        if not hasattr(norm, "row_norm"):
            return None
        return self._mix(stream, norm.row_norm(), norm.out_dtype, rows=rows, keep=False)[1]


class StreamSum:
    """What a layer with several residual streams (hyper-connections) returns in place of its output, beside the streams
    as its last sublayer found them: every stream takes a share of every stream and of that sublayer's output,
        x'_t = sum_s mix[s, t] x_s + out[t] * sum(terms).
    Whoever runs next forms it, a block of the same kind together with what its own sublayer reads and the norm in front of
    that in one pass (`ops.stream_mix_norm`). The model's residual is the sum of the streams: `settle` (float32 [T, n]);
    `normed_rows` is a norm of that sum for chosen rows only (the model's final norm)."""

    def __init__(self, terms: list, mix: torch.Tensor, out: torch.Tensor):
        self.terms, self.mix, self.out = list(terms), mix, out

    def settle(self, streams: torch.Tensor) -> torch.Tensor:
        from ..kernels import ops
        return ops.stream_mix_norm(streams, self.out.numel(), self.terms, self.mix, self.out, None, None, torch.float32, keep=False)[1]

    def normed_rows(self, streams: torch.Tensor, norm: "Norm", rows: torch.Tensor):
        """The norm of the sum of the streams at `rows`, or None for a norm that no kernel can run inside."""
        if not hasattr(norm, "row_norm"):
            return None
        from ..kernels import ops
        return ops.stream_mix_norm(streams, self.out.numel(), self.terms, self.mix, self.out, None, norm.row_norm(), norm.out_dtype,
                                   rows=rows, keep=False)[1]


# Steps of up to this many tokens are chains of short launches: parts that have independent work then put it on further
# streams (0: never). The streams have the default priority; a captured step holds such work as branches of its graph.
SIDE_BRANCH_MAX_TOKENS = 64
_side_streams: dict = {}


class side_branch:
    """`with side_branch(device, slot):` what is launched inside runs on a further stream (one per device and slot) that
    starts behind everything launched so far on the current stream; `join()` afterwards makes the current stream wait
    for it. Library products inside use a workspace of their own. What the branch allocates may be read on the current
    stream only behind `join()`; the caller sees to it that it is not written again before its reader has been
    launched (a later branch of the same slot starts behind whatever was launched before it)."""

    def __init__(self, device: torch.device, slot: int = 1):
        from ..kernels import ops
        key = (device.type, device.index, slot)
        if key not in _side_streams:
            _side_streams[key] = torch.cuda.Stream(device=device)
        self.stream, self.main = _side_streams[key], torch.cuda.current_stream(device)
        self._inner = (torch.cuda.stream(self.stream), ops.second_workspace(slot))

    def __enter__(self):
        self.stream.wait_stream(self.main)
        for c in self._inner:
            c.__enter__()
        return self

    def __exit__(self, *exc):
        for c in reversed(self._inner):
            c.__exit__(*exc)

    def join(self) -> None:
        self.main.wait_stream(self.stream)


def few_tokens(x: torch.Tensor) -> bool:
    """Whether a step with rows x is one whose independent work goes to side branches."""
    return x.is_cuda and 0 < x.shape[0] <= SIDE_BRANCH_MAX_TOKENS


class PositionEncoding(Part):
    """Something applied to queries and keys as a function of token positions."""

    def apply(self, q: torch.Tensor, k: torch.Tensor, positions: torch.Tensor) -> None:
        """Rotate/shift ``q`` [T, Hq, D] and ``k`` [T, Hkv, D] in place."""
        raise NotImplementedError

    def rotary_table(self) -> torch.Tensor | None:
        """[P, D/2, 2] float32 (cos, sin) if this is a half-split rotary encoding that the
        fused query/key kernel can apply; None means ``apply`` must be called."""
        return None


class Mixer(Part):
    """Token mixing: the only part that looks at other positions of a request."""

    def cache_need(self) -> CacheNeed | None:
        return None

    def state_need(self) -> StateNeed | None:
        return None

    def forward(self, x: torch.Tensor, step, cache, state) -> torch.Tensor:
        """x: [T, hidden] -> [T, hidden].

        ``step``: the `StepContext` of this step. ``cache``: a `CacheView` (pages of this
        call's layer, or of the layer it reads) or None. ``state``: this call's state
        tensor ``[num_slots + 1, *shape]`` or None; rows are ``step.state_slots``.
        """
        raise NotImplementedError


class FeedForward(Part):
    def forward(self, x: torch.Tensor) -> torch.Tensor:
        """[T, hidden] -> [T, hidden], or float32 partial sums [P, T, hidden], or a tuple of such tensors whose sum is
        the output (a routed part beside one that every token passes); with `defer_bias` set by the caller, a `Biased` of
        either of the first two."""
        raise NotImplementedError


class Head(Part):
    """Hidden rows to float32 logits. `project` is what a head implements; `forward` is what the model calls."""

    def project(self, x: torch.Tensor) -> torch.Tensor:
        """x [rows, hidden] -> float32 [rows, vocabulary]."""
        raise NotImplementedError

    def forward(self, x: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
        """`out`: a float32 [rows, vocabulary] tensor the logits must end up in (a step with a fixed layout
        keeps one). A head whose product can write there overrides this; by default the result is copied."""
        y = self.project(x)
        if out is None:
            return y
        out.copy_(y)
        return out


@dataclass
class LayerCall:
    """One entry of a model's run order.

    ``layer``: index into the model's layers (a layer may be named by several
    entries: its weights are then shared, each entry has a cache of its own).
    ``cache_of``: index of an *earlier entry* whose cache this entry reads
    instead of owning one; it then writes nothing.
    ``add_start``: right before this entry the embedding's output (the stream as it was before the
    first entry) is added to the stream once more.
    """

    layer: int
    cache_of: int | None = None
    add_start: bool = False


@dataclass
class CacheView:
    """The pages one layer call reads and writes: per tensor of its CacheNeed, [num_pages + 1, *shape
    of a page]. The last page is a spare that belongs to no request: padding rows of a step with a fixed
    layout write there."""

    group: int                 # index of the page group (selects block table and slot mapping)
    tensors: dict              # PageTensor name -> tensor
    page_size: int
    write: bool = True

    @property
    def k(self) -> torch.Tensor:           # [pages, Hkv, page, D] of a keys-and-values layout
        return self.tensors["k"]

    @property
    def v(self) -> torch.Tensor:           # [pages, Hkv, D, page]
        return self.tensors["v"]


# ---------------------------------------------------------------- registries

_REGISTRIES: dict[str, dict[str, type]] = {
    "mixer": {}, "feed_forward": {}, "norm": {}, "position_encoding": {}, "block": {},
}


def register_part(kind: str, name: str):
    """Class decorator: make a part constructible by ``make_part(kind, name, ...)``."""
    if kind not in _REGISTRIES:
        raise KeyError(f"unknown part kind {kind!r}; kinds: {sorted(_REGISTRIES)}")

    def deco(cls):
        _REGISTRIES[kind][name] = cls
        return cls

    return deco


def make_part(kind: str, name: str, **kwargs) -> Part:
    try:
        cls = _REGISTRIES[kind][name]
    except KeyError:
        raise KeyError(f"no {kind} named {name!r}; registered: {sorted(_REGISTRIES.get(kind, {}))}") from None
    return cls(**kwargs)


def registered(kind: str) -> list:
    return sorted(_REGISTRIES[kind])
