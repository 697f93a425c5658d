"""What every part of a layer has in common: a spec (its sizes and constants),
the tensors it owns by name, what it needs of the cache, and a registry that
maps a spec's `kind` to the class that runs it.

A part never sees a model configuration.  It is built from its own spec, the
tensors under its own prefix and the kernel library, so a model may use
different mixers and feed-forwards in different layers, and a new part is added
by registering a class: nothing else changes.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, ClassVar

import torch


@dataclass(frozen=True)
class TensorSpec:
    """One tensor a part owns.

    role decides how the random-weights mode draws it: "matrix" and "embedding"
    N(0, std), "bias" N(0, bias_std), "norm" N(1, norm_std) (ones when
    norm_std is 0), "table" integers.  `integer` tensors are kept as int32; the
    others in the run's dtype unless the file stores them in 32-bit.
    """

    shape: tuple[int, ...]
    role: str = "matrix"
    integer: bool = False


KEY_PIECE = 8  # elements of a key that stay together in a page (csrc/common.h has the same number)


def key_piece_width(head_dim: int) -> int:
    """A key is kept in pieces of KEY_PIECE elements; a head size that is no multiple of it in one piece."""
    return KEY_PIECE if head_dim % KEY_PIECE == 0 else head_dim


VALUE_PIECE = 8  # keys whose values of one dimension stay together in a page (csrc/common.h has the same number)


def value_piece_width(page_size: int) -> int:
    """A page's values are kept in pieces of VALUE_PIECE keys; a page size that is no multiple of it in one piece."""
    return VALUE_PIECE if page_size % VALUE_PIECE == 0 else page_size


class CacheNeed:
    """What a part keeps in the cache from one step to the next.  The cache manager knows two ways of
    giving room, and a need is of one of them: `PagedNeed` (an entry per token, in pages that a request
    holds through a block table) or `SlotNeed` (one entry of fixed size per request).  What an entry *is*
    is the need's own business: a new kind of need is a subclass that says what a page of it holds, and
    nothing in the cache manager, the step function or the scheduler changes.  Needs are compared and
    hashed (frozen dataclasses): runs with equal paged needs share a pool and a block table per request."""


class PagedNeed(CacheNeed):
    """An entry per token.  A subclass has a field `window` (keys at most that are ever read again, None:
    all), may have a field `keep_first` (so many entries at a request's start are read for ever, whatever the
    window) and one `chunk` (instead of a window: a query reads the entries of its own chunk of so many positions,
    counted from the request's start), and says what one page holds."""

    window: int | None = None
    keep_first: int = 0
    chunk: int | None = None

    def first_read(self, position: int) -> int:
        """No query at `position` or later reads an entry before the one returned (the first `keep_first` aside)."""
        if self.window is not None:
            return max(0, position - self.window + 1)
        if self.chunk is not None:
            return position - position % self.chunk
        return 0

    def shared_with(self, other: "CacheNeed") -> "CacheNeed | None":
        """The need of one cell that runs with this need and with `other` both read: None where the two differ in what an
        entry is, else one that keeps entries as long as either asks."""
        return self if other == self else None

    def page_fields(self, page_size: int) -> dict[str, tuple[int, ...]]:
        """name -> shape of ONE page of that field.  The cache keeps each field as a tensor
        [pages, *shape] in the run dtype, and a `CacheCell` shows them by these names."""
        raise NotImplementedError

    def token_rows(self, page: dict[str, torch.Tensor], page_size: int) -> dict[str, torch.Tensor]:
        """One page's fields rearranged so that the token's offset in the page leads: name ->
        [page_size, ...].  The host-side read path (tests, debugging) walks pages through it; kernels
        read the pages as they lie."""
        raise NotImplementedError


class SlotNeed(CacheNeed):
    """One entry of fixed size per request.  A subclass has a field `shape`: the cache keeps a float32
    tensor [request slots, *shape], zeroed when a request takes its slot."""

    shape: tuple[int, ...] = ()


def needs_by_name(need: "CacheNeed | dict[str, CacheNeed] | None") -> "dict[str | None, CacheNeed]":
    """A run's needs by name: none, one (under None), or the several its block named."""
    if need is None:
        return {}
    if isinstance(need, dict):
        if any(not isinstance(name, str) for name in need):
            raise TypeError("several cache needs are named by strings")
        return {name: value for name, value in need.items() if value is not None}
    return {None: need}


@dataclass(frozen=True)
class PagedKeyValue(PagedNeed):
    """Cache need of a mixer that keeps a key and a value per token in pages.  Keys lie in pieces of
    eight elements, the same piece of all the keys of a page side by side ([kv_heads, head_dim / w,
    page_size, w], w = `key_piece_width(head_dim)`): the matrix cores take keys as rows, a lane holding
    one piece of one key and its neighbours that piece of the next keys, and neighbouring lanes should
    read neighbouring bytes.  Values are stored transposed, in pieces of eight keys ([kv_heads, page_size / v,
    head_dim, v], v = `value_piece_width(page_size)`): attention sums over keys, the matrix cores want the
    summed index contiguous, and a lane's neighbours hold the same keys of the next dimensions."""

    num_kv_heads: int
    head_dim: int
    window: int | None = None
    keep_first: int = 0
    chunk: int | None = None

    def __post_init__(self) -> None:
        if self.window is not None and self.chunk is not None:
            raise ValueError("keys and values are read through a window or in chunks, not both")

    def shared_with(self, other: CacheNeed) -> "PagedKeyValue | None":
        if not isinstance(other, PagedKeyValue) or (other.num_kv_heads, other.head_dim) != (self.num_kv_heads, self.head_dim):
            return None
        if other == self:
            return self
        window = chunk = None
        if self.window is not None and other.window is not None:
            window = max(self.window, other.window)
        elif self.keep_first or other.keep_first:
            return None
        elif self.chunk is not None and other.chunk is not None:
            chunk = math.lcm(self.chunk, other.chunk)  # a chunk of either size lies in one of these
        if self.keep_first != other.keep_first:  # (readers say what a cell keeps: those of one cell agree on it)
            return None
        return PagedKeyValue(self.num_kv_heads, self.head_dim, window, self.keep_first, chunk)

    def page_fields(self, page_size: int) -> dict[str, tuple[int, ...]]:
        width = key_piece_width(self.head_dim)
        return {
            "keys": (self.num_kv_heads, self.head_dim // width, page_size, width),
            "values": (self.num_kv_heads, page_size // value_piece_width(page_size), self.head_dim, value_piece_width(page_size)),
        }

    def token_rows(self, page: dict[str, torch.Tensor], page_size: int) -> dict[str, torch.Tensor]:
        keys = page["keys"].permute(2, 0, 1, 3).reshape(page_size, self.num_kv_heads, self.head_dim)
        values = page["values"].permute(1, 3, 0, 2).reshape(page_size, self.num_kv_heads, self.head_dim)
        return {"keys": keys, "values": values}


@dataclass(frozen=True)
class FixedState(SlotNeed):
    """Cache need of a mixer that keeps a state of fixed size per request: one
    slot of `shape` float32 values, zeroed when the request is created."""

    shape: tuple[int, ...]


class Part:
    """Base of norms, position encodings, mixers, feed-forwards and blocks."""

    kind: ClassVar[str] = ""
    # Whether a step through the part is the same sequence of kernel launches whatever the data:
    # then a step of single tokens may be captured into a graph once and replayed.  A part that
    # looks at values on the host (routing that gathers rows, a loop over a request's tokens) says False.
    replayable: ClassVar[bool] = True

    @classmethod
    def tensors(cls, spec: Any) -> dict[str, TensorSpec]:
        """Names (relative to the part's prefix) and shapes of its tensors."""
        return {}

    @classmethod
    def cache_need(cls, spec: Any) -> "CacheNeed | dict[str, CacheNeed] | None":
        """What the part keeps in the cache: nothing, one need, or several by name (a block with two
        mixers side by side, one with pages and one with a state): its cell is then a dict of cells
        by the same names."""
        return None

    def __init__(self, spec: Any, tensors: dict[str, torch.Tensor], kernels: Any) -> None:
        self.spec = spec
        self.kernels = kernels


class Registry:
    """kind -> part class, for one family of parts."""

    def __init__(self, family: str) -> None:
        self.family = family
        self._classes: dict[str, type[Part]] = {}

    def register(self, kind: str):
        def decorate(cls: type[Part]) -> type[Part]:
            if kind in self._classes and self._classes[kind] is not cls:
                raise ValueError(f"{self.family} kind {kind!r} is already registered")
            cls.kind = kind
            self._classes[kind] = cls
            return cls

        return decorate

    def unregister(self, kind: str) -> None:
        self._classes.pop(kind, None)

    def get(self, spec: Any) -> type[Part]:
        kind = getattr(spec, "kind", None)
        if kind not in self._classes:
            known = ", ".join(sorted(self._classes)) or "none"
            raise KeyError(f"no {self.family} of kind {kind!r} is registered (known: {known})")
        return self._classes[kind]

    def tensors(self, spec: Any) -> dict[str, TensorSpec]:
        return self.get(spec).tensors(spec)

    def cache_need(self, spec: Any) -> "CacheNeed | dict[str, CacheNeed] | None":
        return self.get(spec).cache_need(spec)

    def build(self, spec: Any, tensors: dict[str, torch.Tensor], kernels: Any) -> Part:
        return self.get(spec)(spec, tensors, kernels)

    def kinds(self) -> list[str]:
        return sorted(self._classes)


NORMS = Registry("norm")
POSITIONS = Registry("position encoding")
MIXERS = Registry("mixer")
FEED_FORWARDS = Registry("feed-forward")
BLOCKS = Registry("block")
# What acts on the residual stream between the embedding and the first layer (`forward(hidden, batch)`, in
# place: a table of absolute positions, a scale), and on the logits after the head (`forward(logits, batch)
# -> logits`: a bias, a soft cap).  Qwen2 has neither; a model lists them in `ModelSpec.input_parts` and
# `ModelSpec.output_parts`.
STREAM_PARTS = Registry("part on the embedded stream")
LOGIT_PARTS = Registry("part on the logits")
# What stands at the start of a pass through a run of layers that a model walks several times: `forward(hidden,
# delta, embedded, batch, number of the pass) -> hidden`, where `embedded` is the stream as it left the
# embedding (and the input parts).  A model names one in `ModelSpec.pass_entry`, and the runs that begin a
# pass in `LayerRun.enters`.
PASS_PARTS = Registry("part at the start of a pass")


def under(tensors: dict[str, Any], prefix: str) -> dict[str, Any]:
    """The entries of `tensors` below `prefix`, with the prefix removed."""
    return {name[len(prefix):]: value for name, value in tensors.items() if name.startswith(prefix)}


def prefixed(tensors: dict[str, Any], prefix: str) -> dict[str, Any]:
    return {prefix + name: value for name, value in tensors.items()}


def side_by_side(products: list[tuple[torch.Tensor, torch.Tensor | None]]) -> tuple[list[torch.Tensor], list[torch.Tensor] | None]:
    """(weight [N, K], bias or None) of several products over the same rows, as one product's lists of weights and of
    biases: zeros where only some have a bias, None where none has."""
    known = [bias for _, bias in products if bias is not None]
    if not known:
        return [weight for weight, _ in products], None
    biases = [torch.zeros((weight.shape[0],), dtype=known[0].dtype, device=known[0].device) if bias is None else bias for weight, bias in products]
    return [weight for weight, _ in products], biases
