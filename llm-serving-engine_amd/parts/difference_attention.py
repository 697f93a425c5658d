"""Differential attention: two softmax maps a head over the same values, the second taken off the first, with short
convolutions over queries, keys and values, and a temperature of the queries that grows with the position."""

from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from .attention import Mixer
from .base import MIXERS, CacheNeed, FixedState, PagedKeyValue, TensorSpec
from .position import HeadLayout


@dataclass(frozen=True)
class DifferenceAttentionSpec:
    """`num_heads` query heads and `num_kv_heads` key/value heads (query head h reads key/value head h // (heads /
    kv_heads)); a query head and a key head are two maps of `dim` side by side, a value head is `vdim` wide.

    `difference`: the constant c in lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + c and in the (1 - c) on the normed result.
    `taps` (None: none): a causal convolution of so many taps on every channel of the three projections.
    `temperature` (None: none): (coef, every), a query at p is multiplied by 1 + coef ln(floor((p + 1) / every) + 1).
    `norm`: RMS norm of every query and key map with one weight of `dim` for all heads and maps (False: none).
    `own_keys` False: the layer has no key and value projections, it attends over the keys and values of the earlier layer
    run that its `LayerRun.reads` names, with queries (and a convolution of them) of its own."""

    hidden_size: int
    num_heads: int
    num_kv_heads: int
    dim: int
    vdim: int
    scale: float
    eps: float
    difference: float
    taps: int | None = None
    temperature: tuple[float, int] | None = None
    norm: bool = True
    own_keys: bool = True
    kind: str = "difference_attention"

    @property
    def stored_heads(self) -> int:
        """Key/value heads that the layer projects and stores itself."""
        return self.num_kv_heads if self.own_keys else 0

    @property
    def map_width(self) -> int:
        """What one map of a key takes in the cache: a key's two maps lie side by side in one row that is as wide as the
        values', so a map has half of it, a multiple of 16, zeros beyond `dim`."""
        return -(-max(2 * self.dim, self.vdim) // 32) * 16

    @property
    def head_width(self) -> int:
        return 2 * self.map_width

    @property
    def channels(self) -> int:
        """What the convolutions run over: q, k and v side by side."""
        return 2 * self.num_heads * self.dim + self.stored_heads * (2 * self.dim + self.vdim)


@MIXERS.register("difference_attention")
class DifferenceAttention(Mixer):
    """q = norm(conv(W_q x)), k = norm(conv(W_k x)), v = conv(W_v x), q times the temperature; per head, a1 and a2 the
    softmax over (q_m . k_m) * scale of the maps m = 1, 2 applied to v; a1 - lambda a2, divided by its root mean square,
    times (1 - c); W_o.

    A key row of the cache holds both maps of a head, [map 1 | map 2], beside a value row of the same width: one entry a
    key/value head as in plain attention, nothing is stored twice, and a query row [q map 1 | q map 2] meets it whole.
    The convolutions' last taps - 1 inputs are kept in a state slot a request, zeros when it begins.  Convolutions, norms,
    temperature, scores and the difference are float32."""

    @classmethod
    def tensors(cls, spec: DifferenceAttentionSpec) -> dict[str, TensorSpec]:
        sizes = {"q": 2 * spec.num_heads * spec.dim}
        if spec.own_keys:
            sizes.update(k=2 * spec.num_kv_heads * spec.dim, v=spec.num_kv_heads * spec.vdim)
        found = {name: TensorSpec((size, spec.hidden_size)) for name, size in sizes.items()}
        if spec.norm:
            found["q.norm"] = TensorSpec((spec.dim,), role="norm")
            if spec.own_keys:
                found["k.norm"] = TensorSpec((spec.dim,), role="norm")
        if spec.taps is not None:
            found.update({name + ".conv": TensorSpec((size, spec.taps)) for name, size in sizes.items()})
        found.update({name: TensorSpec((spec.dim,), role="bias") for name in ("lq1", "lk1", "lq2", "lk2")})
        found["o"] = TensorSpec((spec.hidden_size, spec.num_heads * spec.vdim))
        return found

    @classmethod
    def cache_need(cls, spec: DifferenceAttentionSpec) -> dict[str, CacheNeed]:
        need: dict[str, CacheNeed] = {"keys": PagedKeyValue(spec.num_kv_heads, spec.head_width)}
        if spec.taps is not None and spec.taps > 1:
            need["window"] = FixedState((spec.taps - 1, spec.channels))
        return need

    def __init__(self, spec: DifferenceAttentionSpec, tensors, kernels) -> None:
        super().__init__(spec, tensors, kernels)
        if spec.num_heads % spec.num_kv_heads:
            raise ValueError("differential attention: the query heads are a multiple of the key/value heads")
        if spec.taps is not None and spec.taps < 1:
            raise ValueError("differential attention: a convolution has one tap or more")
        names = ("q", "k", "v") if spec.own_keys else ("q",)
        rows = spec.num_heads + 2 * spec.stored_heads
        self.layout = HeadLayout(spec.num_heads, spec.num_kv_heads, spec.head_width, rows * spec.head_width)
        self.inputs = kernels.prepare_linear([tensors[name] for name in names], None)  # [q | k | v]
        self.out = kernels.prepare_linear([tensors["o"]], None)
        self.taps = None
        if spec.taps is not None:
            self.taps = kernels.to_device(torch.cat([tensors[name + ".conv"] for name in names], dim=0).float().contiguous())
        self.q_norm = tensors["q.norm"] if spec.norm else None
        self.k_norm = (tensors["k.norm"] if spec.own_keys else self.q_norm) if spec.norm else None
        one, two = (float((tensors[a].double() * tensors[b].double()).sum()) for a, b in (("lq1", "lk1"), ("lq2", "lk2")))
        self.factor = math.exp(one) - math.exp(two) + spec.difference

    def forward(self, x: torch.Tensor, batch, cell) -> torch.Tensor:
        kernels, spec = self.kernels, self.spec
        projected = kernels.linear(x, self.inputs)
        q_size, k_size = 2 * spec.num_heads * spec.dim, 2 * spec.stored_heads * spec.dim
        rows = kernels.convolved_heads(
            projected, 0, q_size, q_size + k_size, spec.num_heads, spec.stored_heads, spec.dim, spec.vdim, spec.head_width, batch,
            cell["keys"] if spec.own_keys else None, maps=2, taps=self.taps, window=cell["window"].state if "window" in cell else None,
            norm=spec.norm, q_weight=self.q_norm, k_weight=self.k_norm, eps=spec.eps, temperature=spec.temperature,
        )
        mixed = kernels.difference_attention(
            rows, self.layout, batch, cell["keys"], spec.scale, spec.vdim, self.factor, spec.eps, 1.0 - spec.difference
        )  # [T, heads * vdim]
        return kernels.linear(mixed, self.out, out_dtype=torch.float32, partial=True)
