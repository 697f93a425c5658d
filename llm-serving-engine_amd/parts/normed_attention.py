"""Attention over a sliding window or in chunks whose queries and keys may be normed, with the options some designs put
around it: heads rotated in part, capped scores, a sink in the softmax's denominator, values blended with an earlier
layer's, values that are the keys, keys and values read from an earlier layer's cache, a learned bias by distance, and a
gate on the result."""

from __future__ import annotations

import dataclasses
from dataclasses import dataclass

import torch

from .attention import Mixer
from .base import MIXERS, PagedKeyValue, TensorSpec, side_by_side
from .position import DistanceBuckets, HeadLayout, LinearScaling, WavelengthScaling, YarnScaling, rotary_frequencies


@dataclass(frozen=True)
class NormedAttentionSpec:
    """`num_heads` query heads and `num_kv_heads` key/value heads (query head h reads key/value head h // (heads /
    kv_heads)); queries and keys of `dim`, values of `vdim`.

    `norm`: "head" (RMS norm of every query and key head with one weight of `dim` for all heads), "unit" (every query and
    key head divided by its root mean square, no weight), "row" (RMS norm of
    the whole query projection and of the whole key projection, with weights as long as they), or None.
    `rot_dims`: the first so many dimensions of every query and key head turn by the position, in adjacent pairs
    (2i, 2i + 1) or, with `pairing` "half", in pairs (i, i + rot_dims / 2), with the frequencies theta^(-2i / rot_dims)
    stretched by `scaling`; 0: positions do not enter.
    `soft_cap`: scores become cap * tanh(score / cap).  `sink`: a learned number a head whose exponential is added
    once to the softmax's denominator.  `gate`: head h's result times sigmoid of row h of a product of the mixer's input.
    `values`: None, "give" (the step's values are shown to later layers under `values_name`) or "take" (v <- (1 - a) v
    + a v_given with the learned number a; the blended v is what is cached).
    `keep_first`: under a window, the first so many tokens of a sequence stay visible to every later query, at their
    own positions (a query at p sees the keys at j <= p with p - j < window or j < keep_first).
    `chunk`: instead of a window, a query at p sees the keys at j <= p with j // chunk == p // chunk.
    `own_keys` False: the layer has no key and value projections, it attends over the cell of the earlier layer run that its
    `LayerRun.reads` names, with queries of its own.
    `keys_as_values`: there is no value projection, the values are the keys as they were projected (before norm and rotation).
    `distance`: a learned bias by distance on every score, behind its scale: row distance.of(p - j) of a table [buckets,
    heads] (`rel`).  `wide_gate`: the heads' results side by side times the sigmoid of a product of the mixer's input, element
    by element.
    `bias` is of the q, k and v projections, `out_bias` of the last.  `joined`: the first and the last product are the
    block's (`Mixer`)."""

    hidden_size: int
    num_heads: int
    num_kv_heads: int
    dim: int
    vdim: int
    scale: float
    eps: float
    window: int | None = None
    bias: bool = False
    norm: str | None = "head"
    rot_dims: int = 0
    theta: float = 10000.0
    scaling: YarnScaling | WavelengthScaling | LinearScaling | None = None
    pairing: str = "adjacent"
    soft_cap: float | None = None
    sink: bool = False
    gate: bool = False
    values: str | None = None
    values_name: str = "values"
    keep_first: int = 0
    chunk: int | None = None
    own_keys: bool = True
    out_bias: bool = False
    keys_as_values: bool = False
    distance: DistanceBuckets | None = None
    wide_gate: bool = False
    joined: bool = False
    kind: str = "normed_attention"

    @property
    def stored_heads(self) -> int:
        """Key/value heads that the layer projects and stores itself."""
        return self.num_kv_heads if self.own_keys else 0

    @property
    def head_width(self) -> int:
        """What a head takes in the cache and in the attention kernels: keys and values side by side have one width
        there, the larger of the two rounded up to a multiple of 16, the rest of a narrower head zeros."""
        return -(-max(self.dim, self.vdim) // 16) * 16


@MIXERS.register("normed_attention")
class NormedAttention(Mixer):
    """q = W_q x (+ b), k, v likewise; norm; rotation; v blended; per head softmax over the keys of the last
    `window` positions of (q . k) * scale, capped, with the sink; the gate; W_o.

    The heads go to the engine's paged attention as rows of `head_width`: a key's or value's columns beyond its own
    size are zeros, which change neither a score nor a result's own columns, and the output projection's weight has
    zero columns where the results do.  Norms, angles, cosines and sines, the blend and the gate are float32.  Where the
    projections are already such rows (sizes of `head_width`, nothing to do to a head) the attention reads them as they lie."""

    joins = True

    @classmethod
    def tensors(cls, spec: NormedAttentionSpec) -> dict[str, TensorSpec]:
        q_size, k_size, v_size = spec.num_heads * spec.dim, spec.num_kv_heads * spec.dim, spec.num_kv_heads * spec.vdim
        found = {"q": TensorSpec((q_size, spec.hidden_size))}
        if spec.own_keys:
            found["k"] = TensorSpec((k_size, spec.hidden_size))
            if not spec.keys_as_values:
                found["v"] = TensorSpec((v_size, spec.hidden_size))
        found["o"] = TensorSpec((spec.hidden_size, spec.num_heads * spec.vdim))
        if spec.bias:
            found["q.b"] = TensorSpec((q_size,), role="bias")
            if spec.own_keys:
                found["k.b"] = TensorSpec((k_size,), role="bias")
                if not spec.keys_as_values:
                    found["v.b"] = TensorSpec((v_size,), role="bias")
        if spec.out_bias:
            found["o.b"] = TensorSpec((spec.hidden_size,), role="bias")
        if spec.norm == "head":
            found.update({"q.norm": TensorSpec((spec.dim,), role="norm"), "k.norm": TensorSpec((spec.dim,), role="norm")})
        elif spec.norm == "row":
            found.update({"q.norm": TensorSpec((q_size,), role="norm"), "k.norm": TensorSpec((k_size,), role="norm")})
        if spec.values is not None:
            found["vmix"] = TensorSpec((), role="bias")  # (a layer that gives its values has the number too, and does not use it)
        if spec.sink:
            found["sink"] = TensorSpec((spec.num_heads,), role="bias")
        if spec.gate:
            found["g"] = TensorSpec((spec.num_heads, spec.hidden_size))
        if spec.wide_gate:
            found["g"] = TensorSpec((spec.num_heads * spec.vdim, spec.hidden_size))
        if spec.distance is not None:
            found["rel"] = TensorSpec((spec.distance.buckets, spec.num_heads), role="bias")
        return found

    @classmethod
    def cache_need(cls, spec: NormedAttentionSpec) -> PagedKeyValue:
        return PagedKeyValue(
            spec.num_kv_heads, spec.head_width, spec.window, spec.keep_first if spec.window is not None else 0, spec.chunk,
        )

    def __init__(self, spec: NormedAttentionSpec, tensors, kernels) -> None:
        super().__init__(spec, tensors, kernels)
        if spec.num_heads % spec.num_kv_heads:
            raise ValueError("normed attention: the query heads are a multiple of the key/value heads")
        if spec.norm not in (None, "head", "unit", "row") or spec.values not in (None, "give", "take"):
            raise ValueError("normed attention: norm is 'head', 'unit', 'row' or None; values 'give', 'take' or None")
        if spec.pairing not in ("adjacent", "half"):
            raise ValueError("normed attention: pairing is 'adjacent' or 'half'")
        if spec.rot_dims % 2 or spec.rot_dims > spec.dim:
            raise ValueError("normed attention: the rotated dimensions are an even number within dim")
        if spec.keep_first < 0:
            raise ValueError("normed attention: keep_first counts tokens")
        if spec.window is not None and spec.chunk is not None:
            raise ValueError("normed attention: a mask is a window or chunks")
        if not spec.own_keys and (spec.norm is not None or spec.values is not None or spec.gate or spec.wide_gate):
            raise ValueError("normed attention: norms, blended values and gates are of layers with keys of their own")
        if (spec.keys_as_values or spec.norm == "unit") and (spec.rot_dims or spec.values is not None or spec.norm == "row"):
            raise ValueError("normed attention: unit norms and values that are the keys go with neither rotation nor blended values")
        if spec.keys_as_values and (spec.dim != spec.vdim or not spec.own_keys):
            raise ValueError("normed attention: values that are the layer's own keys are as wide as they")
        if spec.gate and spec.wide_gate:
            raise ValueError("normed attention: one gate a head or one an element")
        if (spec.wide_gate or spec.distance is not None) and (spec.soft_cap is not None or spec.sink or self.keep_first_of(spec) or spec.chunk is not None):
            raise ValueError("normed attention: a bias by distance and a gate an element go with neither caps, sinks, kept first tokens nor chunks")
        if spec.joined and (spec.gate or spec.wide_gate):
            raise ValueError("normed attention: gates are made beside the queries by the layer's own product")
        self.keep_first = self.keep_first_of(spec)
        heads, width = spec.num_heads, spec.head_width
        self.layout = HeadLayout(heads, spec.num_kv_heads, width, None if spec.own_keys else heads * width)
        # nothing to do to the projections' heads: they are what the attention reads
        self.direct = (
            spec.norm is None and not spec.rot_dims and spec.values != "take" and spec.dim == spec.vdim == width and not spec.gate
            and not spec.keys_as_values and not spec.wide_gate
        )
        names = ["q", "k"] if spec.own_keys and spec.keys_as_values else ["q", "k", "v"] if spec.own_keys else ["q"]
        self.opening = [(tensors[name], tensors[name + ".b"] if spec.bias else None) for name in names]
        if spec.gate or spec.wide_gate:
            self.opening.append((tensors["g"], None))
        self.gate_first = sum(weight.shape[0] for weight, _ in self.opening[: len(names)])  # the gates' first column
        # a bias by distance and a gate an element leave the attention as rows of `vdim` a head: the kernels write them so
        self.finished = spec.distance is not None or spec.wide_gate
        self.distance_bias = None
        if spec.distance is not None:
            table = tensors["rel"].float()[spec.distance.by_distance().to(tensors["rel"].device)]  # [reach, heads]
            self.distance_bias = kernels.prepare_distance_bias(table.t().contiguous())
        self.q_norm = tensors.get("q.norm") if spec.norm else None
        self.k_norm = tensors.get("k.norm") if spec.norm else None
        self.blend = float(tensors["vmix"].float()) if spec.values == "take" else 0.0
        self.sinks = kernels.to_device(tensors["sink"].float().contiguous()) if spec.sink else None
        out = tensors["o"]
        if width != spec.vdim and not self.finished:  # the results' columns beyond vdim are zeros: the weight gets columns for them
            wide = torch.zeros((spec.hidden_size, heads, width), dtype=out.dtype, device=out.device)
            wide[:, :, : spec.vdim] = out.view(spec.hidden_size, heads, spec.vdim)
            out = wide.view(spec.hidden_size, heads * width)
        self.closing = (out.contiguous(), tensors["o.b"] if spec.out_bias else None)
        if not spec.joined:
            self.inputs = kernels.prepare_linear(*side_by_side(self.opening))  # [q | k | v | gates]
            self.out = kernels.prepare_linear([self.closing[0]], [self.closing[1]] if spec.out_bias else None)
        self.frequencies = None
        if spec.rot_dims:
            shared = kernels.__dict__.setdefault("_rotary_frequencies", {})
            key = (spec.rot_dims, spec.theta, spec.scaling)
            if key not in shared:
                frequencies, magnitude = rotary_frequencies(spec.rot_dims, spec.theta, spec.scaling)
                shared[key] = (kernels.to_device(frequencies), magnitude)
            self.frequencies, self.magnitude = shared[key]

    @staticmethod
    def keep_first_of(spec: NormedAttentionSpec) -> int:
        return spec.keep_first if spec.window is not None else 0

    def forward(self, x: torch.Tensor, batch, cell) -> torch.Tensor:
        kernels, spec = self.kernels, self.spec
        projected = kernels.linear(x, self.inputs)  # [T, q | k | v | gates]
        if self.finished:
            return kernels.linear(self.mix(projected, batch, cell, None), self.out, out_dtype=torch.float32, partial=True)
        plain = spec.soft_cap is None and self.sinks is None and not spec.gate and not self.keep_first and spec.chunk is None and spec.own_keys
        if plain:  # the output projection goes with the attention: a kernel library may fuse the two
            rows, layout = self._rows(projected, batch, None)
            return kernels.rotate_store_attend(rows, layout, batch, cell, None, "none", spec.scale, spec.window, project=self.out)
        mixed = self.mix(projected, batch, cell, None)
        if spec.gate:
            kernels.scale_heads(mixed, spec.num_heads, spec.head_width, projected, self.gate_first, "sigmoid")
        return kernels.linear(mixed, self.out, out_dtype=torch.float32, partial=True)

    def _rows(self, projected, batch, cell):
        """Per token the heads' queries, keys and values as the attention reads them (normed, turned, blended, widened),
        and their layout; with a `cell` the keys and values are stored too, unless the rows are the projections."""
        kernels, spec = self.kernels, self.spec
        q_size, k_size, v_size = spec.num_heads * spec.dim, spec.stored_heads * spec.dim, spec.stored_heads * spec.vdim
        given = None
        if spec.values == "give":
            batch.computed[("given values", spec.values_name)] = (projected, q_size + k_size, v_size)
        elif spec.values == "take":
            given = batch.computed.get(("given values", spec.values_name))
            if given is None or given[2] != v_size:
                raise RuntimeError("normed attention: no earlier layer of this step gave values of this size")
        if self.direct and projected.shape[1] % 8 == 0:
            return projected, dataclasses.replace(self.layout, row_stride=projected.shape[1])
        if spec.norm == "unit" or spec.keys_as_values:
            rows = kernels.convolved_heads(
                projected, 0, q_size, q_size if spec.keys_as_values else q_size + k_size, spec.num_heads, spec.stored_heads, spec.dim, spec.vdim,
                spec.head_width, batch, cell if spec.own_keys else None, norm=spec.norm is not None, q_weight=self.q_norm, k_weight=self.k_norm,
                eps=spec.eps,
            )
            return rows, self.layout
        table = kernels.rotary_table(batch, self.frequencies, self.magnitude) if spec.rot_dims else None
        rows = kernels.assemble_heads(
            projected, 0, q_size, q_size + k_size, spec.num_heads, spec.stored_heads, spec.dim, spec.vdim, spec.head_width,
            spec.norm, self.q_norm, self.k_norm, spec.eps, table, spec.rot_dims,
            given[0] if given else None, given[1] if given else 0, self.blend,
            batch=batch, cell=cell if spec.own_keys else None, pairing=spec.pairing,
        )
        return rows, self.layout

    def mix(self, projected: torch.Tensor, batch, cell, out: torch.Tensor | None) -> torch.Tensor:
        kernels, spec = self.kernels, self.spec
        if self.finished:
            rows, layout = self._rows(projected, batch, cell)
            if rows is projected and spec.own_keys:
                kernels.rotate_and_store(rows, layout, batch, cell, None, "none")
            return kernels.paged_attention(
                rows, layout, batch, cell, spec.scale, spec.window, out=out, vdim=spec.vdim, distance_bias=self.distance_bias,
                gates=(projected, self.gate_first) if spec.wide_gate else None,
            )
        scores_as_they_are = spec.soft_cap is None and not self.keep_first
        if self.direct and scores_as_they_are and spec.own_keys:
            rows, layout = self._rows(projected, batch, None)
            if rows is projected:  # keys and values are stored by the attention's own kernel where it can
                return kernels.rotate_store_attend(
                    rows, layout, batch, cell, None, "none", spec.scale, spec.window, sinks=self.sinks, chunk=spec.chunk, out=out,
                )
            kernels.rotate_and_store(rows, layout, batch, cell, None, "none")
        else:
            rows, layout = self._rows(projected, batch, cell)
            if rows is projected and spec.own_keys:
                kernels.rotate_and_store(rows, layout, batch, cell, None, "none")
        return kernels.paged_attention(
            rows, layout, batch, cell, spec.scale, spec.window, soft_cap=spec.soft_cap, sinks=self.sinks, keep_first=self.keep_first,
            chunk=spec.chunk, out=out,
        )
