"""Feed-forward parts."""

from __future__ import annotations

from dataclasses import dataclass

import torch

from .base import FEED_FORWARDS, Part, TensorSpec


class FeedForward(Part):
    """`forward(x)` takes the normed rows [T, hidden] in the run dtype and
    returns the float32 rows to add to the residual stream, or partial sums
    [parts, T, hidden] of them."""

    def forward(self, x: torch.Tensor, batch) -> torch.Tensor:
        raise NotImplementedError


@dataclass(frozen=True)
class GatedMLPSpec:
    hidden_size: int
    intermediate_size: int
    activation: str = "silu"
    kind: str = "gated_mlp"
    # the tensors' names below the part's prefix: gate, up, down
    names: tuple[str, str, str] = ("gate_proj.weight", "up_proj.weight", "down_proj.weight")
    # of the activation "limited_swish": g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(1.702 g) (u + 1)
    limit: float | None = None


@FEED_FORWARDS.register("gated_mlp")
class GatedMLP(FeedForward):
    """down(act(gate(x)) * up(x)) without biases (reference `model.py:180-188`).
    Gate and up run as one product whose epilogue applies act(gate) * up."""

    @classmethod
    def tensors(cls, spec: GatedMLPSpec) -> dict[str, TensorSpec]:
        gate, up, down = spec.names
        return {
            gate: TensorSpec((spec.intermediate_size, spec.hidden_size)),
            up: TensorSpec((spec.intermediate_size, spec.hidden_size)),
            down: TensorSpec((spec.hidden_size, spec.intermediate_size)),
        }

    def __init__(self, spec: GatedMLPSpec, tensors, kernels) -> None:
        super().__init__(spec, tensors, kernels)
        # the kernel library says which activations it has, and refuses another by name
        gate, up, down = spec.names
        if spec.limit is None:
            self.gate_up = kernels.prepare_gated_linear(tensors[gate], tensors[up], spec.activation)
        else:
            self.gate_up = kernels.prepare_gated_linear(tensors[gate], tensors[up], spec.activation, limit=spec.limit)
        self.down = kernels.prepare_linear([tensors[down]], None)

    def forward(self, x: torch.Tensor, batch) -> torch.Tensor:
        activated = self.kernels.gated_linear(x, self.gate_up)
        return self.kernels.linear(activated, self.down, out_dtype=torch.float32, partial=True)


@dataclass(frozen=True)
class DenseMLPSpec:
    """`names`: the tensors' names below the part's prefix: up, down.  `joined`: as a mixer's (`Mixer`): both products are
    the block's."""

    hidden_size: int
    intermediate_size: int
    activation: str = "squared_relu"
    names: tuple[str, str] = ("up", "down")
    joined: bool = False
    kind: str = "dense_mlp"


@FEED_FORWARDS.register("dense_mlp")
class DenseMLP(FeedForward):
    """down(act(up(x))) without biases."""

    joins = True

    @classmethod
    def tensors(cls, spec: DenseMLPSpec) -> dict[str, TensorSpec]:
        up, down = spec.names
        return {
            up: TensorSpec((spec.intermediate_size, spec.hidden_size)),
            down: TensorSpec((spec.hidden_size, spec.intermediate_size)),
        }

    def __init__(self, spec: DenseMLPSpec, tensors, kernels) -> None:
        super().__init__(spec, tensors, kernels)
        up, down = (tensors[name] for name in spec.names)
        self.activation = spec.activation
        self.opening, self.closing = [(up, None)], (down, None)
        if not spec.joined:
            self.up = kernels.prepare_linear([up], None)
            self.down = kernels.prepare_linear([down], None)

    def forward(self, x: torch.Tensor, batch) -> torch.Tensor:
        _, inner = self.kernels.activated_linear(x, self.up, self.activation)
        return self.kernels.linear(inner, self.down, out_dtype=torch.float32, partial=True)
