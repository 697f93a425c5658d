"""Small Dolezen models for the tests: configurations as config.json mappings, random tensors that make every
mechanism count, and model folders.

The sizes differ from layer to layer and avoid coincidences (dim != vdim both ways, heads / kv_heads of 1, 2 and 3,
chunks and windows that are no multiple of a page, scales that are no power of dim, latents of sizes of their own, a
rotation of less than rot_dim, a layer without a feed-forward, layers that read another's keys and values through a
mask of another size)."""

from __future__ import annotations

from pathlib import Path

import torch

from tests.dafutar_cases import run_steps, tokens_of, write_folder as _write_folder  # noqa: F401  (generic helpers)


def attention(heads=6, kv_heads=2, dim=24, vdim=40, chunk=14, scale=0.23, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": mixer}


def latent(heads=3, dim=16, rot_dim=8, vdim=24, q_rank=20, kv_rank=32, scale=0.21, base=700.0, window=11, dims=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
             "rot": {"base": base, "dims": rot_dim if dims is None else dims}}
    if window is not None:
        mixer["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": mixer}


def config_of(layers, vocab=67, width=40, eps=1e-4, scale=1.7):
    """`layers`: [(mixer entry, ff or None)]."""
    return {"architecture": "Dolezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": [dict(mixer, mlp={"kind": "dense", "ff": ff} if ff is not None else None) for mixer, ff in layers]}


# A model with every kind of layer in an order of its own and sizes that differ wherever they can; layers 3 and 5 read the
# keys and values of layers 0 and 2, one through a longer chunk than their owner's and one through a shorter one.
MIXED = config_of(
    [
        (attention(heads=6, kv_heads=2, dim=24, vdim=40, chunk=14), 56),
        (latent(heads=3, dim=16, rot_dim=8, vdim=24, window=11), None),
        (attention(heads=2, kv_heads=1, dim=40, vdim=8, chunk=30, scale=0.17), 20),
        (attention(heads=4, kv_heads=2, dim=24, vdim=40, chunk=21, scale=0.4, kv_from=0), 72),
        (latent(heads=2, dim=8, rot_dim=16, vdim=8, q_rank=12, kv_rank=16, scale=0.4, window=37, dims=10), 24),
        (attention(heads=3, kv_heads=1, dim=40, vdim=8, chunk=9, kv_from=2), None),
    ]
)


def random_tensors(values: dict, seed: int, *, sharp: bool = False) -> dict[str, torch.Tensor]:
    """bfloat16 tensors (the precision model folders hold) by the model's own list of names and shapes.  Matrices are
    drawn so that activations stay of order one; norms, biases and sinks are far enough from one and zero to matter.
    `sharp`: queries and keys are large, so that a softmax looks at one key."""
    from llmserve_amd.registry import resolve_architecture

    architecture = resolve_architecture(values)
    spec = architecture.build_spec(architecture.config_class.from_dict(values))
    generator = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, wanted in spec.tensors().items():
        shape = wanted.shape
        last = name.rsplit(".", 1)[-1]
        if name == "embed":
            value = torch.randn(shape, generator=generator)
        elif last == "sink":
            value = 1.0 + torch.randn(shape, generator=generator)
        elif last == "b":
            value = 0.4 * torch.randn(shape, generator=generator)
        elif wanted.role == "norm":
            value = 1.0 + 0.3 * torch.randn(shape, generator=generator)
        else:
            value = 1.4 * torch.randn(shape, generator=generator) / shape[-1] ** 0.5
            if sharp and last in ("q", "k", "uq", "uk"):
                value = 2.0 * value
        tensors[name] = value.to(torch.bfloat16)
    return tensors


def write_folder(folder: Path, values: dict, seed: int = 1, *, sharp: bool = False, tensors: dict | None = None) -> Path:
    return _write_folder(folder, values, seed, tensors=tensors if tensors is not None else random_tensors(values, seed, sharp=sharp))
