"""Small Dubesun models for the tests: configurations as config.json mappings, random tensors that make every
mechanism count, and model folders.

The sizes differ from layer to layer and avoid coincidences (a map's dim no half of vdim, both ways, one to three query
heads a key head, convolutions of one to six taps and none, temperatures that change every few tokens and none, tables of
distances of several lengths, limits that bite, experts of odd widths, layers without a feed-forward, readers that have
other head counts and convolutions than the layer they read)."""

from __future__ import annotations

from pathlib import Path

import torch

from tests.dafutar_cases import run_steps, tokens_of, write_folder as _write_folder  # noqa: F401  (generic helpers)


def difference(heads=6, kv_heads=2, dim=24, vdim=40, scale=0.23, diff=0.35, conv=4, coef=0.4, every=5, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if conv is not None:
        mixer["conv"] = conv
    if coef is not None:
        mixer["q_temp"] = {"coef": coef, "every": every}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer}


def biased(heads=4, kv_heads=2, dim=24, scale=0.3, bias_max=37, buckets=10):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                                             "bias_max": bias_max, "buckets": buckets}}


def experts(count=5, top=2, ff=24, limit=0.9):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": count, "top": top}}


def config_of(layers, vocab=67, width=40, eps=1e-4, max_positions=512):
    """`layers`: [(mixer entry, feed-forward entry or None)]."""
    return {"architecture": "Dubesun", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
            "layers": [dict(mixer, mlp=mlp) for mixer, mlp in layers]}


# A model with every kind of layer in an order of its own and sizes that differ wherever they can; layers 3 and 5 read the
# keys and values of layers 0 and 2.
MIXED = config_of(
    [
        (difference(heads=6, kv_heads=2, dim=24, vdim=40, conv=4), experts(5, 2, 24)),
        (biased(heads=6, kv_heads=2, dim=16, bias_max=37, buckets=10), None),
        (difference(heads=3, kv_heads=1, dim=8, vdim=24, conv=2, coef=None, diff=0.6, scale=0.5), experts(3, 3, 20, limit=0.4)),
        (difference(heads=2, kv_heads=2, dim=24, vdim=40, conv=6, every=11, diff=0.2, scale=0.4, kv_from=0), experts(7, 1, 8)),
        (biased(heads=3, kv_heads=3, dim=40, bias_max=90, buckets=22, scale=0.15), experts(4, 3, 33)),
        (difference(heads=5, kv_heads=1, dim=8, vdim=24, conv=None, kv_from=2), None),
    ]
)


def random_tensors(values: dict, seed: int) -> dict[str, torch.Tensor]:
    """bfloat16 tensors (the precision model folders hold) by the model's own list of names and shapes.  Matrices are
    drawn so that activations stay of order one; norms, biases, distances, positions and the vectors of lambda are far
    enough from one and zero to matter."""
    from llmserve_amd.registry import resolve_architecture

    architecture = resolve_architecture(values)
    spec = architecture.build_spec(architecture.config_class.from_dict(values))
    generator = torch.Generator().manual_seed(seed)
    tensors = {}
    for name, wanted in spec.tensors().items():
        shape = wanted.shape
        last = name.rsplit(".", 1)[-1]
        value = torch.randn(shape, generator=generator)
        if name == "embed":
            pass
        elif name == "pos":
            value = 0.7 * value
        elif last == "norm1" or name == "final.norm":  # kept as differences from one
            value = 0.3 * value
        elif last == "norm":
            value = 1.0 + 0.3 * value
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            value = value / shape[0] ** 0.25
        elif last == "conv":
            value = value / shape[1] ** 0.5
        elif last == "b":
            value = 0.4 * value
        elif last == "rel":
            value = 1.5 * value
        elif last == "router":
            value = 2.0 * value / shape[-1] ** 0.5
        else:
            value = 1.4 * value / shape[-1] ** 0.5
        tensors[name] = value.to(torch.bfloat16)
    return tensors


def write_folder(folder: Path, values: dict, seed: int = 1, *, tensors: dict | None = None) -> Path:
    """The folder's config.json leaves the length of the tables of distances to the tensors."""
    tensors = tensors if tensors is not None else random_tensors(values, seed)
    bare = dict(values, layers=[dict(layer, mixer={key: value for key, value in layer["mixer"].items() if key != "buckets"}) for layer in values["layers"]])
    return _write_folder(folder, bare, seed, tensors=tensors)
