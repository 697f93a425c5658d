"""The typed configuration of the Dolezen decoder, read from its own config.json.

config.json gives every size and every constant that differs between models of the design: `vocab`, `width`,
`norm.eps`, `embedding.scale` and `layers` (per layer its `type`, the `mixer`'s sizes and its `mlp`, or null for
none).  What may be absent: `kv_heads` (as many as heads), `mask` (every earlier token is seen), `kv_from` (keys
and values of the layer's own), latent attention's `rot.dims` (all of rot_dim), `mlp`, `embedding.scale` (1).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, ClassVar

from .model import ArchitectureConfig, ConfigError, KeyReader

LAYER_TYPES = ("attention", "latent_attention")


@dataclass(frozen=True)
class DolezenAttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int | None  # mask.size: queries see their own chunk of so many positions
    kv_from: int | None  # the layer whose keys and values are read


@dataclass(frozen=True)
class DolezenLatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int | None  # mask.size: queries see the last so many tokens
    rot_base: float
    rot_dims: int


@dataclass(frozen=True)
class DolezenLayer:
    type: str
    mixer: DolezenAttentionMixer | DolezenLatentMixer
    ff: int | None


def _mapping(value: Any, where: str) -> dict[str, Any]:
    if not isinstance(value, dict):
        raise ConfigError(f"{where} must be a mapping, got {value!r}")
    return value


def _read_mask(values: dict[str, Any], where: str) -> int | None:
    if values.get("mask") is None:
        return None
    return KeyReader(_mapping(values["mask"], f"{where}.mask"), f"{where}.mask").integer("size")


def _read_mixer(kind: str, values: dict[str, Any], where: str):
    reader = KeyReader(values, where)
    heads = reader.integer("heads")
    if kind == "attention":
        return DolezenAttentionMixer(
            heads=heads, kv_heads=reader.integer("kv_heads", default=heads), dim=reader.integer("dim"), vdim=reader.integer("vdim"),
            scale=reader.number("scale"), chunk=_read_mask(values, where),
            kv_from=reader.integer("kv_from", minimum=0) if reader.optional("kv_from") is not None else None,
        )
    rot_dim = reader.integer("rot_dim")
    rot = KeyReader(_mapping(values.get("rot"), f"{where}.rot"), f"{where}.rot")
    return DolezenLatentMixer(
        heads=heads, dim=reader.integer("dim"), rot_dim=rot_dim, vdim=reader.integer("vdim"), q_rank=reader.integer("q_rank"),
        kv_rank=reader.integer("kv_rank"), scale=reader.number("scale"), window=_read_mask(values, where), rot_base=rot.number("base"),
        rot_dims=rot.integer("dims", default=rot_dim, minimum=2),
    )


def _read_mlp(values: Any, where: str) -> int | None:
    if values is None:
        return None
    reader = KeyReader(_mapping(values, where), where)
    reader.choice("kind", choices=("dense",))
    return reader.integer("ff")


@dataclass(frozen=True)
class DolezenConfig(ArchitectureConfig):
    architecture: ClassVar[str] = "Dolezen"

    vocab: int
    width: int
    norm_eps: float
    layers: tuple[DolezenLayer, ...]
    embedding_scale: float = 1.0

    def __post_init__(self) -> None:
        if not self.layers:
            raise ConfigError("Dolezen config: no layers")
        for index, layer in enumerate(self.layers):
            mixer, where = layer.mixer, f"Dolezen config: layer {index}"
            if isinstance(mixer, DolezenLatentMixer):
                if mixer.rot_dims % 2 or mixer.rot_dims > mixer.rot_dim:
                    raise ConfigError(f"{where}: rot.dims must be even and at most rot_dim")
                continue
            if mixer.heads % mixer.kv_heads:
                raise ConfigError(f"{where}: heads must be a multiple of kv_heads")
            if mixer.kv_from is not None:
                source = self.layers[mixer.kv_from].mixer if mixer.kv_from < index else None
                if not isinstance(source, DolezenAttentionMixer) or source.kv_from is not None:
                    raise ConfigError(f"{where}: kv_from must name an earlier attention layer with keys and values of its own")
                if (source.kv_heads, source.dim, source.vdim) != (mixer.kv_heads, mixer.dim, mixer.vdim):
                    raise ConfigError(f"{where}: the keys and values of layer {mixer.kv_from} are of other sizes")

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @classmethod
    def from_dict(cls, values: dict[str, Any]) -> "DolezenConfig":
        reader = KeyReader(values, "Dolezen config")
        norm = KeyReader(_mapping(values.get("norm"), "Dolezen config: norm"), "Dolezen config: norm")
        embedding = KeyReader(_mapping(values.get("embedding") or {}, "Dolezen config: embedding"), "Dolezen config: embedding")
        entries = values.get("layers")
        if not isinstance(entries, list):
            raise ConfigError("Dolezen config: 'layers' must be a list")
        layers = []
        for index, entry in enumerate(entries):
            where = f"Dolezen config: layers[{index}]"
            entry = _mapping(entry, where)
            kind = KeyReader(entry, where).choice("type", choices=LAYER_TYPES)
            mixer = _read_mixer(kind, _mapping(entry.get("mixer"), f"{where}.mixer"), f"{where}.mixer")
            layers.append(DolezenLayer(kind, mixer, _read_mlp(entry.get("mlp"), f"{where}.mlp")))
        return cls(
            vocab=reader.integer("vocab"), width=reader.integer("width"), norm_eps=norm.number("eps"), layers=tuple(layers),
            embedding_scale=embedding.number("scale", default=1.0),
        )

    def to_config_json(self) -> dict[str, Any]:
        layers = []
        for layer in self.layers:
            mixer = layer.mixer
            if isinstance(mixer, DolezenAttentionMixer):
                described: dict[str, Any] = {"heads": mixer.heads, "kv_heads": mixer.kv_heads, "dim": mixer.dim, "vdim": mixer.vdim, "scale": mixer.scale}
                if mixer.kv_from is not None:
                    described["kv_from"] = mixer.kv_from
                mask = mixer.chunk
            else:
                described = {"heads": mixer.heads, "dim": mixer.dim, "rot_dim": mixer.rot_dim, "vdim": mixer.vdim, "q_rank": mixer.q_rank,
                             "kv_rank": mixer.kv_rank, "scale": mixer.scale, "rot": {"base": mixer.rot_base, "dims": mixer.rot_dims}}
                mask = mixer.window
            if mask is not None:
                described["mask"] = {"size": mask}
            layers.append({"type": layer.type, "mixer": described, "mlp": None if layer.ff is None else {"kind": "dense", "ff": layer.ff}})
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale}, "layers": layers}
