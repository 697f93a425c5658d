"""The typed configuration of the Dubesun decoder, read from its own config.json.

config.json gives every size and every constant that differs between models of the design: `vocab`, `width`,
`max_positions`, `norm.eps` and `layers` (per layer its `type`, the `mixer`'s sizes and its `mlp`, or null for none).
What may be absent: `kv_heads` (as many as heads), `vdim` of a layer whose values are its keys (dim), `conv` (no
convolutions), `q_temp` (queries as they are), `kv_from` (keys and values of the layer's own), `mlp`.  How many rows a
table of distances has is read from the tensor's shape (or from the mixer's `buckets`, for a model that has no tensors yet).
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any, ClassVar

from .model import ArchitectureConfig, ConfigError, KeyReader

LAYER_TYPES = ("attention", "attention_2")


@dataclass(frozen=True)
class DubesunDifferenceMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    conv: int | None  # taps of the convolutions over queries, keys and values
    temperature: tuple[float, int] | None  # q_temp.coef and q_temp.every
    kv_from: int | None  # the layer whose keys and values are read


@dataclass(frozen=True)
class DubesunBiasedMixer:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    bias_max: float  # the distance at which the last bucket begins
    buckets: int | None  # rows of the table of biases


@dataclass(frozen=True)
class DubesunExperts:
    experts: int
    top: int
    expert_ff: int
    limit: float


@dataclass(frozen=True)
class DubesunLayer:
    type: str
    mixer: DubesunDifferenceMixer | DubesunBiasedMixer
    mlp: DubesunExperts | None


def _mapping(value: Any, where: str) -> dict[str, Any]:
    if not isinstance(value, dict):
        raise ConfigError(f"{where} must be a mapping, got {value!r}")
    return value


def _read_mixer(kind: str, values: dict[str, Any], where: str):
    reader = KeyReader(values, where)
    heads = reader.integer("heads")
    kv_heads = reader.integer("kv_heads", default=heads)
    dim, scale = reader.integer("dim"), reader.number("scale")
    if kind == "attention_2":
        if reader.integer("vdim", default=dim) != dim:
            raise ConfigError(f"{where}: the values are the keys, so 'vdim' is 'dim'")
        return DubesunBiasedMixer(
            heads=heads, kv_heads=kv_heads, dim=dim, scale=scale, bias_max=reader.number("bias_max"),
            buckets=reader.integer("buckets", minimum=2) if reader.optional("buckets") is not None else None,
        )
    temperature = None
    if values.get("q_temp") is not None:
        temp = KeyReader(_mapping(values["q_temp"], f"{where}.q_temp"), f"{where}.q_temp")
        temperature = (temp.number("coef"), temp.integer("every"))
    return DubesunDifferenceMixer(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=reader.integer("vdim"), scale=scale, diff=reader.number("diff"),
        conv=reader.integer("conv") if reader.optional("conv") is not None else None, temperature=temperature,
        kv_from=reader.integer("kv_from", minimum=0) if reader.optional("kv_from") is not None else None,
    )


def _read_mlp(values: Any, where: str) -> DubesunExperts | None:
    if values is None:
        return None
    reader = KeyReader(_mapping(values, where), where)
    reader.choice("kind", choices=("moe",))
    router = KeyReader(_mapping(values.get("router"), f"{where}.router"), f"{where}.router")
    expert = KeyReader(_mapping(values.get("expert"), f"{where}.expert"), f"{where}.expert")
    return DubesunExperts(experts=router.integer("experts"), top=router.integer("top"), expert_ff=expert.integer("ff"), limit=expert.number("limit"))


@dataclass(frozen=True)
class DubesunConfig(ArchitectureConfig):
    architecture: ClassVar[str] = "Dubesun"

    vocab: int
    width: int
    max_positions: int
    norm_eps: float
    layers: tuple[DubesunLayer, ...]

    def __post_init__(self) -> None:
        if not self.layers:
            raise ConfigError("Dubesun config: no layers")
        for index, layer in enumerate(self.layers):
            mixer, where = layer.mixer, f"Dubesun config: layer {index}"
            if mixer.heads % mixer.kv_heads:
                raise ConfigError(f"{where}: heads must be a multiple of kv_heads")
            if layer.mlp is not None and layer.mlp.top > layer.mlp.experts:
                raise ConfigError(f"{where}: more experts a token than there are")
            if layer.mlp is not None and not layer.mlp.limit > 0:
                raise ConfigError(f"{where}: the experts' limit must be positive")
            if isinstance(mixer, DubesunBiasedMixer):
                if mixer.buckets is not None and not mixer.bias_max > mixer.buckets // 2:
                    raise ConfigError(f"{where}: bias_max must lie beyond the buckets of one distance each")
                continue
            if mixer.kv_from is not None:
                source = self.layers[mixer.kv_from].mixer if mixer.kv_from < index else None
                if not isinstance(source, DubesunDifferenceMixer) or source.kv_from is not None:
                    raise ConfigError(f"{where}: kv_from must name an earlier attention layer with keys and values of its own")
                if (source.kv_heads, source.dim, source.vdim) != (mixer.kv_heads, mixer.dim, mixer.vdim):
                    raise ConfigError(f"{where}: the keys and values of layer {mixer.kv_from} are of other sizes")

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def max_position_embeddings(self) -> int:
        """The longest sequence: there is a learned vector for each of so many positions."""
        return self.max_positions

    @classmethod
    def from_dict(cls, values: dict[str, Any]) -> "DubesunConfig":
        reader = KeyReader(values, "Dubesun config")
        norm = KeyReader(_mapping(values.get("norm"), "Dubesun config: norm"), "Dubesun config: norm")
        entries = values.get("layers")
        if not isinstance(entries, list):
            raise ConfigError("Dubesun config: 'layers' must be a list")
        layers = []
        for index, entry in enumerate(entries):
            where = f"Dubesun config: layers[{index}]"
            entry = _mapping(entry, where)
            kind = KeyReader(entry, where).choice("type", choices=LAYER_TYPES)
            mixer = _read_mixer(kind, _mapping(entry.get("mixer"), f"{where}.mixer"), f"{where}.mixer")
            layers.append(DubesunLayer(kind, mixer, _read_mlp(entry.get("mlp"), f"{where}.mlp")))
        return cls(
            vocab=reader.integer("vocab"), width=reader.integer("width"), max_positions=reader.integer("max_positions"),
            norm_eps=norm.number("eps"), layers=tuple(layers),
        )

    def with_sizes_of(self, shapes: dict[str, tuple[int, ...]]) -> "DubesunConfig":
        """The sizes that config.json leaves to the tensors' shapes, read from `shapes` (name -> shape)."""
        layers = []
        for index, layer in enumerate(self.layers):
            mixer, table = layer.mixer, shapes.get(f"l{index}.mix.rel")
            if isinstance(mixer, DubesunBiasedMixer) and mixer.buckets is None and table is not None:
                layer = replace(layer, mixer=replace(mixer, buckets=int(table[0])))
            layers.append(layer)
        return replace(self, layers=tuple(layers))

    def to_config_json(self) -> dict[str, Any]:
        layers = []
        for layer in self.layers:
            mixer, mlp = layer.mixer, layer.mlp
            described: dict[str, Any] = {"heads": mixer.heads, "kv_heads": mixer.kv_heads, "dim": mixer.dim, "scale": mixer.scale}
            if isinstance(mixer, DubesunDifferenceMixer):
                described.update(vdim=mixer.vdim, diff=mixer.diff)
                if mixer.conv is not None:
                    described["conv"] = mixer.conv
                if mixer.temperature is not None:
                    described["q_temp"] = {"coef": mixer.temperature[0], "every": mixer.temperature[1]}
                if mixer.kv_from is not None:
                    described["kv_from"] = mixer.kv_from
            else:
                described.update(vdim=mixer.dim, bias_max=mixer.bias_max)
                if mixer.buckets is not None:
                    described["buckets"] = mixer.buckets
            feed = None
            if mlp is not None:
                feed = {"kind": "moe", "expert": {"ff": mlp.expert_ff, "limit": mlp.limit}, "router": {"experts": mlp.experts, "top": mlp.top}}
            layers.append({"type": layer.type, "mixer": described, "mlp": feed})
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "max_positions": self.max_positions,
                "norm": {"eps": self.norm_eps}, "layers": layers}
