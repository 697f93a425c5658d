"""The Dubesun decoder as a list of parts: layers of differential attention behind short convolutions (some read the
keys and values of an earlier layer) or of attention with a learned bias by distance whose values are its keys, each
beside routed experts that read the same normed rows, and a learned vector of each position on the embedded rows."""

from __future__ import annotations

from ..config.dubesun import DubesunBiasedMixer, DubesunConfig, DubesunDifferenceMixer
from ..config.model import ConfigError
from ..parts import (
    DifferenceAttentionSpec,
    DistanceBuckets,
    LayerDefinition,
    LayerRun,
    ModelSpec,
    NormedAttentionSpec,
    ParallelBlockSpec,
    RMSNormSpec,
    RoutedExpertsSpec,
)
from ..registry import register_architecture


def _mixer_spec(config: DubesunConfig, index: int, mixer):
    if isinstance(mixer, DubesunDifferenceMixer):
        return DifferenceAttentionSpec(
            hidden_size=config.width, num_heads=mixer.heads, num_kv_heads=mixer.kv_heads, dim=mixer.dim, vdim=mixer.vdim, scale=mixer.scale,
            eps=config.norm_eps, difference=mixer.diff, taps=mixer.conv, temperature=mixer.temperature, own_keys=mixer.kv_from is None,
        )
    assert isinstance(mixer, DubesunBiasedMixer)
    if mixer.buckets is None:
        raise ConfigError(f"Dubesun config: layer {index}: 'buckets' is not given (a model folder's tensors give it)")
    return NormedAttentionSpec(
        hidden_size=config.width, num_heads=mixer.heads, num_kv_heads=mixer.kv_heads, dim=mixer.dim, vdim=mixer.dim, scale=mixer.scale,
        eps=config.norm_eps, bias=True, norm="unit", keys_as_values=True, distance=DistanceBuckets(mixer.buckets, mixer.bias_max),
        wide_gate=True,
    )


def dubesun_spec(config: DubesunConfig) -> ModelSpec:
    norm = RMSNormSpec(config.width, config.norm_eps, weight_name="", weight_offset=1.0)
    layers, order = [], []
    for index, layer in enumerate(config.layers):
        feed_forward = None
        if layer.mlp is not None:
            # a softmax over the chosen logits alone: the softmax over all of them, renormalised over the chosen
            feed_forward = RoutedExpertsSpec(
                hidden_size=config.width, num_experts=layer.mlp.experts, top=layer.mlp.top, expert_size=layer.mlp.expert_ff, route_scale=1.0,
                activation="limited_swish", scoring="softmax", gated=True, correction=False, renormalise=True, limit=layer.mlp.limit,
            )
        layers.append(LayerDefinition(f"l{index}.", ParallelBlockSpec(norm, _mixer_spec(config, index, layer.mixer), feed_forward)))
        # a layer over another's keys and values still has the convolution of its own queries to keep inputs for
        reads = getattr(layer.mixer, "kv_from", None)
        order.append(LayerRun(index, reads=reads, reads_only=("keys",) if reads is not None else None))
    return ModelSpec(
        vocab_size=config.vocab,
        hidden_size=config.width,
        layers=tuple(layers),
        run_order=tuple(order),
        final_norm=norm,
        tie_embeddings=False,
        embedding_name="embed",
        final_norm_name="final.norm",
        head_name="head",
        position_name="pos",
        max_positions=config.max_positions,
    )


register_architecture("Dubesun", DubesunConfig, dubesun_spec)
