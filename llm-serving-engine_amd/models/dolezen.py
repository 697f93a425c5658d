"""The Dolezen decoder as a list of parts: layers of attention in chunks with a sink (some read the keys and values
of an earlier layer) or of latent attention over a window, each beside a dense feed-forward that reads the same
normed rows, and a scale on the embedded rows."""

from __future__ import annotations

from ..config.dolezen import DolezenAttentionMixer, DolezenConfig, DolezenLatentMixer
from ..parts import (
    DenseMLPSpec,
    LatentAttentionSpec,
    LayerDefinition,
    LayerRun,
    ModelSpec,
    NormedAttentionSpec,
    ParallelBlockSpec,
    RMSNormSpec,
)
from ..registry import register_architecture


def _mixer_spec(config: DolezenConfig, mixer):
    if isinstance(mixer, DolezenAttentionMixer):
        return NormedAttentionSpec(
            hidden_size=config.width, num_heads=mixer.heads, num_kv_heads=mixer.kv_heads, dim=mixer.dim, vdim=mixer.vdim,
            scale=mixer.scale, eps=config.norm_eps, chunk=mixer.chunk, bias=True, out_bias=True, norm=None, sink=True,
            own_keys=mixer.kv_from is None,
        )
    assert isinstance(mixer, DolezenLatentMixer)
    return LatentAttentionSpec(
        hidden_size=config.width, num_heads=mixer.heads, dim=mixer.dim, rot_dim=mixer.rot_dim, vdim=mixer.vdim, q_rank=mixer.q_rank,
        kv_rank=mixer.kv_rank, scale=mixer.scale, eps=config.norm_eps, rot_dims=mixer.rot_dims, theta=mixer.rot_base, pairing="half",
        window=mixer.window,
    )


def dolezen_spec(config: DolezenConfig) -> ModelSpec:
    norm = RMSNormSpec(config.width, config.norm_eps, weight_name="")
    layers, order = [], []
    for index, layer in enumerate(config.layers):
        feed_forward = DenseMLPSpec(config.width, layer.ff, "squared_relu") if layer.ff is not None else None
        layers.append(LayerDefinition(f"l{index}.", ParallelBlockSpec(norm, _mixer_spec(config, layer.mixer), feed_forward)))
        order.append(LayerRun(index, reads=getattr(layer.mixer, "kv_from", None)))
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
        embedding_scale=config.embedding_scale,
    )


register_architecture("Dolezen", DolezenConfig, dolezen_spec)
