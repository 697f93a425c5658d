"""A plain, slow implementation of the Dolezen decoder, one function per mechanism, in float64 on the CPU.

It shares no code with the engine: it reads a model folder's config.json as a plain dict and its tensors by
name, and runs a whole sequence at once (no cache, no pages).  The tests compare the engine with it; `forward`
also returns the residual stream after every layer.

Notation: W x means `x @ W.T` for a weight stored [out, in]; positions count from 0; n tokens.
"""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F = torch.float64


def read_folder(folder):
    from safetensors import safe_open

    folder = Path(folder)
    config = json.loads((folder / "config.json").read_text())
    tensors = {}
    with safe_open(str(folder / "model.safetensors"), framework="pt", device="cpu") as source:
        for name in source.keys():
            value = source.get_tensor(name)
            tensors[name] = value.to(F) if value.dtype.is_floating_point else value
    return config, tensors


# ---------------------------------------------------------------------------- norm, rotation


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def turn_halves(x, positions, dims, base):
    """x [n, heads, width]: dimension i turns with dimension i + dims / 2, by the angle position * base^(-2i / dims); the
    dimensions from `dims` on pass unchanged."""
    out = x.clone()
    for i in range(dims // 2):
        angle = positions.to(F) * float(base) ** (-2.0 * i / dims)
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[..., i], x[..., i + dims // 2]
        out[..., i] = u * cos - v * sin
        out[..., i + dims // 2] = v * cos + u * sin
    return out


# ---------------------------------------------------------------------------- who sees whom


def window_mask(n, size):
    """[n, n]: query i (row) sees key j where 0 <= i - j < size; every earlier one where size is None."""
    distance = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (distance >= 0) & (distance < (size if size is not None else n + 1))


def chunk_mask(n, size):
    """[n, n]: query i sees key j <= i of its own chunk of `size` positions, counted from position 0."""
    place = torch.arange(n)
    seen = place[:, None] >= place[None, :]
    if size is not None:
        seen &= (place // size)[:, None] == (place // size)[None, :]
    return seen


# ---------------------------------------------------------------------------- softmax


def softmax_over(q, k, v, scale, seen, sinks=None):
    """q [n, H, d], k [n, G, d], v [n, G, dv]; `sinks` [H]: an exponential more in every denominator of its head."""
    n, heads, _ = q.shape
    out = torch.zeros((n, heads, v.shape[-1]), dtype=F)
    for h in range(heads):
        g = h // (heads // k.shape[1])
        scores = (q[:, h] @ k[:, g].T) * scale
        scores = scores.masked_fill(~seen, -math.inf)
        top = scores.max(-1, keepdim=True).values
        if sinks is not None:
            top = torch.maximum(top, sinks[h].expand_as(top))
        weights = torch.exp(scores - top)
        total = weights.sum(-1, keepdim=True)
        if sinks is not None:
            total = total + torch.exp(sinks[h] - top)
        out[:, h] = (weights / total) @ v[:, g]
    return out


# ---------------------------------------------------------------------------- mixers


def attention_keys_values(h, m, t, prefix):
    n, kv_heads = h.shape[0], m["kv_heads"]
    k = (h @ t[prefix + "k"].T + t[prefix + "k.b"]).view(n, kv_heads, m["dim"])
    v = (h @ t[prefix + "v"].T + t[prefix + "v.b"]).view(n, kv_heads, m["vdim"])
    return k, v


def attention_mixer(h, m, t, prefix, keys_values):
    n, heads = h.shape[0], m["heads"]
    q = (h @ t[prefix + "q"].T + t[prefix + "q.b"]).view(n, heads, m["dim"])
    k, v = keys_values
    mask = m.get("mask")
    mixed = softmax_over(q, k, v, m["scale"], chunk_mask(n, mask["size"] if mask else None), t[prefix + "sink"])
    return mixed.reshape(n, heads * m["vdim"]) @ t[prefix + "o"].T + t[prefix + "o.b"]


def latent_mixer(h, positions, m, t, prefix, eps):
    heads, dim, rot_dim, vdim, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    n, rot, mask = h.shape[0], m["rot"], m.get("mask")
    q = (rms_norm(h @ t[prefix + "dq"].T, t[prefix + "dq.norm"], eps) @ t[prefix + "uq"].T).view(n, heads, dim + rot_dim)
    down = h @ t[prefix + "dkv"].T
    c = rms_norm(down[:, :rank], t[prefix + "dkv.norm"], eps)
    shared = turn_halves(down[:, rank:].view(n, 1, rot_dim), positions, rot["dims"], rot["base"])
    turned = turn_halves(q[..., dim:], positions, rot["dims"], rot["base"])
    keys = (c @ t[prefix + "uk"].T).view(n, heads, dim)
    values = (c @ t[prefix + "uv"].T).view(n, heads, vdim)
    mixed = softmax_over(
        torch.cat([q[..., :dim], turned], dim=-1), torch.cat([keys, shared.expand(n, heads, rot_dim)], dim=-1), values, m["scale"],
        window_mask(n, mask["size"] if mask else None),
    )
    return mixed.reshape(n, heads * vdim) @ t[prefix + "o"].T


# ---------------------------------------------------------------------------- feed-forward


def squared_relu(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def feed_forward(h, t, prefix):
    return squared_relu(h @ t[prefix + "up"].T) @ t[prefix + "down"].T


# ---------------------------------------------------------------------------- the model


def forward(config, t, tokens):
    """(logits [n, vocab], the stream after every layer [layers, n, width])."""
    eps = config["norm"]["eps"]
    positions = torch.arange(len(tokens))
    x = t["embed"][torch.tensor(tokens)] * config["embedding"]["scale"]
    keys_values, streams = {}, []
    for index, layer in enumerate(config["layers"]):
        prefix, m = f"l{index}.", layer["mixer"]
        h = rms_norm(x, t[prefix + "norm1"], eps)
        if layer["type"] == "attention":
            source = m.get("kv_from")
            if source is None:
                keys_values[index] = attention_keys_values(h, m, t, prefix + "mix.")
            update = attention_mixer(h, m, t, prefix + "mix.", keys_values[index if source is None else source])
        else:
            update = latent_mixer(h, positions, m, t, prefix + "mix.", eps)
        if layer.get("mlp"):
            update = update + feed_forward(h, t, prefix + "mlp.")
        x = x + update
        streams.append(x.clone())
    return rms_norm(x, t["final.norm"], eps) @ t["head"].T, torch.stack(streams)
