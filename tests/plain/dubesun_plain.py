"""A plain, slow implementation of the Dubesun decoder, one function per mechanism, in float64 on the CPU.

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


# ---------------------------------------------------------------------------- norms, convolution, temperature


def over_root_mean_square(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, weight, eps):
    """An RMS norm whose weight is kept as its difference from one."""
    return over_root_mean_square(x, eps) * (1.0 + weight)


def convolve(u, taps):
    """u [n, channels], taps [channels, width]: row t is the sum over j of taps[:, j] times the row width - 1 - j before t."""
    n, width = u.shape[0], taps.shape[1]
    out = torch.zeros_like(u)
    for t in range(n):
        for j in range(width):
            source = t - width + 1 + j
            if source >= 0:
                out[t] += taps[:, j] * u[source]
    return out


def query_temperature(n, coef, every):
    """[n]: what the query at position p is multiplied by."""
    return torch.tensor([1.0 + coef * math.log(math.floor((p + 1) / every) + 1) for p in range(n)], dtype=F)


# ---------------------------------------------------------------------------- scores by distance


def distance_bucket(distance, buckets, furthest):
    """The first half of the buckets holds a distance each; the second half grows geometrically up to `furthest`."""
    exact = buckets // 2
    if distance < exact:
        return distance
    place = exact + math.floor(math.log(distance / exact) / math.log(furthest / exact) * (buckets - exact))
    return int(min(buckets - 1, place))


def distance_bias(n, table, furthest):
    """table [buckets, H] -> [H, n, n]: what is added to the score of query i (row) for key j <= i."""
    by_distance = torch.stack([table[distance_bucket(d, table.shape[0], furthest)] for d in range(n)])  # [n, H]
    distance = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).clamp(min=0)
    return by_distance[distance].permute(2, 0, 1)


# ---------------------------------------------------------------------------- softmax


def softmax_over(q, k, v, scale, bias=None):
    """q [n, H, d], k [n, G, d], v [n, Gv, dv]; every query sees itself and what came before; `bias` [H, n, n]."""
    n, heads, _ = q.shape
    later = torch.arange(n)[:, None] < torch.arange(n)[None, :]
    out = torch.zeros((n, heads, v.shape[-1]), dtype=F)
    for h in range(heads):
        scores = (q[:, h] @ k[:, h // (heads // k.shape[1])].T) * scale
        if bias is not None:
            scores = scores + bias[h]
        weights = torch.softmax(scores.masked_fill(later, -math.inf), dim=-1)
        out[:, h] = weights @ v[:, h // (heads // v.shape[1])]
    return out


def difference_factor(t, prefix, constant):
    one = math.exp(float((t[prefix + "lq1"] * t[prefix + "lk1"]).sum()))
    two = math.exp(float((t[prefix + "lq2"] * t[prefix + "lk2"]).sum()))
    return one - two + constant


# ---------------------------------------------------------------------------- mixers


def projected(h, m, t, prefix, name):
    """One projection behind its convolution (where the mixer has one)."""
    u = h @ t[prefix + name].T
    return convolve(u, t[prefix + name + ".conv"]) if m.get("conv") else u


def difference_keys_values(h, m, t, prefix, eps):
    n, kv_heads, dim = h.shape[0], m["kv_heads"], m["dim"]
    k = projected(h, m, t, prefix, "k").view(n, kv_heads, 2, dim)
    k = over_root_mean_square(k, eps) * t[prefix + "k.norm"]
    return k, projected(h, m, t, prefix, "v").view(n, kv_heads, m["vdim"])


def difference_mixer(h, m, t, prefix, eps, keys_values):
    """Two softmax maps a head over the same values; the second, times one learned number, is taken off the first."""
    n, heads, dim = h.shape[0], m["heads"], m["dim"]
    q = projected(h, m, t, prefix, "q").view(n, heads, 2, dim)
    q = over_root_mean_square(q, eps) * t[prefix + "q.norm"]
    if m.get("q_temp"):
        q = q * query_temperature(n, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None, None]
    k, v = keys_values
    one = softmax_over(q[:, :, 0], k[:, :, 0], v, m["scale"])
    two = softmax_over(q[:, :, 1], k[:, :, 1], v, m["scale"])
    mixed = one - difference_factor(t, prefix, m["diff"]) * two
    mixed = over_root_mean_square(mixed, eps) * (1.0 - m["diff"])
    return mixed.reshape(n, heads * m["vdim"]) @ t[prefix + "o"].T


def biased_mixer(h, m, t, prefix, eps):
    """The values are the keys as they were projected; scores have a learned bias by distance; the result is gated."""
    n, heads, kv_heads, dim = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ t[prefix + "q"].T + t[prefix + "q.b"]).view(n, heads, dim)
    k = (h @ t[prefix + "k"].T + t[prefix + "k.b"]).view(n, kv_heads, dim)
    bias = distance_bias(n, t[prefix + "rel"], m["bias_max"])
    mixed = softmax_over(over_root_mean_square(q, eps), over_root_mean_square(k, eps), k, m["scale"], bias)
    gated = mixed.reshape(n, heads * m["vdim"]) * torch.sigmoid(h @ t[prefix + "g"].T)
    return gated @ t[prefix + "o"].T


# ---------------------------------------------------------------------------- feed-forward


def expert(h, t, prefix, limit):
    g = (h @ t[prefix + "gate"].T).clamp(max=limit)
    u = (h @ t[prefix + "up"].T).clamp(-limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ t[prefix + "down"].T


def experts(h, spec, t, prefix):
    """Every token through the experts with its largest logits, weighted by a softmax over those logits alone."""
    logits = h @ t[prefix + "router"].T
    out = torch.zeros_like(h)
    for row in range(h.shape[0]):
        best = sorted(range(spec["router"]["experts"]), key=lambda e: (-float(logits[row, e]), e))[: spec["router"]["top"]]
        weights = torch.softmax(logits[row, best], dim=-1)
        for weight, e in zip(weights, best):
            out[row] += weight * expert(h[row], t, f"{prefix}e{e}.", spec["expert"]["limit"])
    return out


# ---------------------------------------------------------------------------- the model


def forward(config, t, tokens):
    """(logits [n, vocab], the stream after every layer [layers, n, width])."""
    eps = config["norm"]["eps"]
    x = t["embed"][torch.tensor(tokens)] + t["pos"][: len(tokens)]
    keys_values, streams = {}, []
    for index, layer in enumerate(config["layers"]):
        prefix, m = f"l{index}.", layer["mixer"]
        h = norm_around_zero(x, t[prefix + "norm1"], eps)
        if layer["type"] == "attention":
            source = m.get("kv_from")
            if source is None:
                keys_values[index] = difference_keys_values(h, m, t, prefix + "mix.", eps)
            update = difference_mixer(h, m, t, prefix + "mix.", eps, keys_values[index if source is None else source])
        else:
            update = biased_mixer(h, m, t, prefix + "mix.", eps)
        if layer.get("mlp"):
            update = update + experts(h, layer["mlp"], t, prefix + "mlp.")
        x = x + update
        streams.append(x.clone())
    return norm_around_zero(x, t["final.norm"], eps) @ t["head"].T, torch.stack(streams)
