"""Setodra, plainly: one function per mechanism, written from the design's equations, whole sequences at once (no
cache, no pages, no state carried between calls), float64 by default.  Nothing here is shared with the package: the
tests hold the engine's results against these.

``r`` is a rounding function (identity by default): with ``rounding_to(torch.bfloat16)`` the functions round where
16-bit kernels round (products' results, rows that products read, cached rows), which shows what such a run may lose.
"""
from __future__ import annotations

import json
import math
import os

import torch
from safetensors import safe_open


def same(x):
    return x


def rounding_to(dtype):
    return lambda x: x.to(dtype).to(x.dtype)


def read_folder(folder, dtype=torch.float64):
    with open(os.path.join(folder, "config.json")) as handle:
        config = json.load(handle)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as handle:
        for name in handle.keys():
            tensor = handle.get_tensor(name)
            tensors[name] = tensor.to(dtype) if tensor.is_floating_point() else tensor
    return config, tensors


def unit_root_mean_square(x, eps):
    """x / sqrt(mean(x^2) + eps), eps inside the root."""
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def norm(x, weight, eps):
    return unit_root_mean_square(x, eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def rotation(sizes):
    """(dims, frequencies in float64, what cosines and sines are multiplied by) of a mixer's ``rot``; None: nothing turns."""
    rot = sizes.get("rot")
    if not rot:
        return None
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    scaling = rot.get("scaling")
    if not scaling:
        return dims, plain, 1.0
    factor, original = scaling["factor"], scaling["original"]

    def turns_at(count):            # the dimension whose pair turns ``count`` times over the original length
        return dims * math.log(original / (2.0 * math.pi * count)) / (2.0 * math.log(base))

    low = max(math.floor(turns_at(scaling["fast"])), 0)
    high = min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    mixed = []
    for i, f in enumerate(plain):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        mixed.append(f / factor * ramp + f * (1.0 - ramp))
    return dims, mixed, 0.1 * math.log(factor) + 1.0


def rotate(x, positions, turned):
    """x [T, heads, d]: dimension i turns with dimension i + dims/2 by the angle position * f_i; the rest passes."""
    if turned is None:
        return x
    dims, freqs, amplitude = turned
    half = dims // 2
    angle = positions.to(x.dtype)[:, None] * torch.tensor(freqs, dtype=x.dtype)[None, :]
    c, s = amplitude * torch.cos(angle)[:, None, :], amplitude * torch.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def latent_attention(h, t, p, sizes, eps, r=same):
    """Keys and values from one normed latent a token, one rotated key part shared by the heads."""
    n, heads, dim, rot_dim, vdim, rank = h.shape[0], sizes["heads"], sizes["dim"], sizes["rot_dim"], sizes["vdim"], sizes["kv_rank"]
    q = r(h @ t[p + "q"].T).view(n, heads, dim + rot_dim)
    down = r(h @ t[p + "dkv"].T)
    latent = r(norm(down[:, :rank], t[p + "dkv.norm"], eps))
    turned, positions = rotation(sizes), torch.arange(n)
    key_part = r(rotate(down[:, rank:].view(n, 1, rot_dim), positions, turned))
    query_part = r(rotate(q[..., dim:], positions, turned))
    keys = (latent @ t[p + "uk"].T).view(n, heads, dim)
    values = (latent @ t[p + "uv"].T).view(n, heads, vdim)
    scores = torch.einsum("ihd,jhd->hij", q[..., :dim], keys) + torch.einsum("ihd,jd->hij", query_part, key_part[:, 0])
    hidden = torch.arange(n)[None, :] > torch.arange(n)[:, None]
    weights = r(torch.softmax((scores * sizes["scale"]).masked_fill(hidden, float("-inf")), dim=-1))
    mixed = r(torch.einsum("hij,jhd->ihd", weights, values)).reshape(n, heads * vdim)
    return r(mixed @ t[p + "o"].T)


def retention(h, t, p, sizes, eps, r=same):
    """A matrix per head under a fixed decay; no softmax, no denominator."""
    n, heads, dim, vdim = h.shape[0], sizes["heads"], sizes["dim"], sizes["vdim"]
    q, k = r(h @ t[p + "q"].T).view(n, heads, dim), r(h @ t[p + "k"].T).view(n, heads, dim)
    v = r(h @ t[p + "v"].T).view(n, heads, vdim)
    turned, positions = rotation(sizes), torch.arange(n)
    q, k = rotate(q, positions, turned), rotate(k, positions, turned) * dim ** -0.5
    decay = torch.tensor(sizes["decay"], dtype=h.dtype)
    S = torch.zeros(heads, dim, vdim, dtype=h.dtype)
    out = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for step in range(n):
        S = decay[:, None, None] * S + k[step][:, :, None] * v[step][:, None, :]
        out[step] = torch.einsum("hdv,hd->hv", S, q[step])
    out = unit_root_mean_square(out, eps).reshape(n, heads * vdim)
    return r(r(out * silu(r(h @ t[p + "g"].T))) @ t[p + "o"].T)


def short_convolution(x, taps, bias):
    """Per channel over time: the last column of ``taps`` meets the token itself, the one before it the token before."""
    count = taps.shape[1]
    padded = torch.cat([x.new_zeros(count - 1, x.shape[1]), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(count)) + bias


def mamba2(h, t, p, sizes, eps, r=same):
    """State-space duality: one decay per head and token, keys and queries (B and C) shared by groups of heads."""
    n, heads, vdim, state, groups = h.shape[0], sizes["heads"], sizes["vdim"], sizes["state"], sizes["groups"]
    inner, each = heads * vdim, heads // groups
    both = r(h @ t[p + "in"].T)
    z, through, dt = both[:, :inner], both[:, inner:2 * inner + 2 * groups * state], both[:, 2 * inner + 2 * groups * state:]
    through = r(silu(short_convolution(through, t[p + "conv"], t[p + "conv.b"])))
    x = through[:, :inner].view(n, heads, vdim)
    B = through[:, inner:inner + groups * state].view(n, groups, state).repeat_interleave(each, dim=1)
    C = through[:, inner + groups * state:].view(n, groups, state).repeat_interleave(each, dim=1)
    dt = torch.nn.functional.softplus(dt + t[p + "dt_bias"], threshold=1e9)
    decay = torch.exp(-torch.exp(t[p + "A_log"]) * dt)
    S = torch.zeros(heads, state, vdim, dtype=h.dtype)
    y = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for step in range(n):
        S = decay[step][:, None, None] * S + dt[step][:, None, None] * B[step][:, :, None] * x[step][:, None, :]
        y[step] = torch.einsum("hnv,hn->hv", S, C[step]) + t[p + "D"][:, None] * x[step]
    y = y.reshape(n, inner) * silu(z)
    y = unit_root_mean_square(y.view(n, sizes["norm_groups"], -1), eps).reshape(n, inner) * t[p + "norm"]
    return r(r(y) @ t[p + "o"].T)


def mixer(kind, h, t, p, sizes, eps, r=same):
    return {"latent_attention": latent_attention, "retention": retention, "mamba2": mamba2}[kind](h, t, p, sizes, eps, r)


def gated(h, t, p, r=same):
    return r(silu(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


def route(h, t, p, router):
    """(chosen [T, top], weights [T, top]): the choice is made with the correction, the weights without it."""
    scores = torch.softmax(h @ t[p + "router"].T, dim=-1)
    chosen = torch.topk(scores + t[p + "correction"], router["top"], dim=-1).indices
    picked = scores.gather(1, chosen)
    return chosen, picked / (picked.sum(dim=-1, keepdim=True) + 1e-20) * router["scale"]


def experts(h, t, p, mlp, r=same):
    chosen, weights = route(h, t, p, mlp["router"])
    out = torch.zeros_like(h)
    for token in range(h.shape[0]):
        row = h[token:token + 1]
        for e, w in zip(chosen[token].tolist(), weights[token]):
            out[token] += w * (row if e >= mlp["router"]["experts"] else gated(row, t, f"{p}e{e}.", r))[0]
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ t[p + "shared.sg"].T) * gated(h, t, p + "shared.", r)
    return out


def passes(config):
    """The layers in the order they run: (layer, number of the pass that begins right before it or None)."""
    count, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(count)]
    runs = [(i, None) for i in range(loop["start"])]
    for number in range(loop["times"]):
        runs += [(i, number if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], count)]


def forward(config, t, tokens, r=same, keep=None):
    """Logits [T, vocab] of a whole sequence.  ``keep``: a list that gets the stream behind every layer run."""
    eps = config["norm"]["eps"]
    begin = t["embed"][torch.tensor(tokens)] * (config.get("embedding") or {}).get("scale", 1.0)
    x = begin
    for index, number in passes(config):
        if number is not None:
            if number:
                x = x + begin
            x = x + t["loop.step"][number]
        layer, p = config["layers"][index], f"l{index}."
        x = x + mixer(layer["type"], r(norm(x, t[p + "norm1"], eps)), t, p + "mix.", layer["mixer"], eps, r)
        if layer.get("mlp") is not None:
            x = x + experts(r(norm(x, t[p + "norm2"], eps)), t, p + "mlp.", layer["mlp"], r)
        if keep is not None:
            keep.append(x)
    return r(norm(x, t["final.norm"], eps)) @ t["head"].T


def greedy_generate(config, t, prompt, new_tokens):
    tokens = list(prompt)
    for _ in range(new_tokens):
        tokens.append(int(forward(config, t, tokens)[-1].argmax()))
    return tokens[len(prompt):]
