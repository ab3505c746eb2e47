"""Mefurax, plainly: one function per mechanism, written from the design's equations, whole sequences at once (no
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


def norm_around_zero(x, weight, eps):
    """The stored weight is what is added to 1."""
    return unit_root_mean_square(x, eps) * (1.0 + weight)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def projected(h, t, name, r=same):
    y = h @ t[name].T
    if name + ".b" in t:
        y = y + t[name + ".b"]
    return r(y)


def convolved(u, taps):
    """Per channel over time: the last column of ``taps`` meets the token itself, the one before it the token before."""
    count = taps.shape[1]
    before = torch.cat([u.new_zeros(count - 1, u.shape[1]), u])
    return sum(before[j:j + u.shape[0]] * taps[:, j] for j in range(count))


def rotate_pairs(x, positions, dims, base):
    """x [T, heads, d]: dimensions 2i and 2i + 1 turn together by position * base^(-2i/dims); those from ``dims`` on pass."""
    freqs = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    angle = positions.to(x.dtype)[:, None] * freqs[None, :]
    c, s = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2], out[..., 1:dims:2] = u * c - v * s, v * c + u * s
    return out


def slopes(heads):
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def in_window(n, size):
    """[i, j]: whether position i sees position j, itself and the size - 1 before it (None: all before it)."""
    back = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (back >= 0) & (back < size) if size is not None else back >= 0


def in_chunk(n, size):
    """[i, j]: whether j is not behind i and lies in the same chunk of ``size`` positions counted from 0."""
    place = torch.arange(n)
    seen = place[:, None] >= place[None, :]
    return seen & (place[:, None] // size == place[None, :] // size) if size is not None else seen


def softmax_over(scores, seen):
    return torch.softmax(scores.masked_fill(~seen, float("-inf")), dim=-1)


def attend(q, k, v, sizes, bend, seen, r=same):
    """q [T, H, d], k [T, G, d], v [T, G, vdim] -> [T, H, vdim]; ``bend(scores [H, T, T])`` is what scaled scores become."""
    share = sizes["heads"] // sizes.get("kv_heads", sizes["heads"])
    k, v = k.repeat_interleave(share, dim=1), v.repeat_interleave(share, dim=1)
    scores = bend(torch.einsum("ihd,jhd->hij", q, k) * sizes["scale"])
    return torch.einsum("hij,jhd->ihd", r(softmax_over(scores, seen)), v)


def mixed_values(v, t, p, sizes, firsts, r=same):
    """The layer's values after mixing with those of the first layer that mixes; ``firsts``: a list, empty before that layer."""
    if not sizes.get("v_mix"):
        return r(v)
    if not firsts:
        firsts.append(r(v))
        return firsts[0]
    lam = t[p + "vmix"]
    return r((1.0 - lam) * v + lam * firsts[0])


def attention(h, t, p, sizes, eps, firsts, r=same):
    """Convolved projections, norms over the whole projection, no rotation, a bias that grows with the distance, a window."""
    n, H, G, dim, vdim = h.shape[0], sizes["heads"], sizes.get("kv_heads", sizes["heads"]), sizes["dim"], sizes["vdim"]
    q, k, v = (convolved(projected(h, t, p + name, r), t[p + name + ".conv"]) for name in "qkv")
    q, k = r(norm(q, t[p + "q.norm"], eps)).view(n, H, dim), r(norm(k, t[p + "k.norm"], eps)).view(n, G, dim)
    v = mixed_values(v, t, p, sizes, firsts, r).view(n, G, vdim)
    back = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).to(h.dtype)
    slope = torch.tensor(slopes(H), dtype=h.dtype)[:, None, None]
    out = attend(q, k, v, sizes, lambda s: s - slope * back, in_window(n, (sizes.get("mask") or {}).get("size")), r)
    return r(r(out).reshape(n, H * vdim) @ t[p + "o"].T)


def attention_2(h, t, p, sizes, eps, firsts, r=same):
    """Rotated neighbouring pairs, then heads of unit root mean square, capped scores, chunks, a gate a head."""
    n, H, G, dim, vdim = h.shape[0], sizes["heads"], sizes.get("kv_heads", sizes["heads"]), sizes["dim"], sizes["vdim"]
    positions, rot, cap = torch.arange(n), sizes["rot"], sizes["softcap"]
    q = projected(h, t, p + "q", r).view(n, H, dim)
    k = projected(h, t, p + "k", r).view(n, G, dim)
    q = r(unit_root_mean_square(rotate_pairs(q, positions, rot["dims"], rot["base"]), eps))
    k = r(unit_root_mean_square(rotate_pairs(k, positions, rot["dims"], rot["base"]), eps))
    v = mixed_values(projected(h, t, p + "v", r), t, p, sizes, firsts, r).view(n, G, vdim)
    out = attend(q, k, v, sizes, lambda s: cap * torch.tanh(s / cap), in_chunk(n, (sizes.get("mask") or {}).get("size")), r)
    out = out * torch.sigmoid(projected(h, t, p + "g", r))[:, :, None]
    return r(r(out).reshape(n, H * vdim) @ t[p + "o"].T)


def mixer(kind, h, t, p, sizes, eps, firsts, r=same):
    return {"attention": attention, "attention_2": attention_2}[kind](h, t, p, sizes, eps, firsts, r)


def dense(h, t, p, r=same):
    gate, up = r(h @ t[p + "gate"].T), r(h @ t[p + "up"].T)
    return r(r(gelu_tanh(gate) * up) @ t[p + "down"].T)


def expert(h, t, p, r=same):
    return r(relu_squared(h @ t[p + "up"].T)) @ t[p + "down"].T


def shared_expert(h, t, p, r=same):
    """The same; a 16-bit run makes it of products of its own, each of whose results it rounds."""
    return r(r(relu_squared(r(h @ t[p + "up"].T))) @ t[p + "down"].T)


def route(h, t, p, router):
    """(chosen [T, top], weights [T, top]): the largest logits, weighted by the softmax over the chosen ones."""
    picked, chosen = torch.topk(h @ t[p + "router"].T, router["top"], dim=-1)
    return chosen, torch.softmax(picked, dim=-1)


def experts(h, read, t, p, mlp, r=same):
    """``h``: the rows the router sees; ``read``: the rows the experts see (a 16-bit run rounds those)."""
    chosen, weights = route(h, t, p, mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        token, place = torch.nonzero(chosen == e, as_tuple=True)
        if len(token):
            out[token] += weights[token, place][:, None] * expert(read[token], t, f"{p}e{e}.", r)
    if mlp.get("shared"):
        out = out + shared_expert(read, t, p + "shared.", r)
    return out


def forward(config, t, tokens, r=same, keep=None):
    """Logits [T, vocab] of a whole sequence.  ``keep``: a list that gets the stream behind every layer."""
    eps, alpha = config["norm"]["eps"], config["postln_alpha"]
    x = t["embed"][torch.tensor(tokens)]
    firsts = []
    for index, layer in enumerate(config["layers"]):
        p = f"l{index}."
        x = norm_around_zero(alpha * x + mixer(layer["type"], r(x), t, p + "mix.", layer["mixer"], eps, firsts, r), t[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            y = dense(r(x), t, p + "mlp.", r) if mlp["kind"] == "dense" else experts(x, r(x), t, p + "mlp.", mlp, r)
            x = norm_around_zero(alpha * x + y, t[p + "norm2"], eps)
        if keep is not None:
            keep.append(x)
    return r(norm_around_zero(x, t["final.norm"], eps)) @ t["head"].T


def greedy_generate(config, t, prompt, new_tokens):
    tokens = list(prompt)
    for _ in range(new_tokens):
        tokens.append(int(forward(config, t, tokens)[-1].argmax()))
    return tokens[len(prompt):]
