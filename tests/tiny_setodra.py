"""The tests' own small Setodra configurations; they differ in every size, constant and option: the order of the layers,
layers without a feed-forward, loops over several layers, over one layer, passed once and not there at all, rotations of a
part of a head, of the whole head and of nothing, with and without stretching, heads that are no multiple of anything, groups
of one head, of several and of all, parts of the norm that cut through heads, convolutions of one, two, four and six taps,
routers with and without identity experts, with and without a shared expert, that use one and that use all."""
from __future__ import annotations

import functools
import tempfile

import plain_setodra as plain
from llmserver_amd.config import config_from_dict
from llmserver_amd.weights import RandomInit, write_random_model


def rotation(dims, base, scaling=None):
    rot = {"dims": dims, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return rot


def latent(heads, dim, rot_dim, vdim, rank, scale, base, scaling=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                                  "rot": rotation(rot_dim, base, scaling)}}


def retention(dim, vdim, decay, rot=None):
    mixer = {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        mixer["rot"] = rotation(*rot)
    return {"type": "retention", "mixer": mixer}


def space(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}}


def moe(ff, experts, top, scale=1.0, identity=None, shared=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if identity is not None:
        router["identity"] = identity
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def config(vocab, width, eps, layers, **top):
    return {"architecture": "Setodra", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": [{**mixer, "mlp": mlp} for mixer, mlp in layers], **top}


SA = config(97, 48, 1e-5, [
    (space(4, 6, 10, 2, 4, 3), moe(20, 5, 2, 1.7, identity=3, shared=28)),
    (latent(3, 8, 12, 6, 10, 0.3, 1000.0, (4.0, 64, 8.0, 1.0)), moe(12, 7, 3, 0.8, identity=1, shared=9)),
    (retention(10, 7, (0.9, 0.99), rot=(6, 50.0)), None),
    (space(3, 10, 5, 1, 1, 1), moe(16, 4, 4, 2.5, identity=2))],
    loop={"start": 1, "stop": 3, "times": 3}, embedding={"scale": 2.0})
SB = config(130, 64, 1e-6, [
    (retention(16, 20, (0.8, 0.95, 0.999)), moe(24, 6, 1, 1.2)),
    (latent(2, 12, 6, 20, 26, 0.22, 1e6), None),
    (space(6, 8, 12, 6, 6, 2), moe(10, 3, 2, 1.0, identity=4, shared=40)),
    (latent(5, 6, 16, 4, 7, 0.4, 300.0, (2.5, 100, 20.0, 3.0)), moe(33, 8, 2, 1.0, shared=7))])
# Sizes in the kernels' own steps (heads of 32 and 64, cache rows of 48, pages of 16, experts of 32)
SC = config(200, 64, 3e-5, [
    (space(4, 32, 64, 2, 4, 2), moe(32, 8, 3, 1.5, identity=4, shared=64)),
    (retention(32, 64, (0.97, 0.999), rot=(32, 2e4)), moe(32, 4, 2, 1.0, identity=4, shared=32)),
    (latent(4, 32, 16, 32, 32, 0.16, 5e4, (8.0, 32, 4.0, 1.0)), moe(64, 6, 2, 1.3, identity=2, shared=32))],
    loop={"start": 0, "stop": 3, "times": 2}, embedding={"scale": 0.7})
SD = config(50, 32, 3e-4, [(space(2, 8, 8, 1, 2, 2), moe(12, 5, 5, 0.9, identity=1, shared=16))], loop={"start": 0, "stop": 1, "times": 1})
SE = config(61, 40, 1e-5, [
    (retention(8, 8, (0.5,), rot=(8, 100.0)), moe(9, 2, 1, 1.0, identity=1)),
    (space(5, 4, 3, 5, 3, 4), None)],
    loop={"start": 1, "stop": 2, "times": 2}, embedding={"scale": 3.0})

CASES = {"SA": (SA, RandomInit(seed=3, std=0.15, norm_noise=0.3, bias_std=0.3), 16),
         "SB": (SB, RandomInit(seed=8, std=0.12, norm_noise=0.2, bias_std=0.2), 8),
         "SC": (SC, RandomInit(seed=5, std=0.1, norm_noise=0.3, bias_std=0.2), 16),
         "SD": (SD, RandomInit(seed=2, std=0.25, norm_noise=0.3, bias_std=0.3), 8),
         "SE": (SE, RandomInit(seed=21, std=0.2, norm_noise=0.25, bias_std=0.3), 4)}

_FOLDERS = {}


def model_folder(case: str) -> str:
    if case not in _FOLDERS:
        raw, init, _ = CASES[case]
        folder = tempfile.mkdtemp(prefix=f"llmserver_amd_test_{case}_")
        write_random_model(config_from_dict(dict(raw)), folder, init)
        _FOLDERS[case] = folder
    return _FOLDERS[case]


@functools.lru_cache(maxsize=None)
def plain_model(case: str):
    return plain.read_folder(model_folder(case))


@functools.lru_cache(maxsize=None)
def plain_logits(case: str, tokens: tuple):
    raw, tensors = plain_model(case)
    return plain.forward(raw, tensors, list(tokens))
