"""The tests' own small Mefurax configurations; they differ in every size, constant and option: the order of the layers, layers
without a feed-forward, dense and routed ones, with and without a shared expert, windows and chunks shorter and longer than a
page and than a sequence and not there at all, groups of one head, of several and of all, heads that are no multiple of
anything, values wider and narrower than the keys, rotations of a part and of the whole head, convolutions of one to six taps,
capped and uncapped scores, values mixed in all layers, in some, in one and in none, first mixed in either kind of layer."""
from __future__ import annotations

import functools
import tempfile

import plain_mefurax as plain
from llmserver_amd.config import config_from_dict
from llmserver_amd.weights import RandomInit, write_random_model


def sloped(heads, kv_heads, dim, vdim, scale, conv, window, v_mix=True):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv, "v_mix": v_mix}
    if window is not None:
        mixer["mask"] = {"size": window}
    return {"type": "attention", "mixer": mixer}


def chunked(heads, kv_heads, dim, vdim, scale, rot, cap, chunk, v_mix=True):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"dims": rot[0], "base": rot[1]}, "softcap": cap,
             "v_mix": v_mix}
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    return {"type": "attention_2", "mixer": mixer}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def config(vocab, width, eps, alpha, layers):
    return {"architecture": "Mefurax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha,
            "layers": [{**mixer, "mlp": mlp} for mixer, mlp in layers]}


MA = config(97, 48, 1e-5, 1.7, [
    (chunked(3, 1, 10, 6, 0.4, (4, 1000.0), 6.0, 12), moe(20, 5, 2, 28)),
    (sloped(4, 2, 6, 3, 0.5, 3, 9), dense(40)),
    (chunked(4, 2, 8, 3, 0.35, (8, 50.0), 20.0, 21), None),
    (sloped(6, 3, 5, 2, 0.6, 2, 17), moe(12, 7, 3))])
MB = config(130, 64, 1e-6, 3.0, [
    (sloped(5, 5, 8, 4, 0.3, 6, None), moe(24, 6, 1, 9)),
    (chunked(2, 2, 12, 20, 0.22, (6, 1e5), 3.0, None, v_mix=False), moe(10, 3, 3, 40)),
    (sloped(2, 1, 16, 20, 0.2, 1, 30), None),
    (chunked(4, 4, 6, 5, 0.5, (2, 300.0), 50.0, 40), dense(70))])
# Sizes in the kernels' own steps (heads of 32 and 64, pages of 16, experts of 32)
MC = config(200, 64, 3e-5, 1.2, [
    (chunked(4, 2, 64, 32, 0.125, (32, 2e4), 15.0, 48), dense(96)),
    (sloped(4, 4, 32, 16, 0.2, 4, 40), moe(32, 8, 3, 64)),
    (sloped(8, 1, 16, 64, 0.3, 3, 100), moe(64, 4, 2, 32)),
    (chunked(2, 2, 32, 32, 0.25, (32, 5e4), 8.0, 32), moe(32, 6, 1))])
MD = config(50, 32, 3e-4, 0.8, [(sloped(3, 3, 8, 5, 0.5, 2, 1), dense(24))])
ME = config(61, 40, 1e-5, 2.0, [
    (sloped(2, 2, 6, 7, 0.4, 5, 6, v_mix=False), None),
    (chunked(3, 3, 4, 9, 0.7, (4, 100.0), 2.0, 5, v_mix=False), moe(9, 2, 2)),
    (chunked(1, 1, 30, 11, 0.2, (10, 10.0), 4.0, 1), dense(33))])

CASES = {"MA": (MA, RandomInit(seed=3, std=0.15, norm_noise=0.3, bias_std=0.3), 16),
         "MB": (MB, RandomInit(seed=8, std=0.12, norm_noise=0.2, bias_std=0.2), 8),
         "MC": (MC, RandomInit(seed=5, std=0.12, norm_noise=0.3, bias_std=0.3), 16),
         "MD": (MD, RandomInit(seed=2, std=0.25, norm_noise=0.3, bias_std=0.3), 8),
         "ME": (ME, RandomInit(seed=21, std=0.2, norm_noise=0.25, bias_std=0.3), 4)}

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
