"""Shared by the Vivulorn tests: small configurations, model folders with seeded random weights, ways of cutting a run."""

from __future__ import annotations

import copy
import json
import os
import random
import tempfile
from functools import lru_cache

import numpy as np
import torch

import plain_vivulorn

_TMP = tempfile.TemporaryDirectory(prefix="llmx_amd_vivulorn_")


def attention(heads, kv_heads, dim, vdim, scale, base, dims, scaling=None):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base):
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                                "rot": {"base": base, "dims": rot_dim}}


def delta(heads, kv_heads, dim, vdim, conv):
    return "delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def model(vocab, width, eps, scale, softcap, loop, layers):
    """layers: ((type, mixer), ff or None); loop: (start, stop, times) or None."""
    out = {"architecture": "Vivulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": [{"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}} for (kind, mixer), ff in layers]}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if softcap:
        out["logit_softcap"] = softcap
    return out


# A: sizes the matrix-core products and attentions take; keys shared by two heads, values narrower than keys in one layer (the rules
#    kernel) and as wide in another; part of a head rotated; a delta rule in the run that repeats and one behind it.
CONFIG_A = model(312, 96, 1e-6, 2.5, 11.0, (1, 3, 2), [
    (attention(4, 2, 32, 32, 0.21, 10000.0, 16, (4.0, 64, 16.0, 2.0)), 112),
    (attention(6, 3, 48, 32, 0.17, 5000.0, 48, (3.0, 256, 24.0, 1.5)), 64),
    (delta(4, 2, 16, 24, 3), 80),
    (latent(3, 24, 16, 40, 48, 0.19, 700.0), 128),
    (delta(2, 2, 40, 16, 4), None),
])
# B: sizes no kernel tiles evenly; pages of 4; one key head for all heads; a convolution of one tap; the repeated run starts the
#    model; odd widths; no soft cap; a frequency blend whose ramp has no width.
CONFIG_B = model(97, 54, 1e-3, 0.75, None, (0, 2, 3), [
    (delta(3, 3, 5, 7, 1), 21),
    (attention(3, 1, 10, 6, 0.5, 77.0, 6, (2.0, 7, 1.1, 1.0)), None),
    (latent(3, 5, 6, 7, 10, 0.45, 30.0), 10),
    (delta(4, 1, 9, 3, 5), None),
])
# C: the whole model repeats; wide and narrow heads; no rotated dims; no blend; one head; more taps than short prompts have tokens;
#    latent heads that make two column groups.
CONFIG_C = model(160, 64, 1e-5, 1.0, 30.0, (0, 4, 2), [
    (latent(18, 8, 8, 16, 32, 0.3, 400.0), 48),
    (attention(2, 2, 16, 48, 0.25, 500.0, 0), 40),
    (delta(2, 1, 72, 40, 8), None),
    (attention(1, 1, 128, 128, 0.1, 1e6, 64), 24),
])
# D: recurrent layers only (no pages), no repeated run; a head wider than the model; a state of 200 x 33
CONFIG_D = model(80, 48, 1e-6, 1.5, 20.0, None, [
    (delta(2, 1, 200, 33, 2), 72),
    (delta(5, 5, 12, 64, 4), None),
    (delta(4, 2, 128, 128, 4), 32),
])
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D}
PAGES = {"A": 16, "B": 4, "C": 16, "D": 16}
SEEDS = {"A": 71, "B": 72, "C": 73, "D": 74}


def write_folder(config: dict, seed: int, folder: str, edit=None) -> str:
    """A model folder of `config` with the framework's seeded random weights; `edit(tensors)` may change them first."""
    from llmx_amd import RandomInit
    from llmx_amd.models import read_config
    from llmx_amd.weights.folder import random_tensors
    from llmx_amd.weights.safetensors_io import write_safetensors
    cfg = read_config(copy.deepcopy(config))
    tensors = random_tensors(cfg, RandomInit(seed=seed, std=0.08, norm_std=0.2, bias_range=0.5, storage="bfloat16"))
    if edit is not None:
        edit(tensors)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors, metadata={"format": "pt"})
    return folder


@lru_cache(maxsize=None)
def model_folder(name: str) -> str:
    return write_folder(CONFIGS[name], SEEDS[name], os.path.join(_TMP.name, name))


def load_plain(folder: str):
    """(config dict, {name: float64 numpy array}) of a model folder, read with the safetensors package."""
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    tensors = {k: v.to(torch.float64).numpy() for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return config, tensors


@lru_cache(maxsize=None)
def plain(name: str):
    return load_plain(model_folder(name))


def tokens_for(name: str, length: int, seed: int):
    rng = random.Random(7919 * seed + length)
    return [rng.randrange(CONFIGS[name]["vocab"]) for _ in range(length)]


@lru_cache(maxsize=None)
def plain_logits(name: str, length: int, seed: int):
    config, tensors = plain(name)
    return torch.from_numpy(plain_vivulorn.forward(config, tensors, tokens_for(name, length, seed)))


def greedy(config, tensors, prompt, n):
    """n tokens, each the largest logit after everything before it (the whole sequence is run again for each)."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(np.argmax(plain_vivulorn.forward(config, tensors, seq)[-1])))
    return seq[len(prompt):]


def portions(length: int, seed: int, smallest: int = 2):
    """Cuts [0, length) into portions of changing size, several of them of `smallest` tokens."""
    rng = random.Random(seed)
    cuts, at = [], 0
    sizes = [smallest, 7, smallest, 16, 3, 33, smallest, 64, 5]
    while at < length:
        n = min(length - at, sizes[len(cuts) % len(sizes)] if rng.random() < 0.7 else rng.randrange(1, 40))
        cuts.append((at, at + n))
        at += n
    return cuts
