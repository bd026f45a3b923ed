"""Shared by the Neruzen tests: small configurations, model folders with seeded random weights, ways of cutting a run."""

from __future__ import annotations

import copy
import json
import os
import random
import tempfile
from functools import lru_cache

import numpy as np
import torch

import plain_neruzen

_TMP = tempfile.TemporaryDirectory(prefix="llmx_amd_neruzen_")


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, window, base, dims=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                  "scale": scale, "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim if dims is None else dims}}}


def lightning(dim, vdim, decay):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}}


def retention(dim, vdim, decay, base, dims):
    return {"type": "retention", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": dims}}}


def moe(experts, groups, keep, top, ff, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def model(vocab, width, eps, bigram, layers):
    return {"architecture": "Neruzen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": layers}


# A: sizes the matrix-core kernels take, pages of 16: every mixer, experts with and without a shared one, a layer without a
#    feed-forward; windows that end inside pages; cache rows that need padding (48 + 8) and rows that do not (32 + 32); 16 heads.
CONFIG_A = model(320, 128, 1e-6, (211, 13, 5), [
    layer(latent(4, 24, 8, 40, 48, 48, 0.2, 40, 3000.0), moe(6, 3, 2, 2, 32, 48)),
    layer(retention(16, 24, (0.9, 0.97, 0.995), 500.0, 8), None),
    layer(latent(16, 16, 32, 16, 64, 32, 0.15, 101, 50000.0), moe(4, 2, 1, 1, 48)),
    layer(lightning(40, 16, (0.75, 0.998)), moe(8, 4, 2, 3, 24, 24)),
])
# B: sizes no kernel tiles evenly (the universal kernels run), pages of 4; one bucket; groups of one expert; every expert of
#    the kept groups picked; decays of 1 and close to 0; a window of 5.
CONFIG_B = model(97, 54, 1e-5, (1, 3, 2), [
    layer(lightning(7, 9, (0.5,)), moe(3, 3, 2, 2, 10, 5)),
    layer(latent(3, 5, 6, 7, 9, 10, 0.45, 5, 77.0), moe(6, 2, 1, 3, 7)),
    layer(retention(10, 6, (1.0, 0.01), 77.0, 10), moe(5, 5, 1, 1, 11, 13)),
])
# C: edges: a window of one key; a window wider than any prompt here; no rotated dims of a retention's heads and all of them;
#    key widths at and above a wave; multipliers far above the buckets; the last layer without a feed-forward.
CONFIG_C = model(128, 64, 1e-6, (37, 10 ** 12 + 39, 2 * 10 ** 9 + 11), [
    layer(latent(2, 16, 16, 8, 32, 64, 0.3, 1, 5000.0), moe(8, 1, 1, 2, 16, 16)),
    layer(retention(80, 40, (0.99, 0.999, 0.95, 0.6), 100.0, 80), moe(4, 4, 2, 2, 24)),
    layer(latent(8, 8, 8, 24, 16, 16, 0.25, 400, 100.0, 4), moe(16, 4, 2, 4, 8, 40)),
    layer(lightning(64, 100, (0.98,)), moe(2, 1, 1, 1, 32, 8)),
    layer(retention(24, 8, (0.9, 0.99), 1000.0, 0), None),
])
# D: states of 128 x 128 and 200 x 33, a latent of 128 with a rotated part of 64, windows on and one beyond a page's border
CONFIG_D = model(512, 256, 1e-6, (1000, 31337, 7), [
    layer(retention(128, 128, (0.96875, 0.99609375), 10000.0, 64), moe(16, 4, 2, 4, 32, 64)),
    layer(latent(6, 48, 64, 32, 80, 128, 0.09, 64, 500000.0), moe(8, 2, 1, 4, 64, 64)),
    layer(lightning(200, 33, (0.995,)), moe(4, 2, 2, 4, 16)),
    layer(latent(4, 64, 16, 96, 96, 64, 0.11, 65, 1000.0), None),
])
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D}
PAGES = {"A": 16, "B": 4, "C": 16, "D": 16}
SEEDS = {"A": 51, "B": 52, "C": 53, "D": 54}


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
    rng = random.Random(4241 * seed + length)
    return [rng.randrange(CONFIGS[name]["vocab"]) for _ in range(length)]


@lru_cache(maxsize=None)
def plain_logits(name: str, length: int, seed: int):
    config, tensors = plain(name)
    return torch.from_numpy(plain_neruzen.forward(config, tensors, tokens_for(name, length, seed)))


class Picks:
    """An engine observer that keeps every routed layer's picks and router logits by (request, position)."""

    def __init__(self):
        self.rows = {}      # request -> {layer: {position: (ids, logits)}}

    def __call__(self, step, kind, **tensors):
        if kind != "routing":
            return
        ids, z = tensors["ids"].cpu().numpy(), tensors["logits"].cpu().numpy()
        for e in step.entries:
            at = self.rows.setdefault(e.request, {}).setdefault(step.run_index, {})
            for r in range(e.n):
                at[e.past + r] = (ids[e.row0 + r].copy(), z[e.row0 + r].copy())

    def of(self, request, length):
        """{layer: ids [length, top]} of a request."""
        return {i: np.stack([rows[p][0] for p in range(length)]) for i, rows in self.rows[request].items()}

    def logits_of(self, request, length):
        return {i: np.stack([rows[p][1] for p in range(length)]) for i, rows in self.rows[request].items()}


def greedy(config, tensors, prompt, n):
    """n tokens, each the largest logit after everything before it (the whole sequence is run again for each)."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(np.argmax(plain_neruzen.forward(config, tensors, seq)[-1])))
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
