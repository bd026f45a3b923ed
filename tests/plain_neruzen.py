"""Neruzen computed plainly: whole sequences, float64, no cache, one function a mechanism.

This file shares no code with `llmx_amd`; it reads a configuration (a dict with config.json's keys) and a dict of numpy
arrays by the model folder's tensor names.  Notation: T tokens, E the model's width, H heads, D key width, R rotated key
width, V value width, C latent width, F an inner feed-forward width; weights are [out, in] and applied as x @ W.T.

Input:        x_t = embed[token_t] + bigram[row], row = (previous * a + token * b) mod buckets, the table's last row for the
              sequence's first token
A layer:      h = N(x); x <- x + (mixer(S(h)) + ff(h))     N(y) = y / rms(y) * w, one norm for both sublayers;
              S(h)_t = h_t + (h_(t-1) - h_t) * s (h_(-1) = 0), s a factor a coordinate
Mixers:       "latent_attention": windowed softmax attention whose queries, keys and values are low-rank expansions
              "lightning":        S_t = g_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t over silu projections, one norm over all heads
              "retention":        the same recurrence over rotated q and k, every head's result of unit rms
Feed-forward: gated units (silu) of which a router picks some, by groups, beside one that always runs; or none
Output:       N, then an untied head
"""

from __future__ import annotations

import math

import numpy as np


# ---------------------------------------------------------------------------- small pieces
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def softmax_rows(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def rotate_halves(x, positions, rot):
    """x [T, ..., D]: dims (i, i + dims/2), i < dims/2, turn by positions * base^(-2i/dims); dims beyond `dims` pass."""
    dims = int(rot["dims"])
    if dims == 0:
        return x
    half = dims // 2
    f = float(rot["base"]) ** (-2.0 * np.arange(half, dtype=np.float64) / dims)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    shape = (len(positions),) + (1,) * (x.ndim - 2) + (half,)
    c, s = np.cos(angle).reshape(shape), np.sin(angle).reshape(shape)
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


# ---------------------------------------------------------------------------- input
def bigram_rows(tokens, cfg):
    """The bigram table's row of every token of a sequence."""
    rows = []
    for i, t in enumerate(tokens):
        if i == 0:
            rows.append(int(cfg["buckets"]))
        else:
            rows.append((int(tokens[i - 1]) * int(cfg["mul_prev"]) + int(t) * int(cfg["mul_cur"])) % int(cfg["buckets"]))
    return rows


def embed(tokens, W, config):
    return W["embed"][np.asarray(tokens)] + W["bigram"][np.asarray(bigram_rows(tokens, config["embedding"]["bigram"]))]


def token_shift(h, s):
    before = np.concatenate([np.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * s


# ---------------------------------------------------------------------------- mixers
def window_mask(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i - j < size)


def latent_attention(h, W, p, cfg, eps):
    T = h.shape[0]
    H, D, R, V, C = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    cq = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps)
    q = (cq @ W[p + "uq"].T).reshape(T, H, D + R)
    down = h @ W[p + "dkv"].T
    c = rms_norm(down[:, :C], W[p + "dkv.norm"], eps)
    positions = np.arange(T)
    k_rot = rotate_halves(down[:, C:], positions, cfg["rot"])
    q_rot = rotate_halves(q[..., D:], positions, cfg["rot"])
    k = (c @ W[p + "uk"].T).reshape(T, H, D)
    v = (c @ W[p + "uv"].T).reshape(T, H, V)
    mask = window_mask(T, cfg["mask"]["size"])
    out = np.zeros((T, H, V))
    for n in range(H):
        s = (q[:, n, :D] @ k[:, n].T + q_rot[:, n] @ k_rot.T) * cfg["scale"]
        out[:, n] = softmax_rows(np.where(mask, s, -np.inf)) @ v[:, n]
    return out.reshape(T, H * V) @ W[p + "o"].T


def decayed_outer_products(q, k, v, decay, state=None):
    """q, k [T, H, D], v [T, H, V], decay [H]: S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  Returns (o [T, H, V], S [H, D, V])."""
    T, H, D = q.shape
    V = v.shape[2]
    S = np.zeros((H, D, V)) if state is None else np.array(state, dtype=np.float64)
    g = np.asarray(decay, dtype=np.float64)[:, None, None]
    o = np.zeros((T, H, V))
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def lightning(h, W, p, cfg, eps):
    T = h.shape[0]
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = silu(h @ W[p + "q"].T).reshape(T, H, D)
    k = silu(h @ W[p + "k"].T).reshape(T, H, D)
    v = silu(h @ W[p + "v"].T).reshape(T, H, V)
    o, _ = decayed_outer_products(q, k, v, cfg["decay"])
    y = rms_norm(o.reshape(T, H * V), W[p + "norm"], eps) * sigmoid(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


def retention(h, W, p, cfg, eps):
    T = h.shape[0]
    H, D, V = cfg["heads"], cfg["dim"], cfg["vdim"]
    positions = np.arange(T)
    q = rotate_halves((h @ W[p + "q"].T).reshape(T, H, D), positions, cfg["rot"])
    k = rotate_halves((h @ W[p + "k"].T).reshape(T, H, D), positions, cfg["rot"]) * D ** -0.5
    v = (h @ W[p + "v"].T).reshape(T, H, V)
    o, _ = decayed_outer_products(q, k, v, cfg["decay"])
    y = rms_unit(o, eps).reshape(T, H * V) * silu(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


# ---------------------------------------------------------------------------- feed-forward
def gated_unit(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(h, W, p, cfg, picks=None):
    """(ids [T, top], weights [T, top], logits [T, X]): softmax scores over all experts; the `keep` groups (of neighbours)
    with the largest best score stay in, of their experts the `top` best are picked (the lowest number first among
    equals); the weights are the picked scores over their sum.  `picks` replaces the choice, not the scores."""
    r = cfg["router"]
    X, top = r["experts"], r["top"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ W[p + "router"].T
    s = softmax_rows(z)
    if picks is None:
        G, per = groups["count"], X // groups["count"]
        ids = np.zeros((h.shape[0], top), dtype=np.int64)
        for t in range(h.shape[0]):
            best = np.array([s[t, g * per:(g + 1) * per].max() for g in range(G)])
            kept = np.argsort(-best, kind="stable")[: groups["keep"]]
            key = np.full(X, -np.inf)
            for g in kept:
                key[g * per:(g + 1) * per] = s[t, g * per:(g + 1) * per]
            ids[t] = np.argsort(-key, kind="stable")[:top]
    else:
        ids = np.asarray(picks)
    picked = np.take_along_axis(s, ids, axis=-1)
    return ids, picked / (picked.sum(axis=-1, keepdims=True) + 1e-20), z


def experts(h, W, p, cfg, picks=None):
    ids, weights, _ = route(h, W, p, cfg, picks)
    out = np.zeros((h.shape[0], W[p + "e0.down"].shape[0]))
    for e in range(cfg["router"]["experts"]):
        where, slot = np.nonzero(ids == e)
        if len(where):
            np.add.at(out, where, weights[where, slot][:, None] * gated_unit(h[where], W, f"{p}e{e}."))
    if cfg.get("shared"):
        out = out + gated_unit(h, W, p + "shared.")
    return out


# ---------------------------------------------------------------------------- the model
MIXERS = {"latent_attention": latent_attention, "lightning": lightning, "retention": retention}


def layer(x, W, i, config, picks=None):
    entry, eps = config["layers"][i], config["norm"]["eps"]
    h = rms_norm(x, W[f"l{i}.norm1"], eps)
    y = MIXERS[entry["type"]](token_shift(h, W[f"l{i}.shift"]), W, f"l{i}.mix.", entry["mixer"], eps)
    if entry.get("mlp") is not None:
        y = y + experts(h, W, f"l{i}.mlp.", entry["mlp"], picks)
    return x + y


def forward(config, W, tokens, picks=None, layers_out=None):
    """Logits [T, vocab] of the whole sequence; `picks` {layer: ids [T, top]} replaces the router's choice in those layers;
    `layers_out` (a list) receives the residual after every layer."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    x = embed(tokens, W, config)
    for i in range(len(config["layers"])):
        x = layer(x, W, i, config, None if picks is None else picks.get(i))
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, W["final.norm"], config["norm"]["eps"]) @ W["head"].T
