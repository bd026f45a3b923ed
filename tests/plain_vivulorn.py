"""Vivulorn computed plainly: whole sequences, float64, no cache, one function a mechanism.

This file shares no code with `llmx_amd`; it reads a configuration (a dict with config.json's keys) and a dict of numpy
arrays by the model folder's tensor names.  Notation: T tokens, E the model's width, H heads, G key heads, D key width, V value
width; weights are [out, in] and applied as x @ W.T.

Start:        x0 = table[token] * scale, x = x0
A layer:      x <- x + mixer(LN1(x)) ; x <- x + ff(LN2(x))       (LN with a weight and a bias; the second line only with an ff)
A pass:       before the first layer of every pass of the repeated run, x <- W_in [x ; x0]
Mixers:       "attention" (norms over whole projections, halved rotary pairs with a YaRN blend, a gate a value),
              "latent_attention" (keys and values from one latent a token, interleaved pairs, a sink a head),
              "delta" (gated delta rule with one decay a head)
Feed-forward: W_down gelu(W_up h + b) + b', the exact gelu
Output:       LN, the embedding's table, cap * tanh(logits / cap)
"""

from __future__ import annotations

import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


# ---------------------------------------------------------------------------- small pieces
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu(z):
    """z Phi(z), Phi the normal distribution function."""
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def layer_norm(x, w, b, eps):
    mu = x.mean(axis=-1, keepdims=True)
    dev = x - mu
    return dev / np.sqrt((dev * dev).mean(axis=-1, keepdims=True) + eps) * w + b


def rms_unit(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def soft_cap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


# ---------------------------------------------------------------------------- rotation
def rotary_frequencies(dims, base, scaling):
    """(frequency of each of the dims/2 pairs, the factor on cos and sin); scaling {factor, original, fast, slow}: pairs that
    turn often within `original` positions are kept, pairs that turn rarely slowed down by `factor`, a ramp between."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate(x, positions, dims, base, scaling=None, interleaved=False):
    """x [T, heads, D]: the first `dims` dims of every head turn in pairs, (i, i + dims/2) or (2i, 2i + 1); the rest pass."""
    if dims == 0:
        return x
    f, magnitude = rotary_frequencies(dims, base, scaling)
    angle = np.asarray(positions, dtype=np.float64)[:, None] * f[None, :]
    c, s = np.cos(angle)[:, None, :] * magnitude, np.sin(angle)[:, None, :] * magnitude
    first = np.arange(0, dims, 2) if interleaved else np.arange(dims // 2)
    second = first + (1 if interleaved else dims // 2)
    out = x.copy()
    u, v = x[..., first], x[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


# ---------------------------------------------------------------------------- softmax attention
def causal_attention(q, k, v, scale, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; head h reads key head h // (H / G); `sink` [H]: one more logit a head
    in the denominator, with nothing in the numerator."""
    T, H, _ = q.shape
    share = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        s = (q[:, h] @ k[:, h // share].T) * scale
        s[np.triu_indices(T, 1)] = -np.inf
        top = s.max(axis=1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        p = np.exp(s - top)
        den = p.sum(axis=1, keepdims=True)
        if sink is not None:
            den = den + np.exp(sink[h] - top)
        out[:, h] = (p / den) @ v[:, h // share]
    return out


def attention_mixer(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (rms_unit(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(T, H, D)
    k = (rms_unit(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(T, G, D)
    v = (h @ w[p + "v"].T).reshape(T, G, V)
    rot = m["rot"]
    q, k = (rotate(a, positions, rot["dims"], rot["base"], rot.get("scaling")) for a in (q, k))
    o = causal_attention(q, k, v, m["scale"]).reshape(T, H * V)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def latent_attention_mixer(h, w, p, m, eps, positions):
    """Keys and values are formed in full from the latents here: k_n = [W_uk,n c | rotated part], v_n = W_uv,n c."""
    T = h.shape[0]
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    rot = m["rot"]
    q = (h @ w[p + "q"].T).reshape(T, H, D + R)
    down = h @ w[p + "dkv"].T
    c = rms_unit(down[:, :C], eps) * w[p + "dkv.norm"]
    k_rot = rotate(down[:, None, C:], positions, rot["dims"], rot["base"], interleaved=True)
    q = np.concatenate([q[..., :D], rotate(q[..., D:], positions, rot["dims"], rot["base"], interleaved=True)], axis=-1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, D), np.repeat(k_rot, H, axis=1)], axis=-1)
    v = (c @ w[p + "uv"].T).reshape(T, H, V)
    return causal_attention(q, k, v, m["scale"], w[p + "sink"]).reshape(T, H * V) @ w[p + "o"].T


# ---------------------------------------------------------------------------- gated delta rule
def short_conv_silu(x, taps_w):
    """x [T, C]; taps_w [C, taps], the last column weighs the current token; zeros before the start; then silu."""
    T, C = x.shape
    taps = taps_w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C)), x], axis=0)
    y = np.zeros((T, C))
    for j in range(taps):
        y += padded[j:j + T] * taps_w[:, j]
    return silu(y)


def unit(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def delta_scan(q, k, v, decay, beta):
    """q, k [T, H, D], v [T, H, V], decay, beta [T, H] -> (o [T, H, V], S [H, D, V] after the last token)."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]))
    o = np.zeros(v.shape)
    for t in range(T):
        S = S * decay[t][:, None, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def delta_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv_silu(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q = np.repeat(unit(q.reshape(T, G, D)) * D ** -0.5, H // G, axis=1)
    k = np.repeat(unit(k.reshape(T, G, D)), H // G, axis=1)
    beta = sigmoid(h @ w[p + "b"].T)
    decay = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = delta_scan(q, k, v.reshape(T, H, V), decay, beta)
    y = rms_unit(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).reshape(T, H, V)
    return y.reshape(T, H * V) @ w[p + "o"].T


# ---------------------------------------------------------------------------- feed-forward, pass input, the model
def feed_forward(h, w, p):
    return gelu(h @ w[p + "up"].T + w[p + "up.b"]) @ w[p + "down"].T + w[p + "down.b"]


def pass_input(x, x0, w_in):
    return np.concatenate([x, x0], axis=1) @ w_in.T


def run_order(config):
    """[(layer, whether a pass of the repeated run starts here)] in the order the layers run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    return ([(i, False) for i in range(a)] + [(i, i == a) for _ in range(times) for i in range(a, b)] + [(i, False) for i in range(b, n)])


def forward(config, w, tokens, trace=None):
    """Logits [T, vocab]; `trace` (a list) receives the residual stream after every layer run."""
    eps = config["norm"]["eps"]
    x0 = w["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    x = x0
    pos = np.arange(len(tokens))
    for i, opens in run_order(config):
        layer, p = config["layers"][i], f"l{i}."
        if opens:
            x = pass_input(x, x0, w["loop.in"])
        h = layer_norm(x, w[p + "norm1"], w[p + "norm1.b"], eps)
        if layer["type"] == "attention":
            x = x + attention_mixer(h, w, p + "mix.", layer["mixer"], eps, pos)
        elif layer["type"] == "latent_attention":
            x = x + latent_attention_mixer(h, w, p + "mix.", layer["mixer"], eps, pos)
        else:
            x = x + delta_mixer(h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            x = x + feed_forward(layer_norm(x, w[p + "norm2"], w[p + "norm2.b"], eps), w, p + "mlp.")
        if trace is not None:
            trace.append(x.copy())
    x = layer_norm(x, w["final.norm"], w["final.norm.b"], eps)
    return soft_cap(x @ w["embed"].T, config.get("logit_softcap"))
