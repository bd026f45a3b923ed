"""Vivulorn on the CPU: the plain implementation's functions against cases with known answers, the configuration reader's refusals,
and the assembly's tensor list and run order."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest

import plain_vivulorn as plain
from vivulorn_cases import CONFIGS, CONFIG_A, CONFIG_C, CONFIG_D, load_plain, model_folder


def test_layer_norm_and_gelu():
    rng = np.random.default_rng(0)
    x = rng.normal(size=(3, 17)) * 5 + 2
    y = plain.layer_norm(x, np.ones(17), np.zeros(17), 0.0)
    assert np.allclose(y.mean(-1), 0.0) and np.allclose((y * y).mean(-1), 1.0)
    w, b = rng.normal(size=17), rng.normal(size=17)
    dev = x - x.mean(-1, keepdims=True)
    assert np.allclose(plain.layer_norm(x, w, b, 0.3), dev / np.sqrt(x.var(-1, keepdims=True) + 0.3) * w + b)
    assert np.allclose(plain.gelu(np.array([0.0, 1.0, -1.0, 8.0])), [0.0, 0.8413447460685429, -0.15865525393145707, 8.0])
    assert np.isclose(plain.soft_cap(1000.0, 7.0), 7.0) and plain.soft_cap(3.0, None) == 3.0


def test_rotation_pairs_lengths_and_distance():
    rng = np.random.default_rng(1)
    x = rng.normal(size=(5, 2, 12))
    for interleaved in (False, True):
        y = plain.rotate(x, [0, 1, 7, 100, 1000], 8, 10000.0, interleaved=interleaved)
        assert np.allclose(y[..., 8:], x[..., 8:]) and np.allclose(y[0], x[0])
        assert np.allclose(np.linalg.norm(y[..., :8], axis=-1), np.linalg.norm(x[..., :8], axis=-1))
        q, k = rng.normal(size=(1, 1, 8)), rng.normal(size=(1, 1, 8))
        at = lambda v, p: plain.rotate(v, [p], 8, 500.0, interleaved=interleaved)[0, 0]
        assert np.isclose(at(q, 9) @ at(k, 4), at(q, 105) @ at(k, 100))
    e = np.zeros((1, 1, 12))
    e[0, 0, 1], e[0, 0, 5] = 1.0, 2.0
    a = 3 * 10000.0 ** (-2 / 8)
    assert np.allclose(plain.rotate(e, [3], 8, 10000.0)[0, 0, [1, 5]], [math.cos(a) - 2 * math.sin(a), 2 * math.cos(a) + math.sin(a)])
    e = np.zeros((1, 1, 12))
    e[0, 0, 2], e[0, 0, 3] = 1.0, 2.0
    assert np.allclose(plain.rotate(e, [3], 8, 10000.0, interleaved=True)[0, 0, [2, 3]], [math.cos(a) - 2 * math.sin(a), 2 * math.cos(a) + math.sin(a)])


def test_frequency_blend():
    f, one = plain.rotary_frequencies(16, 100.0, None)
    assert one == 1.0 and np.allclose(f, 100.0 ** (-np.arange(8) / 8))
    sc = {"factor": 4.0, "original": 64, "fast": 2.0, "slow": 0.5}
    g, magnitude = plain.rotary_frequencies(16, 100.0, sc)
    assert np.isclose(magnitude, 0.1 * math.log(4.0) + 1.0)
    turns = 64 * f / (2 * math.pi)
    assert np.allclose(g[turns > 3.5], f[turns > 3.5]) and np.allclose(g[turns < 0.3], f[turns < 0.3] / 4.0)
    assert np.all(g <= f) and np.all(g >= f / 4.0) and np.any((g < f * 0.999) & (g > f / 4.0 * 1.001))
    x = np.ones((1, 1, 16))
    assert np.isclose(np.linalg.norm(plain.rotate(x, [5], 16, 100.0, sc)), 4.0 * magnitude)
    # a ramp without width is a step
    g, _ = plain.rotary_frequencies(16, 100.0, {"factor": 2.0, "original": 64, "fast": 1.0, "slow": 0.99999})
    assert set(np.round(g / f, 6)) <= {0.5, 1.0}


def test_attention_is_causal_groups_heads_and_takes_a_sink():
    rng = np.random.default_rng(2)
    T, H, G, D, V = 7, 4, 2, 5, 3
    q, k, v = rng.normal(size=(T, H, D)), rng.normal(size=(T, G, D)), rng.normal(size=(T, G, V))
    o = plain.causal_attention(q, k, v, 0.3)
    assert np.allclose(o[0, 0], v[0, 0]) and np.allclose(o[0, 3], v[0, 1])
    s = q[5, 2] @ k[:6, 1].T * 0.3
    p = np.exp(s)
    assert np.allclose(o[5, 2], (p / p.sum()) @ v[:6, 1])
    k2, v2 = k.copy(), v.copy()
    k2[6], v2[6] = 9.0, -9.0
    assert np.allclose(plain.causal_attention(q, k2, v2, 0.3)[:6], o[:6])
    sink = np.array([0.0, 2.0, -1.0, 60.0])
    w = plain.causal_attention(q, k, v, 0.3, sink)
    assert np.allclose(w[5, 2], (p / (p.sum() + math.exp(-1.0))) @ v[:6, 1])
    assert np.abs(w[:, 3]).max() < 1e-20 and np.allclose(plain.causal_attention(q, k, v, 0.3, np.full(4, -1e9)), o)


def test_attention_norms_whole_projections_and_gates_every_value():
    rng = np.random.default_rng(3)
    T, E, H, G, D, V = 4, 6, 2, 1, 4, 3
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": 0.5, "rot": {"base": 100.0, "dims": 0}}
    w = {"q": rng.normal(size=(H * D, E)), "k": rng.normal(size=(G * D, E)), "v": rng.normal(size=(G * V, E)), "g": rng.normal(size=(H * V, E)),
         "o": np.eye(H * V), "q.norm": rng.normal(size=H * D), "k.norm": np.zeros(G * D)}
    w = {"p." + n: x for n, x in w.items()}
    h = rng.normal(size=(T, E))
    out = plain.attention_mixer(h, w, "p.", m, 0.1, np.arange(T))
    # keys of zeros: every row is the running mean of the values, times its own gates
    mean = np.cumsum(h @ w["p.v"].T, axis=0) / np.arange(1, T + 1)[:, None]
    assert np.allclose(out, np.tile(mean, (1, H)) * plain.sigmoid(h @ w["p.g"].T))
    # the norm takes all heads together: scaling one head's rows of W_q changes the other head's scores
    w["p.k.norm"] = np.ones(G * D)
    a = plain.attention_mixer(h, w, "p.", m, 0.1, np.arange(T))
    w["p.q"] = np.concatenate([w["p.q"][:D] * 10.0, w["p.q"][D:]])
    assert not np.allclose(plain.attention_mixer(h, w, "p.", m, 0.1, np.arange(T))[:, V:], a[:, V:])


def test_latent_attention_scores_over_expanded_keys_equal_scores_over_latents():
    rng = np.random.default_rng(4)
    T, E, H, D, R, V, C = 6, 8, 3, 4, 2, 5, 7
    m = {"heads": H, "dim": D, "rot_dim": R, "vdim": V, "kv_rank": C, "scale": 0.4, "rot": {"base": 50.0, "dims": R}}
    w = {"p.q": rng.normal(size=(H * (D + R), E)), "p.dkv": rng.normal(size=(C + R, E)), "p.dkv.norm": rng.normal(size=C),
         "p.uk": rng.normal(size=(H * D, C)), "p.uv": rng.normal(size=(H * V, C)), "p.sink": rng.normal(size=H), "p.o": np.eye(H * V)}
    h = rng.normal(size=(T, E))
    out = plain.latent_attention_mixer(h, w, "p.", m, 1e-3, np.arange(T))
    down = h @ w["p.dkv"].T
    c = plain.rms_unit(down[:, :C], 1e-3) * w["p.dkv.norm"]
    kr = plain.rotate(down[:, None, C:], np.arange(T), R, 50.0, interleaved=True)[:, 0]
    q = (h @ w["p.q"].T).reshape(T, H, D + R)
    qr = plain.rotate(q[..., D:], np.arange(T), R, 50.0, interleaved=True)
    for n in range(H):
        ql = q[:, n, :D] @ w["p.uk"][n * D:(n + 1) * D]
        s = (ql @ c.T + qr[:, n] @ kr.T) * 0.4
        p = np.tril(np.exp(s))
        mixed = (p / (p.sum(1, keepdims=True) + math.exp(w["p.sink"][n]))) @ c
        assert np.allclose(out[:, n * V:(n + 1) * V], mixed @ w["p.uv"][n * V:(n + 1) * V].T)


def test_delta_rule():
    rng = np.random.default_rng(5)
    T, H, D, V = 6, 2, 4, 3
    k, v = plain.unit(rng.normal(size=(T, H, D))), rng.normal(size=(T, H, V))
    # beta 1, no decay: reading with the key just written gives the value just written
    o, S = plain.delta_scan(k, k, v, np.ones((T, H)), np.ones((T, H)))
    assert np.allclose(o, v, atol=1e-5)
    # a key written twice is overwritten, not summed; an orthogonal one is left alone
    e = np.zeros((3, 1, D))
    e[0, 0, 0] = e[2, 0, 0] = e[1, 0, 1] = 1.0
    o, S = plain.delta_scan(e, e, v[:3, :1], np.ones((3, 1)), np.ones((3, 1)))
    assert np.allclose(S[0, 0], v[2, 0]) and np.allclose(S[0, 1], v[1, 0])
    # the decay acts before the correction and the read-out sees the write
    g, b = np.array([[0.5]]), np.array([[0.25]])
    o, S = plain.delta_scan(e[:1], e[:1], v[:1, :1], g, b)
    o2, S2 = plain.delta_scan(e[[0, 0]], e[[0, 0]], v[[0, 0], :1], np.array([[0.5], [0.5]]), np.array([[0.25], [0.25]]))
    assert np.allclose(o[0, 0], 0.25 * v[0, 0]) and np.allclose(o2[1, 0], (0.125 + 0.25 * (1 - 0.125)) * v[0, 0])
    x, taps = rng.normal(size=(5, 2)), rng.normal(size=(2, 3))
    y = plain.short_conv_silu(x, taps)
    assert np.allclose(y[0], plain.silu(taps[:, 2] * x[0])) and np.allclose(y[4], plain.silu(taps[:, 0] * x[2] + taps[:, 1] * x[3] + taps[:, 2] * x[4]))
    assert np.allclose(plain.unit(np.array([3.0, 4.0])), [0.6, 0.8], atol=1e-6) and np.allclose(plain.unit(np.zeros(3)), 0.0)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_run_order_configuration_and_tensors(name):
    """The configuration survives its own JSON; the assembly lists the folder's tensors, gives every pass caches of its own and
    opens each pass with the one product."""
    from llmx_amd.models import assemble, read_config
    config = CONFIGS[name]
    cfg = read_config(copy.deepcopy(config))
    assert type(cfg).from_json(cfg.to_json()) == cfg
    spec = assemble(cfg)
    order = plain.run_order(config)
    assert [(e.layer, e.before == 0) for e in spec.run_order] == order and [e.cache for e in spec.run_order] == list(range(len(order)))
    assert [i for i, _ in order] == [i for i, _ in cfg.passes()] and len(spec.inputs) == (1 if config.get("loop") else 0)
    if config.get("loop"):
        a, b, n = (config["loop"][k] for k in ("start", "stop", "times"))
        assert len(order) == len(config["layers"]) + (b - a) * (n - 1) and sum(opens for _, opens in order) == n
    _, tensors = load_plain(model_folder(name))
    E = config["width"]
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        assert (f"l{i}.norm2" in tensors) == (layer["mlp"] is not None) == (f"l{i}.mlp.up.b" in tensors)
        if layer["type"] == "attention":
            assert tensors[p + "q.norm"].shape == (m["heads"] * m["dim"],) and tensors[p + "g"].shape == (m["heads"] * m["vdim"], E)
        elif layer["type"] == "latent_attention":
            assert tensors[p + "sink"].shape == (m["heads"],) and tensors[p + "dkv"].shape == (m["kv_rank"] + m["rot_dim"], E)
        else:
            assert tensors[p + "v.conv"].shape == (m["heads"] * m["vdim"], m["conv"]) and tensors[p + "dt_bias"].shape == (m["heads"],)
    assert "head" not in tensors and ("loop.in" in tensors) == bool(config.get("loop"))


def test_every_pass_reads_the_embedding_and_its_own_state():
    """The plain model: a pass more changes the logits, and what a pass adds depends on the embedding's half of the product."""
    config, tensors = load_plain(model_folder("A"))
    ids = [5, 9, 200, 31]
    base = plain.forward(config, tensors, ids)
    more = copy.deepcopy(config)
    more["loop"]["times"] += 1
    assert not np.allclose(plain.forward(more, tensors, ids), base)
    E = config["width"]
    cut = dict(tensors)
    cut["loop.in"] = tensors["loop.in"].copy()
    cut["loop.in"][:, E:] = 0.0
    assert not np.allclose(plain.forward(config, cut, ids), base)
    trace = []
    plain.forward(config, tensors, ids, trace)
    assert len(trace) == len(plain.run_order(config))


def _broken(config, path, value):
    out = copy.deepcopy(config)
    at = out
    for p in path[:-1]:
        at = at[p]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return out


@pytest.mark.parametrize("path,value,names", [
    (("width",), None, "width"), (("layers",), [], "layers"), (("layers", 0, "type"), "mamba", "layers[0].type"),
    (("layers", 0, "mixer", "kv_heads"), 3, "kv_heads"), (("layers", 0, "mixer", "rot", "dims"), 34, "rot.dims"),
    (("layers", 0, "mixer", "rot", "scaling", "kind"), "yarn", "kind"), (("layers", 0, "mixer", "window"), 5, "window"),
    (("layers", 3, "mixer", "rot", "dims"), 8, "dims"), (("layers", 3, "mixer", "rot_dim"), 15, "dims"),
    (("layers", 3, "mixer", "rot", "scaling"), {"factor": 2.0}, "scaling"), (("layers", 2, "mixer", "conv"), 0, "conv"), (("layers", 2, "mixer", "dim"), 300, "dim"), (("layers", 0, "mlp", "kind"), "moe", "kind"),
    (("loop", "stop"), 9, "loop"), (("loop", "times"), 0, "times"), (("logit_softcap",), -1.0, "logit_softcap"), (("embedding", "rows"), 1, "rows"),
    (("norm", "eps"), "x", "eps"), (("experts",), 4, "experts")], ids=lambda x: str(x) if not isinstance(x, (tuple, list)) else "-".join(map(str, x)))
def test_configurations_that_are_refused(path, value, names):
    from llmx_amd import ConfigError
    from llmx_amd.models import read_config
    with pytest.raises(ConfigError, match=names.replace("[", r"\[").replace("]", r"\]")):
        read_config(_broken(CONFIG_A, path, value))


def test_optional_keys():
    from llmx_amd.models import read_config
    bare = copy.deepcopy(CONFIG_D)
    del bare["embedding"], bare["logit_softcap"]
    cfg = read_config(bare)
    null = copy.deepcopy(CONFIG_A)
    null["layers"][3]["mixer"]["rot"]["scaling"] = None
    assert read_config(null) == read_config(copy.deepcopy(CONFIG_A))
    assert cfg.embedding_scale == 1.0 and cfg.logit_softcap is None and cfg.loop is None
    assert read_config(dict(CONFIG_C, name="x", seed=3)).vocab_size == CONFIG_C["vocab"]
