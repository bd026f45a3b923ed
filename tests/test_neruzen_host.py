"""Neruzen on the CPU: pins of the plain implementation (tests/plain_neruzen.py), the configuration reader's round trip and
refusals, the assembly's tensor list and cache needs, and the work plan of windowed latent attention."""

from __future__ import annotations

import copy
import math

import numpy as np
import pytest

import plain_neruzen as plain
from neruzen_cases import CONFIG_A, CONFIG_B, CONFIG_C, CONFIGS


# ---------------------------------------------------------------------------- the plain implementation's pins
def test_bigram_rows_and_the_first_token():
    cfg = {"buckets": 10, "mul_prev": 7, "mul_cur": 3}
    assert plain.bigram_rows([4, 9, 9], cfg) == [10, (4 * 7 + 9 * 3) % 10, (9 * 7 + 9 * 3) % 10]
    W = {"embed": np.arange(12.0).reshape(6, 2), "bigram": 100.0 * np.arange(8.0)[:, None] * np.ones((1, 2))}
    x = plain.embed([5, 1], W, {"embedding": {"bigram": {"buckets": 7, "mul_prev": 2, "mul_cur": 1}}})
    assert np.allclose(x, [[10.0 + 700.0, 11.0 + 700.0], [2.0 + 100.0 * (11 % 7), 3.0 + 100.0 * (11 % 7)]])


def test_token_shift_mixes_with_the_row_before():
    h = np.array([[1.0, 2.0], [3.0, 5.0], [0.0, 0.0]])
    s = np.array([0.25, 1.0])
    assert np.allclose(plain.token_shift(h, s), [[0.75, 0.0], [2.5, 2.0], [0.75, 5.0]])


def test_the_window_says_who_sees_whom():
    m = plain.window_mask(6, 3)
    assert m[5].tolist() == [False, False, False, True, True, True] and m[1].tolist() == [True, True] + [False] * 4
    assert plain.window_mask(4, 1).tolist() == np.eye(4, dtype=bool).tolist()


def test_rotation_pairs_halves_and_keeps_relative_positions():
    x = np.random.default_rng(1).normal(size=(6, 2, 8))
    r = plain.rotate_halves(x, np.arange(6), {"base": 100.0, "dims": 4})
    assert np.allclose(r[..., 4:], x[..., 4:]) and np.allclose(r[0], x[0])
    assert np.allclose(np.hypot(r[..., 0], r[..., 2]), np.hypot(x[..., 0], x[..., 2]))     # dims 0 and 2 are a pair
    assert np.allclose(r[3, 0, 0], x[3, 0, 0] * math.cos(3.0) - x[3, 0, 2] * math.sin(3.0))
    a = plain.rotate_halves(np.tile(x[:1], (6, 1, 1)), np.arange(6), {"base": 100.0, "dims": 8})
    assert np.isclose(a[1, 0] @ a[3, 0], a[2, 0] @ a[4, 0])
    assert plain.rotate_halves(x, np.arange(6), {"base": 100.0, "dims": 0}) is x


def test_decayed_outer_products_against_the_sums_written_out_and_across_a_cut():
    rng = np.random.default_rng(2)
    T, H, D, V = 9, 2, 5, 3
    q, k, v = rng.normal(size=(T, H, D)), rng.normal(size=(T, H, D)), rng.normal(size=(T, H, V))
    g = [0.9, 0.5]
    o, S = plain.decayed_outer_products(q, k, v, g)
    for t in (0, 4, 8):
        for h in range(H):
            want = sum(g[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert np.allclose(o[t, h], want)
    o1, S1 = plain.decayed_outer_products(q[:4], k[:4], v[:4], g)
    o2, S2 = plain.decayed_outer_products(q[4:], k[4:], v[4:], g, S1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(S2, S)


def test_latent_attention_is_softmax_over_expanded_keys_of_the_window():
    rng = np.random.default_rng(3)
    E, T = 12, 7
    cfg = {"heads": 2, "dim": 3, "rot_dim": 4, "vdim": 5, "q_rank": 6, "kv_rank": 4, "scale": 0.7, "mask": {"size": 3}, "rot": {"base": 50.0, "dims": 4}}
    W = {"a." + n: rng.normal(size=s) for n, s in (("dq", (6, E)), ("uq", (14, 6)), ("dkv", (8, E)), ("uk", (6, 4)), ("uv", (10, 4)))}
    W.update({"a.dq.norm": rng.uniform(0.5, 1.5, 6), "a.dkv.norm": rng.uniform(0.5, 1.5, 4), "a.o": np.eye(10)})
    h = rng.normal(size=(T, E))
    y = plain.latent_attention(h, W, "a.", cfg, 1e-6).reshape(T, 2, 5)
    c = plain.rms_norm((h @ W["a.dkv"].T)[:, :4], W["a.dkv.norm"], 1e-6)
    v = (c @ W["a.uv"].T).reshape(T, 2, 5)
    assert np.allclose(y[0], v[0])                                                  # one key: its value
    lo, hi = v[4:7].min(0), v[4:7].max(0)
    assert np.all(y[6] >= lo - 1e-12) and np.all(y[6] <= hi + 1e-12)                # a mixture of the window's three values
    # a key before the window changes nothing, one inside does
    h2, h3 = h.copy(), h.copy()
    h2[3] += 1.0
    h3[4] += 1.0
    assert np.allclose(plain.latent_attention(h2, W, "a.", cfg, 1e-6).reshape(T, 2, 5)[6], y[6])
    assert not np.allclose(plain.latent_attention(h3, W, "a.", cfg, 1e-6).reshape(T, 2, 5)[6], y[6])


def test_routing_by_groups():
    E = 6
    W = {"r.router": np.eye(6)}
    cfg = {"router": {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}}
    h = np.array([[0.0, 3.0, 2.9, 2.8, -1.0, 0.0], [1.0, 1.0, 0.0, 0.0, 0.5, 1.0]])
    ids, w, z = plain.route(h, W, "r.", cfg)
    # the best expert decides the group (0, 1), whose other member is picked though (2, 3) hold better ones
    assert ids.tolist() == [[1, 0], [0, 1]] and np.allclose(w.sum(-1), 1.0)
    assert np.isclose(w[0, 0] / w[0, 1], math.exp(3.0))
    cfg["router"]["groups"]["keep"] = 2
    assert plain.route(h, W, "r.", cfg)[0].tolist() == [[1, 2], [0, 1]]
    cfg["router"]["groups"] = {"count": 1, "keep": 1}
    assert plain.route(h, W, "r.", cfg)[0].tolist() == [[1, 2], [0, 1]]
    one = {"router": {"experts": 6, "top": 1, "groups": {"count": 6, "keep": 1}}}
    assert np.allclose(plain.route(h, W, "r.", one)[1], 1.0)            # a single pick weighs 1


def test_a_layer_is_one_norm_a_shift_for_the_mixer_and_a_sum():
    from neruzen_cases import plain as plain_of
    config, W = plain_of("A")
    x = np.random.default_rng(5).normal(size=(6, config["width"]))
    i, eps = 3, config["norm"]["eps"]
    entry = config["layers"][i]
    h = plain.rms_norm(x, W[f"l{i}.norm1"], eps)
    want = x + plain.lightning(plain.token_shift(h, W[f"l{i}.shift"]), W, f"l{i}.mix.", entry["mixer"], eps) + plain.experts(h, W, f"l{i}.mlp.", entry["mlp"])
    assert np.allclose(plain.layer(x, W, i, config), want)


# ---------------------------------------------------------------------------- configuration and assembly
def test_configuration_round_trip_and_refusals():
    from llmx_amd.config import ConfigError
    from llmx_amd.models import read_config
    for name, config in CONFIGS.items():
        cfg = read_config(copy.deepcopy(config))
        assert read_config(cfg.to_json()) == cfg and cfg.vocab_size == config["vocab"], name
    bare = copy.deepcopy(CONFIG_B)
    del bare["layers"][0]["mlp"]["router"]["groups"]
    m = read_config(bare).layers[0].mlp
    assert (m.group_count, m.group_keep) == (1, 1) and read_config(copy.deepcopy(CONFIG_B)).layers[1].mlp.shared_ff is None

    def refused(edit, text):
        c = copy.deepcopy(CONFIG_A)
        edit(c)
        with pytest.raises(ConfigError, match=text):
            read_config(c)

    refused(lambda c: c["layers"][0]["mixer"].pop("q_rank"), r"missing key layers\[0\]\.mixer\.q_rank")
    refused(lambda c: c["layers"][0]["mixer"].pop("mask"), r"layers\[0\]\.mixer\.mask")
    refused(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), r"layers\[0\]\.mixer\.mask\.size")
    refused(lambda c: c["layers"][0]["mixer"].update(gate=1), r"layers\[0\]\.mixer\.gate is not one this engine reads")
    refused(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), r"layers\[0\]\.mixer\.rot\.dims")
    refused(lambda c: c["layers"][1].update(type="retention_2"), r"layers\[1\]\.type")
    refused(lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), r"layers\[1\]\.mixer\.decay")
    refused(lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5]), r"layers\[1\]\.mixer\.decay")
    refused(lambda c: c["layers"][1]["mixer"].update(dim=300), r"layers\[1\]\.mixer\.dim")
    refused(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), r"layers\[0\]\.mlp\.router\.groups\.count")
    refused(lambda c: c["layers"][3]["mlp"]["router"]["groups"].update(keep=1), r"layers\[3\]\.mlp\.router\.groups\.keep")
    refused(lambda c: c["layers"][0]["mlp"]["router"].update(top=9), r"layers\[0\]\.mlp\.router\.top")
    refused(lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), r"layers\[0\]\.mlp\.shared\.ff")
    refused(lambda c: c["layers"][0]["mlp"].update(kind="dense"), r"layers\[0\]\.mlp\.kind")
    refused(lambda c: c["embedding"]["bigram"].pop("mul_cur"), r"missing key embedding\.bigram\.mul_cur")
    refused(lambda c: c["embedding"]["bigram"].update(buckets=0), r"embedding\.bigram\.buckets")
    refused(lambda c: c.update(residual_mult=2.0), "key residual_mult is not one this engine reads")


def test_assembly_lists_the_designs_tensors_and_cache_needs():
    import torch
    from llmx_amd.engine.model import BuiltModel
    from llmx_amd.models import read_config, registry
    from llmx_amd.parts.base import BuildContext
    from llmx_amd.parts.spec import CompositeNeed, PagedNeed, StateNeed
    model = BuiltModel(registry.assemble(read_config(copy.deepcopy(CONFIG_A))), BuildContext(torch.float32, torch.device("cpu"), 64, 16))
    names = {s.name: tuple(s.shape) for s in model.tensor_specs()}
    assert names["embed"] == (320, 128) and names["bigram"] == (212, 128) and names["head"] == (320, 128)
    assert names["l0.mix.dq"] == (48, 128) and names["l0.mix.dq.norm"] == (48,) and names["l0.mix.uq"] == (4 * 32, 48)
    assert names["l0.mix.dkv"] == (56, 128) and names["l0.mix.uk"] == (96, 48) and names["l0.mix.uv"] == (160, 48) and names["l0.mix.o"] == (128, 160)
    assert "l0.mix.q" not in names and "l0.mix.g" not in names and names["l0.shift"] == (128,) and "l0.norm2" not in names
    assert names["l1.mix.g"] == (72, 128) and "l1.mix.norm" not in names and names["l3.mix.norm"] == (32,)
    assert names["l0.mlp.e5.gate"] == (32, 128) and names["l0.mlp.shared.down"] == (128, 48) and names["l0.mlp.router"] == (6, 128)
    assert not any(n.startswith("l1.mlp") for n in names) and "l2.mlp.shared.gate" not in names
    needs = model.cache_needs()
    assert all(isinstance(n, CompositeNeed) and n.members[1] == StateNeed((128,)) for n in needs)
    assert [getattr(n.members[0], "window", None) for n in needs] == [40, None, 101, None]
    assert isinstance(needs[0].members[0], PagedNeed) and needs[0].members[0].tensors[0].shape == (56,)
    assert needs[1].members[0] == StateNeed((3 * 3 * 16 * 8,)) and model.embedding.cache_need() == StateNeed((1,), "int32")


def test_decayed_attention_refuses_what_it_does_not_compute():
    import torch
    from llmx_amd.parts.base import BuildContext, build_part
    from llmx_amd.parts.spec import PartSpec
    ctx = BuildContext(torch.float32, torch.device("cpu"), 64, 16)
    base = {"hidden": 8, "heads": 2, "dim": 4, "vdim": 4, "decay": [0.5, 0.5], "eps": 1e-6}
    build_part("mixer", PartSpec("decayed_linear_attention", base, "m."), ctx)
    for bad in ({"decay": [0.5]}, {"operands": "relu"}, {"norm": "none"}, {"gate": "tanh"}, {"dim": 300},
                {"operands": "rotated", "position": PartSpec("rotary_scaled", {"dims": 4, "base": 10.0, "pairing": "interleaved"})}):
        with pytest.raises(ValueError, match="decayed linear attention"):
            build_part("mixer", PartSpec("decayed_linear_attention", dict(base, **bad), "m."), ctx)
    with pytest.raises(ValueError, match="equal groups"):
        build_part("feed_forward", PartSpec("routed_experts", {"hidden": 8, "experts": 6, "top_k": 3, "intermediate": 4, "groups": {"count": 3, "keep": 1}}, "f."), ctx)


# ---------------------------------------------------------------------------- work plans
def test_the_plan_of_a_windowed_decode_step_stays_the_same_while_the_row_moves_on():
    from llmx_amd import ops
    window, split = 150, ops.LATENT_SPLIT_WINDOW_KEYS
    most = (window + split - 2) // split + 1
    plans = {id(ops.latent_plan([1, 1], 4, "cpu", contexts=[c, 40], window=window)) for c in range(400, 700)}
    assert len(plans) == 1
    plan = ops.latent_plan([1, 1], 4, "cpu", contexts=[450, 40], window=window)
    assert plan.n_slots == most and plan.n_merges == 1 and plan.window == window
    for c in range(1, 700):           # as many blocks as the row's keys can touch
        lo, hi = max(0, c - window), c - 1
        got = ops.latent_plan([1], 4, "cpu", contexts=[c], window=window)
        assert hi // split - lo // split + 1 <= max(1, got.n_slots or 1) <= most
