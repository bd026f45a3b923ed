"""Vivulorn in the engine against the plain implementation (tests/plain_vivulorn.py), mechanism by mechanism and whole.

Kernels alone: layer norms with a bias, products with a bias and the exact gelu in every form, attention's preparation with values of a
width of their own, attention with a gate a value and latent attention with a sink over shuffled pages, with one query made to fit a
single key at the pages' and segments' edges, the product that opens a pass, the delta rule row by row, step by step and chunk by
chunk.  Then the engine under every way of cutting the same tokens into steps: in float32 against the plain implementation within
F32_TOL (and bit for bit among cuttings whose portions are too short for the chunked recurrence), in bfloat16 within BF16_TOL; pages and
request seats that are used again; long decoding; greedy generation through `generate`; the trace replay tool and the command line.
"""

from __future__ import annotations

import copy
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_vivulorn as plain
from vivulorn_cases import CONFIGS, PAGES, greedy, load_plain, model_folder, plain_logits, portions, tokens_for, write_folder

pytestmark = pytest.mark.gpu

F32_TOL = 1e-5      # |engine - plain| over all logits relative to the largest |logit|: float32 sums in another order
CUT_TOL = 1e-5      # two cuttings of the same tokens where one runs the recurrence by chunks, float32
# the serving path against the plain implementation (float64, nothing rounded): the largest difference and the root mean square of
# all, relative to the logits'.  Met: A 2.6e-2 and 9.2e-3, B 4.0e-3 and 4.1e-3, C 5.4e-3 and 4.9e-3, D 3.0e-2 and 7.3e-3
BF16_TOL = {"A": 4e-2, "B": 8e-3, "C": 1e-2, "D": 4.5e-2}
BF16_RMS = {"A": 1.3e-2, "B": 6e-3, "C": 7.5e-3, "D": 1.1e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [torch.float32, torch.bfloat16]
DTYPE_IDS = ["float32", "bfloat16"]


def ops():
    from llmx_amd import ops as o
    return o


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a)).to(device="cuda", dtype=dtype).contiguous()


def f64(t):
    return t.double().cpu().numpy()


def close(got, want, tol, what=""):
    got, want = (torch.as_tensor(np.asarray(t.cpu() if isinstance(t, torch.Tensor) else t)).double() for t in (got, want))
    err = float((got - want).abs().max()) / max(float(want.abs().max()), 1e-30)
    assert err <= tol, f"{what}: relative error {err:.3e} above {tol:.1e}"
    return err


# ---------------------------------------------------------------------------
# kernels alone: norms, products, the pass's product
@pytest.mark.parametrize("width", [1, 54, 97, 1500, 2048, 3001, 4096, 5000, 9001])
def test_layer_norm_with_a_bias(width):
    """Rows kept in registers, read again, and of lengths that are no multiple of four; picked rows; both outputs."""
    o = ops()
    rng = np.random.default_rng(width)
    x, w, b = dev(rng.normal(size=(7, width)) * 3 + 5), dev(rng.normal(size=width)), dev(rng.normal(size=width))
    pick = dev([6, 0, 3], torch.int32)
    want = plain.layer_norm(f64(x), f64(w), f64(b), 1e-3)
    for rows, picked in ((want, None), (want[[6, 0, 3]], pick)):
        out, out32 = (torch.full((rows.shape[0], width), 9.0, device="cuda", dtype=d) for d in (torch.bfloat16, torch.float32))
        o.layernorm(x, w, 1e-3, out, out32, picked, bias=b)
        close(out32, rows, 3e-6, "float32")
        assert torch.equal(out, out32.bfloat16())
        alone = torch.empty_like(out32)
        o.layernorm(x, w, 1e-3, alone, None, picked, bias=b)
        assert torch.equal(alone, out32)
    plain_form, zero = torch.empty(7, width, device="cuda"), torch.empty(7, width, device="cuda")
    o.layernorm(x, w, 1e-3, plain_form)
    o.layernorm(x, w, 1e-3, zero, bias=torch.zeros_like(b))
    close(plain_form, f64(zero), 3e-6, "no bias is a bias of zeros")


# (rows, features, inner): the forms of the product kernels (weight streaming with one and more tiles of rows and two strips, tiles, runs
# apart, wide tiles, bounded tiles, universal)
PRODUCTS = [(1, 48, 96), (3, 2000, 1024), (20, 64, 128), (33, 6200, 64), (40, 256, 2048), (64, 512, 768), (200, 130, 72), (300, 512, 256),
            (1100, 6144, 128), (5, 21, 54), (70, 33, 30)]


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("shape", PRODUCTS, ids=lambda s: "x".join(map(str, s)))
def test_products_with_a_bias_and_the_exact_gelu(dtype, shape):
    o = ops()
    M, N, K = shape
    rng = np.random.default_rng(M + N)
    a, w, b = dev(rng.normal(size=(M, K)), dtype), dev(rng.normal(size=(N, K)) / K ** 0.5, dtype), dev(rng.normal(size=N))
    scratch = lambda name, s, d: torch.empty(s, dtype=d, device="cuda")
    z = f64(a) @ f64(w).T + f64(b)
    for out_type in (torch.float32, dtype):
        tol = 5e-6 if out_type == torch.float32 else 5e-3
        c = torch.full((M, N), 9.0, device="cuda", dtype=out_type)
        o.gemm(a, w, c, scratch=scratch, act=(o.ACT_GELU_BIAS, b))
        close(c.float(), plain.gelu(z), tol, "gelu of a biased product")
        o.gemm(a, w, c, scratch=scratch, act=(o.ACT_BIAS, b))
        close(c.float(), z, tol, "a biased product")
    old = dev(rng.normal(size=(M, N)))
    c = old.clone()
    o.gemm(a, w, c, o.EPI_ADD, scratch=scratch, act=(o.ACT_BIAS, b))
    close(c, f64(old) + z, 5e-6, "a biased product that is added")
    first = torch.empty(1, N, device="cuda")            # a row's bits do not depend on the others
    rows = torch.empty(M, N, device="cuda")
    o.gemm(a, w, rows, scratch=scratch, act=(o.ACT_GELU_BIAS, b))
    o.gemm(a[:1].contiguous(), w, first, scratch=scratch, act=(o.ACT_GELU_BIAS, b))
    if dtype == torch.bfloat16 or M <= 64:
        assert torch.equal(first[0], rows[0])
    with pytest.raises(o.KernelError):
        o.gemm(a, w, c, o.EPI_ADD, act=(o.ACT_GELU_BIAS, b))
    with pytest.raises(o.KernelError):
        o.gemm(a, w, c, act=(o.ACT_BIAS, b[:-1].contiguous()))


@pytest.mark.parametrize("width", [72, 1000, 2048, 4096])
def test_products_that_form_their_layer_norm_themselves(width):
    """A step of very few rows: the product handed the residual and the norm gives the bits of the norm kernel and the product."""
    o = ops()
    rng = np.random.default_rng(width)
    nw, nb = dev(rng.normal(size=width)), dev(rng.normal(size=width))
    for rows in (1, 2, 4):
        x = dev(rng.normal(size=(rows, width)) * 3 + 1)
        h = torch.empty(rows, width, device="cuda", dtype=torch.bfloat16)
        o.layernorm(x, nw, 1e-3, h, bias=nb)
        for n in (16, 130, 4096):
            w, b = dev(rng.normal(size=(n, width)), torch.bfloat16), dev(rng.normal(size=n))
            assert o.gemm_can_norm_rows(rows, w, torch.float32)
            for out_type, act in ((torch.float32, None), (torch.bfloat16, (o.ACT_GELU_BIAS, b))):
                apart, together = (torch.empty(rows, n, device="cuda", dtype=out_type) for _ in range(2))
                o.gemm(h, w, apart, act=act)
                o.gemm(o.NormedRows(x, nw, 1e-3, nb), w, together, act=act)
                assert torch.equal(apart, together), f"{rows} rows, {n} features"
    with pytest.raises(o.KernelError):
        o.NormedRows(dev(np.zeros((1, 6002))), dev(np.zeros(6002)), 1e-3, dev(np.zeros(6002)))
    with pytest.raises(o.KernelError):
        o.gemm_f32(o.NormedRows(x, nw, 1e-3, nb), dev(np.zeros((8, width))), torch.empty(4, 8, device="cuda"))


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("width", [54, 96, 2048])
def test_joined_rows(dtype, width):
    o = ops()
    rng = np.random.default_rng(width)
    x, x0, y = (dev(rng.normal(size=(11, width))) for _ in range(3))
    out = torch.full((11, 2 * width), 9.0, device="cuda", dtype=dtype)
    o.join_rows(x, x0, out)
    assert torch.equal(out, torch.cat([x, x0], 1).to(dtype))
    o.join_rows(y, None, out)                           # a later pass: the second half stays
    assert torch.equal(out, torch.cat([y, x0], 1).to(dtype))


# ---------------------------------------------------------------------------
# kernels alone: attention
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("rows", [5, 300])
@pytest.mark.parametrize("sizes", [(4, 2, 32, 48, 16), (3, 1, 10, 6, 6), (2, 2, 16, 16, 16), (5, 5, 12, 20, 0)], ids=lambda s: "x".join(map(str, s)))
def test_norms_of_whole_projections_rotation_and_cache_rows(dtype, rows, sizes):
    H, G, D, V, dims = sizes
    o = ops()
    from llmx_amd.parts.position import scaled_table
    rng = np.random.default_rng(D + rows)
    page, past, eps = 8, 13, 1e-2
    n_pages = -(-(past + rows) // page)
    order = list(range(n_pages + 2))
    random.Random(1).shuffle(order)
    scaling = {"factor": 4.0, "original": 32, "fast": 4.0, "slow": 0.5}
    width = H * D + G * D + G * V + H * V + 3
    pre, wq, wk = dev(rng.normal(size=(rows, width))), dev(rng.uniform(0.5, 1.5, H * D)), dev(rng.uniform(0.5, 1.5, G * D))
    cos_sin = dev(scaled_table(past + rows, dims, 300.0, scaling, True))
    kc, vc = torch.zeros(n_pages + 2, G, page, D, device="cuda", dtype=dtype), torch.zeros(n_pages + 2, G, V, page, device="cuda", dtype=dtype)
    q = torch.empty(rows, H * D, device="cuda", dtype=dtype)
    pos, entry = dev(np.arange(past, past + rows), torch.int32), dev(np.zeros(rows), torch.int32)
    o.qknorm_rope_kvwrite(pre, wq, wk, cos_sin, pos, entry, dev([order], torch.int32), q, kc, vc, eps, H, G, D, dims, o.QKNORM_PROJECTION)
    p = f64(pre)
    at = np.arange(past, past + rows)
    turn = lambda x: plain.rotate(x, at, dims, 300.0, scaling)
    tol = 3e-6 if dtype == torch.float32 else 5e-3
    close(q.float(), turn((plain.rms_unit(p[:, :H * D], eps) * f64(wq)).reshape(rows, H, D)).reshape(rows, -1), tol, "queries")
    keys = torch.stack([kc[order[t // page], :, t % page] for t in at]).float()
    values = torch.stack([vc[order[t // page], :, :, t % page] for t in at]).float()
    k0 = H * D
    close(keys, turn((plain.rms_unit(p[:, k0:k0 + G * D], eps) * f64(wk)).reshape(rows, G, D)), tol, "keys")
    close(values, p[:, k0 + G * D:k0 + G * D + G * V].reshape(rows, G, V), tol, "values")


def _paged(rng, length, page):
    order = list(range(-(-length // page) + 3))
    random.Random(length).shuffle(order)
    return order, torch.tensor([order[p // page] * page + p % page for p in range(length)], device="cuda")


def _attention_case(dtype, H, G, D, V, page, length, runs, sharp=(), seed=0):
    """Attention with a gate a value over shuffled pages, beside an unrelated request; sharp: (row, key) pairs whose queries are made
    to fit that key alone.  runs: [(first row, end), ...].  Returns (got, plain, launches)."""
    o = ops()
    rng = np.random.default_rng(seed + 100 * H + D)
    q, k, v = rng.normal(size=(length, H, D)) * 0.4, rng.normal(size=(length, G, D)), rng.normal(size=(length, G, V))
    for row, key in sharp:
        q[row] = np.repeat(k[key], H // G, axis=0) * 4.0
    gate = dev(rng.normal(size=(length, H * V + 5)) * 2)
    order, at = _paged(rng, length, page)
    kc, vc = (torch.zeros(len(order) * page, G, w, device="cuda", dtype=dtype) for w in (D, V))
    qd, kd, vd = dev(q, dtype), dev(k, dtype), dev(v, dtype)
    kc[at], vc[at] = kd, vd
    kc = kc.view(len(order), page, G, D).transpose(1, 2).contiguous()
    vc = vc.view(len(order), page, G, V).permute(0, 2, 3, 1).contiguous()
    table = order[:-(-length // page)]
    tables = dev([[-1] * len(table), table], torch.int32)
    scale = 0.9 / D ** 0.5
    out, ran = torch.zeros(length, H * V), {}
    for a, b in runs:
        n = b - a
        pos, entry = dev(np.arange(a, b), torch.int32), dev(np.ones(n), torch.int32)
        got = torch.zeros(n, H * V, device="cuda", dtype=dtype)
        plan = rules = by_rules = None
        if dtype == torch.bfloat16 and V == D and o.attention_mfma_ok(dtype, D, page):
            plan = o.attention_plan([0, n], [0, b], H, G, "cuda")
        elif o.attention_rules_ok(dtype, D, V, page):
            rules, by_rules = o.ScoreRules(), o.rules_plan([0, n], [0, b], H, G, 1, "cuda", shared=o.attention_rules_shared_ok(D, V))
        o.take_launches()
        o.paged_attention(qd[a:b].reshape(n, -1).contiguous(), kc, vc, pos, entry, tables, got, scale, H, plan=plan, rules=rules, rules_plan=by_rules,
                          output_gate=gate[a:b, 2:2 + H * V])
        for name, times in o.take_launches().items():
            ran[name] = ran.get(name, 0) + times
        out[a:b] = got.float().cpu()
    want = plain.causal_attention(f64(qd), f64(kd), f64(vd), scale).reshape(length, -1) * plain.sigmoid(f64(gate)[:, 2:2 + H * V])
    return out, want, ran


ATT_TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}
ATT_CASES = [(4, 2, 32, 32, 16, 300), (6, 3, 128, 128, 16, 700), (2, 1, 64, 64, 48, 400), (4, 4, 48, 32, 16, 300), (8, 2, 64, 128, 16, 300), (3, 1, 10, 6, 4, 150),
             (1, 1, 16, 16, 16, 200), (20, 1, 32, 32, 16, 180)]


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("case", ATT_CASES, ids=lambda c: "x".join(map(str, c)))
def test_attention_with_a_gate_a_value(dtype, case):
    H, G, D, V, page, length = case
    # single keys: far away, at pages' and segments' borders, the row itself; the first rows
    rows = [length - 1, length - 2, length - 17, 1, 140]
    keys = [0, 1, page - 1, page, 127, 128, 129]
    sharp = [(r, min(k, r)) for r, k in zip(rows * 3, keys * 3)][:len(rows)] + [(length - 5, length - 5), (length - 6, length - 7), (131, 128), (133, 127)]
    whole, want, ran = _attention_case(dtype, *case, [(0, length)], sharp)
    close(whole, want, ATT_TOL[dtype], "a prompt")
    if dtype == torch.bfloat16:
        if D == V and D % 16 == 0:
            assert any(n.startswith("attention.tiles") for n in ran) and "attention.generic" not in ran and "attention.rules" not in ran
        elif D % 16 == 0:
            assert any(n.startswith("attention.rules") for n in ran) and "attention.generic" not in ran
    tail = length - 24
    decoded, _, ran = _attention_case(dtype, *case, [(0, tail)] + [(i, i + 1) for i in range(tail, length)], sharp)
    close(decoded, want, ATT_TOL[dtype], "a decoded tail")
    if dtype == torch.float32 or D % 16 == 0:
        assert torch.equal(decoded, whole)
    cuts = list(range(0, length - 2, 37)) + [length]
    pieces, _, _ = _attention_case(dtype, *case, list(zip(cuts, cuts[1:])), sharp)
    assert torch.equal(pieces, whole)


def test_every_key_of_a_sharp_row_counts_once():
    """One decoded row and one portion's row whose query fits each of some keys in turn: the key's value comes out."""
    for dtype in DTYPES:
        for D, V in ((64, 64), (32, 48), (10, 6)):
            page = 16 if D > 10 else 4
            for row, key in ((255, 0), (255, 127), (255, 128), (255, 254), (256, 255), (256, 256), (130, 129), (17, 16), (2, 1)):
                for runs in ([(row, row + 1)], [(max(0, row - 3), row + 2)]):
                    got, want, _ = _attention_case(dtype, 2, 1, D, V, page, row + 2, runs, [(row, key)], seed=row + key)
                    close(got[row], want[row], ATT_TOL[dtype], f"row {row}, key {key}, width {D}")


def _latent_case(dtype, H, C, R, page, length, runs, sink, sharp=(), row_major=True, tiles=True):
    """Attention over latents with a sink a head, as _attention_case."""
    o = ops()
    rng = np.random.default_rng(H * 1000 + C + length)
    c, r = rng.normal(size=(length, C)), rng.normal(size=(length, R))
    ql, qr = rng.normal(size=(length, H, C)) * 0.3, rng.normal(size=(length, H, R)) * 0.3
    for row, key in sharp:
        ql[row], qr[row] = c[key] * 4.0, r[key] * 4.0
    cores = o.latent_attention_mfma_ok(dtype, C, R, page, o.latent_cache_width(C, R))
    width = o.latent_cache_width(C, R) if cores else C + R
    order, at = _paged(rng, length, page)
    cache = torch.zeros(len(order), page, width, device="cuda", dtype=dtype)
    cd, rd, qld, qrd = dev(c, dtype), dev(r, dtype), dev(ql, dtype), dev(qr, dtype)
    cache.view(-1, width)[at, :C], cache.view(-1, width)[at, C:C + R] = cd, rd
    cache_t = cache[:, :, :C].transpose(1, 2).contiguous()
    table = order[:-(-length // page)]
    tables = dev([[-1] * len(table), table], torch.int32)
    scale, sink_d = 1.2 / (C + R) ** 0.5, dev(sink)
    out, ran = torch.zeros(length, H, C), {}
    for a, b in runs:
        n = b - a
        x, y = qld[a:b], qrd[a:b]
        if not row_major:
            x, y = x.transpose(0, 1), y.transpose(0, 1)
        x, y = x.contiguous(), y.contiguous()
        mixed = torch.zeros_like(x)
        plan = o.latent_plan([0, n], H, "cuda", contexts=[0, b], tiles=tiles) if cores else None
        o.take_launches()
        o.latent_attention(x, y, cache, dev(np.arange(a, b), torch.int32), dev(np.ones(n), torch.int32), tables, mixed, scale,
                           cache_t=cache_t if cores else None, plan=plan, row_major=row_major, sink=sink_d)
        for name, times in o.take_launches().items():
            ran[name] = ran.get(name, 0) + times
        out[a:b] = (mixed if row_major else mixed.transpose(0, 1)).float().cpu()
    q = np.concatenate([f64(qld), f64(qrd)], axis=-1)
    keys = np.concatenate([f64(cd), f64(rd)], axis=-1)[:, None]
    return out, plain.causal_attention(q, keys, f64(cd)[:, None], scale, f64(sink_d)), ran, cores


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("case", [(4, 48, 8, 16, 300), (3, 10, 6, 4, 150), (16, 128, 64, 16, 330), (18, 32, 32, 16, 200), (2, 64, 16, 48, 500), (5, 512, 64, 16, 400),
                                  (1, 16, 8, 16, 290), (6, 256, 64, 16, 200)], ids=lambda c: "x".join(map(str, c)))
def test_latent_attention_with_a_sink(dtype, case):
    H, C, R, page, length = case
    # sinks that hardly count, count like a key, outweigh every key, and one whose exponential alone would overflow
    sink = [(-30.0, 0.5, 3.0, 7.0, 1.0, 95.0)[h % 6] for h in range(H)]
    sharp = [(length - 1, 0), (length - 2, 63), (length - 18, 64), (length - 19, 127), (140, 128), (length - 3, length - 3), (1, 0), (64, 63)]
    whole, want, ran, cores = _latent_case(dtype, *case, [(0, length)], sink, sharp)
    close(whole, want, ATT_TOL[dtype], "a prompt")
    for h in range(H):          # every head by itself: a head that the sink empties shows nothing in the largest values
        big = float(np.abs(want[:, h]).max())
        if big > 1e-30:
            assert float((whole[:, h].double() - torch.as_tensor(want[:, h])).abs().max()) <= 2 * ATT_TOL[dtype] * big, f"head {h}"
        else:
            assert float(whole[:, h].abs().max()) < 1e-30
    assert ("latent_attention.tiles" in ran) == cores
    tail = length - 20
    decoded, _, ran, _ = _latent_case(dtype, *case, [(0, tail)] + [(i, i + 1) for i in range(tail, length)], sink, sharp)
    close(decoded, want, ATT_TOL[dtype], "a decoded tail")
    if cores:
        assert ran["latent_attention.merge"] == 20
    cuts = list(range(0, length - 2, 23)) + [length]
    pieces, _, _, _ = _latent_case(dtype, *case, list(zip(cuts, cuts[1:])), sink, sharp)
    assert torch.equal(pieces, whole)
    other, _, _, _ = _latent_case(dtype, *case, [(0, length)], sink, sharp, row_major=False, tiles=False)
    assert torch.equal(other, whole)
    first, _, _, _ = _latent_case(dtype, *case, [(0, 1), (1, 2), (2, 3)], sink, sharp)
    close(first[:3], want[:3], ATT_TOL[dtype], "the first tokens one by one")
    bare, no_sink, _, _ = _latent_case(dtype, *case, [(0, length)], [-1e30] * H, sharp)
    close(bare, no_sink, ATT_TOL[dtype], "a sink of nothing")
    assert float(np.abs(no_sink - want).max()) > 0.1 * float(np.abs(no_sink).max()) or H == 1      # leaving the sinks out shows


# ---------------------------------------------------------------------------
# kernels alone: the delta rule
class Delta:
    """One layer's projected rows and weights for a run of T tokens, and its plain results."""

    def __init__(self, H, G, D, V, taps, T, seed, forget=2.0):
        rng = np.random.default_rng(seed)
        self.sizes, self.taps, self.T = (H, G, D, V), taps, T
        self.C = 2 * G * D + H * V
        self.pre = rng.normal(size=(T, self.C + 2 * H + 3)).astype(np.float32)
        self.pre[:, :2 * G * D] += 0.8                   # keys that resemble each other: corrections matter
        self.conv = (rng.normal(size=(self.C, taps)) * 0.6).astype(np.float32)
        self.dt_bias, self.a_log = rng.normal(size=H).astype(np.float32), (rng.normal(size=H) * forget - 3).astype(np.float32)
        if T > 40:
            self.pre[33, self.C + H:self.C + 2 * H] = 60.0       # one token forgets (nearly) everything
        p = self.pre.astype(np.float64)
        act = plain.short_conv_silu(p[:, :self.C], self.conv.astype(np.float64))
        share = lambda x: np.repeat(plain.unit(x.reshape(T, G, D)), H // G, axis=1)
        q, k, v = share(act[:, :G * D]) * D ** -0.5, share(act[:, G * D:2 * G * D]), act[:, 2 * G * D:].reshape(T, H, V)
        beta = plain.sigmoid(p[:, self.C:self.C + H])
        decay = np.exp(-np.exp(self.a_log.astype(np.float64)) * plain.softplus(p[:, self.C + H:self.C + 2 * H] + self.dt_bias))
        self.o, self.S = plain.delta_scan(q, k, v, decay, beta)
        self.o = self.o.reshape(T, H * V)
        self.weights = [dev(x) for x in (self.conv, self.dt_bias, self.a_log)]
        self.matrix = ops().state_matrix_size(H, D, V)
        self.stride = -(-(self.matrix + (taps - 1) * self.C) // 4) * 4

    def step(self, rows, counts, state, slots_read, slots_write, form=None):
        """A step over `rows` [T, ld]: prepared and carried on as the mixer does; form "step", "scan" or "chunks" forces a kernel."""
        o = ops()
        H, G, D, V = self.sizes
        T, C = rows.shape[0], self.C
        starts = np.concatenate([[0], np.cumsum(counts)[:-1]])
        er, sr, sw = dev(np.stack([starts, counts], axis=1), torch.int32), dev(slots_read, torch.int32), dev(slots_write, torch.int32)
        entry = dev(np.repeat(np.arange(len(counts)), counts), torch.int32)
        conv, dt_bias, a_log = self.weights
        out = torch.full((T, H * V), 9.0, device="cuda")
        a = rows[:, C + H:C + 2 * H]
        if form == "step" or (form is None and max(counts) == 1):
            o.delta_step(rows, conv, a, dt_bias, a_log, state, self.matrix, sr, sw, er, out, D ** -0.5, G, H, D, V, C, head_decay=True)
            return out
        q, k, v, decay, beta, log_decay = (torch.full((T, w), 9.0, device="cuda") for w in (G * D, G * D, H * V, H, H, H))
        o.delta_prep(rows, conv, a, dt_bias, a_log, state, self.matrix, sr, entry, er, q, k, v, decay, beta, G, H, D, V, C, head_decay=True, log_decay=log_decay)
        tail = (rows[:, :C], self.taps, self.matrix) if self.taps > 1 else None
        plan = o.decayed_plan(counts, "cuda") if form is None else o.DecayedPlan(counts, 64, "cuda") if form == "chunks" else None
        if form == "chunks":
            assert plan.short_entries == 0
        if plan is not None:
            o.delta_chunks(q, k, v, log_decay, beta, state, sr, sw, er, out, D ** -0.5, H, G, D, V, plan, tail=tail)
        if plan is None or plan.short_entries:
            o.state_scan(q, k, v, decay, beta, state, sr, sw, er, out, D ** -0.5, H, G, D, V, tail=tail, max_rows=max(counts), head_decay=True,
                         max_rows_here=o.DECAYED_CHUNKS_MIN_ROWS - 1 if plan is not None else 0)
        return out

    def run(self, cuts, form=lambda n: None):
        pre = dev(self.pre)
        state = torch.zeros(3, self.stride, device="cuda")
        state[2] = 5.0
        held, out = 0, []
        for a, b in cuts:
            out.append(self.step(pre[a:b].contiguous(), [b - a], state, [held], [1 - held], form(b - a)))
            held = 1 - held
        assert bool((state[2] == 5.0).all())
        H, G, D, V = self.sizes
        tail = state[held][self.matrix:self.matrix + (self.taps - 1) * self.C].cpu()
        return torch.cat(out).cpu(), ops().state_matrix_plain(state[held], H, D, V).cpu(), tail


DELTA_SIZES = [(4, 2, 16, 24, 3), (3, 3, 5, 7, 1), (2, 1, 128, 128, 4), (2, 1, 72, 40, 8), (1, 1, 200, 33, 2), (6, 2, 64, 16, 4), (1, 1, 256, 100, 4), (4, 1, 33, 1, 6)]


@pytest.mark.parametrize("sizes", DELTA_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_delta_rule_by_rows_by_steps_and_by_chunks(sizes):
    T = 333
    case = Delta(*sizes, T, sum(sizes))
    results = {
        "row by row": case.run([(0, 100), (100, 103), (103, T)], lambda n: "scan"),
        "step by step": case.run([(i, i + 1) for i in range(T)], lambda n: "step"),
        "chunk by chunk": case.run([(0, T)], lambda n: "chunks"),
        "in turns": case.run([(0, 5), (5, 140), (140, 141), (141, 142), (142, 330), (330, T)]),
        "two long runs": case.run([(0, 129), (129, T)], lambda n: "chunks"),
        "pairs": case.run([(i, min(i + 2, T)) for i in range(0, T, 2)]),
    }
    for what, (o, S, tail) in results.items():
        close(o, case.o, 2e-5, what)
        close(S, case.S, 2e-5, "state, " + what)
        if case.taps > 1:
            assert torch.equal(tail, torch.from_numpy(case.pre[T - case.taps + 1:, :case.C].flatten())), what
    for what in ("step by step", "pairs"):
        assert torch.equal(results[what][0], results["row by row"][0]) and torch.equal(results[what][1], results["row by row"][1])


def test_delta_rule_remembers_over_many_chunks_and_forgets_at_once():
    """Decays of nearly 1: the state after 1,100 tokens still holds the first key; then a token whose decay is 0."""
    case = Delta(2, 1, 32, 16, 4, 1100, 3, forget=0.0)
    case.a_log[:] = -9.0
    again = Delta.__new__(Delta)
    again.__dict__.update(case.__dict__)
    p = case.pre.astype(np.float64)
    for at, what in ((None, "remembers"), (900, "forgets")):
        pre = case.pre.copy()
        pre[33, case.C + 2:case.C + 4] = 0.0
        if at is not None:
            pre[at, case.C + 2:case.C + 4] = 3e6
        again.pre = pre
        H, G, D, V = case.sizes
        act = plain.short_conv_silu(pre[:, :case.C].astype(np.float64), case.conv.astype(np.float64))
        k, v = np.repeat(plain.unit(act[:, G * D:2 * G * D].reshape(-1, G, D)), H, axis=1), act[:, 2 * G * D:].reshape(-1, H, V)
        q = np.repeat(plain.unit(act[:, :G * D].reshape(-1, G, D)), H, axis=1) * D ** -0.5
        beta = plain.sigmoid(pre[:, case.C:case.C + H].astype(np.float64))
        decay = np.exp(-np.exp(-9.0) * plain.softplus(pre[:, case.C + H:case.C + 2 * H].astype(np.float64) + case.dt_bias))
        want, S = plain.delta_scan(q, k, v, decay, beta)
        again.weights = [case.weights[0], case.weights[1], dev(case.a_log)]
        for cuts in ([(0, 1100)], [(0, 500), (500, 501), (501, 1100)]):
            o, got, _ = again.run(cuts)
            assert bool(torch.isfinite(o).all()) and bool(torch.isfinite(got).all())
            close(o, want.reshape(1100, -1), 4e-5, what)
            close(got, S, 4e-5, what)
    assert p.shape[0] == 1100


def test_long_and_short_entries_share_a_step_of_the_delta_rule():
    """Two long entries, a short one and a single token in one step: every entry has the bits, the state and the tail it has alone, and
    the preparation's form for many rows has the bits of the other."""
    o = ops()
    H, G, D, V, taps = 2, 1, 32, 24, 4
    counts = [150, 1, 300, 40]
    case = Delta(H, G, D, V, taps, sum(counts), 1)
    pre = dev(case.pre)
    start = dev(np.random.default_rng(2).normal(size=(9, case.stride)))
    state = start.clone()
    together = case.step(pre, counts, state, [0, 1, 2, 3], [4, 5, 6, 7])
    at = 0
    for i, n in enumerate(counts):
        s = start.clone()
        alone = case.step(pre[at:at + n].contiguous(), [n], s, [i], [4 + i])
        assert torch.equal(alone, together[at:at + n]), f"entry {i}"
        plain_of = lambda t: o.state_matrix_plain(t[4 + i], H, D, V)
        assert torch.equal(plain_of(s), plain_of(state)) and torch.equal(s[4 + i][case.matrix:], state[4 + i][case.matrix:]), f"entry {i}"
        at += n
    assert torch.equal(state[:4], start[:4]) and torch.equal(state[8], start[8])


# ---------------------------------------------------------------------------
# the engine
def make_engine(name, dtype, kv_tokens=1024, max_requests=4, graphs=True, folder=None):
    from llmx_amd.engine import Engine
    return Engine.load(folder or model_folder(name), dtype=dtype, kv_tokens=kv_tokens, page_tokens=PAGES[name], max_requests=max_requests, graphs=graphs)


@pytest.fixture(scope="module", params=[(n, d) for n in CONFIGS for d in ("float32", "bfloat16")], ids=lambda p: f"{p[0]}-{p[1]}")
def setup(request):
    name, dtype = request.param
    return name, dtype, make_engine(name, dtype)


def run_cut(engine, rid, tokens, cuts):
    from llmx_amd.engine import StepEntry
    engine.add_request(rid)
    rows = [engine.step([StepEntry(rid, tokens[a:b], list(range(b - a)))]).clone() for a, b in cuts]
    engine.end_request(rid)
    return torch.cat(rows).cpu()


def against(name, dtype, got, want, what="", tol=None):
    want = torch.as_tensor(want)
    if dtype == "float32":
        close(got, want, tol or F32_TOL, what)
        return
    rms = float((got.double() - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
    assert rms <= BF16_RMS[name], f"{what}: root mean square of the differences {rms:.3e} of the logits'"
    close(got, want, BF16_TOL[name], what)


LENGTHS = (1, 2, 9, 33, 75, 127, 130, 200)


def test_whole_prompts_and_every_layer(setup):
    name, dtype, engine = setup
    for seed, length in enumerate(LENGTHS):
        against(name, dtype, run_cut(engine, "w", tokens_for(name, length, seed), [(0, length)]), plain_logits(name, length, seed), f"{length} tokens")
    if dtype != "float32":
        return
    config, tensors = load_plain(model_folder(name))
    tokens = tokens_for(name, 140, 99)
    layers, seen = [], []
    plain.forward(config, tensors, tokens, layers)
    engine.observer = lambda step, kind, **t: seen.append(t["residual"].clone()) if kind == "layer" else None
    try:
        run_cut(engine, "layers", tokens, [(0, 140)])
    finally:
        engine.observer = None
    assert len(seen) == len(layers) == len(plain.run_order(config))
    for i, (got, want) in enumerate(zip(seen, layers)):
        close(got, want, F32_TOL, f"residual after layer run {i}")


def test_prompt_against_token_by_token_and_portions(setup):
    """Whole, token by token from the first token, most of it whole and the rest one by one, portions of changing size down to two
    tokens and to one, pairs, a long portion after short ones.  float32: cuttings whose portions are all too short for the
    chunked recurrence agree bit for bit, the others within CUT_TOL; bfloat16: each against the plain implementation."""
    name, dtype, engine = setup
    length, seed = 170, 5
    tokens = tokens_for(name, length, seed)
    cuttings = {
        "one by one": [(i, i + 1) for i in range(length)],
        "decoded tail": [(0, 120)] + [(i, i + 1) for i in range(120, length)],
        "portions": portions(length, 1),
        "portions of one": portions(length, 2, smallest=1),
        "pairs": [(i, min(i + 2, length)) for i in range(0, length, 2)],
        "whole": [(0, length)],
        "long after short": [(0, 3), (3, 4), (4, 150), (150, 151), (151, length)],
    }
    want = plain_logits(name, length, seed)
    rows = {}
    for what, cuts in cuttings.items():
        rows[what] = run_cut(engine, what, tokens, cuts)
        against(name, dtype, rows[what], want, what)
    if dtype == "float32":
        for what in cuttings:
            if max(b - a for a, b in cuttings[what]) < ops().DECAYED_CHUNKS_MIN_ROWS:
                assert torch.equal(rows[what], rows["one by one"]), f"{what}: first at row {int((rows[what] != rows['one by one']).any(1).nonzero()[0])}"
            else:
                close(rows[what], rows["one by one"], CUT_TOL, what)


def test_unequal_requests_in_one_batch_and_reused_pages_and_seats(setup):
    """Eight requests of unequal length through four seats, portions of some beside single tokens of others, in an engine
    with so few pages that ended requests' pages and seats are taken again by later ones; every row has the bits it has when
    its request runs alone in a fresh engine under the same cuts."""
    from llmx_amd.engine import StepEntry
    name, dtype, _ = setup
    lengths = [150, 23, 1, 96, 40, 17, 164, 5]
    engine = make_engine(name, dtype, kv_tokens=4 * 176, max_requests=4)
    rng = random.Random(3)
    waiting = list(range(len(lengths)))
    live, fed, got, cuts = [], {}, {i: [] for i in range(len(lengths))}, {i: [] for i in range(len(lengths))}
    while waiting or live:
        while waiting and len(live) < 4:
            i = waiting.pop(0)
            engine.add_request(i)
            live.append(i)
            fed[i] = 0
        entries, taken = [], []
        for i in live:
            if rng.random() < 0.2 and len(live) > 1:
                continue                                     # a request may be left out of a step
            left = lengths[i] - fed[i]
            n = 1 if rng.random() < 0.4 else min(left, rng.choice([2, 3, 8, 16, 31, 140]))
            entries.append(StepEntry(i, tokens_for(name, lengths[i], 20 + i)[fed[i]:fed[i] + n], list(range(n))))
            taken.append((i, n))
        if not entries:
            continue
        out = engine.step(entries).clone().cpu()
        at = 0
        for i, n in taken:
            got[i].append(out[at:at + n])
            cuts[i].append((fed[i], fed[i] + n))
            at += n
            fed[i] += n
            if fed[i] == lengths[i]:
                engine.end_request(i)
                live.remove(i)
    alone = make_engine(name, dtype)
    for i, n in enumerate(lengths):
        want = run_cut(alone, i, tokens_for(name, n, 20 + i), cuts[i])
        assert torch.equal(torch.cat(got[i]), want), f"request {i} in batches against itself alone"
        against(name, dtype, want, plain_logits(name, n, 20 + i), f"request {i}")
    assert all(engine.cache.pages_in_use(g) == 0 for g in range(len(engine.cache.groups)))
    assert engine.cache.slots.in_use == 0


def test_long_decoding_and_graph_replays(setup):
    """A short prompt, then 230 tokens one by one: an engine that replays decode steps as graphs against one that does not, and
    against the plain implementation."""
    name, dtype, engine = setup
    length, seed = 250, 8
    tokens = tokens_for(name, length, seed)
    cuts = [(0, 20)] + [(i, i + 1) for i in range(20, length)]
    before = engine.graph_replays
    got = run_cut(engine, "long", tokens, cuts)
    assert engine.graphs and engine.graph_replays - before > 150
    assert torch.equal(run_cut(make_engine(name, dtype, graphs=False), "long", tokens, cuts), got)
    against(name, dtype, got, plain_logits(name, length, seed))


def test_which_kernels_a_serving_step_takes():
    """The launch witness: a bfloat16 step at sizes the matrix cores take (configuration A: seven layer runs) runs the design's kernels
    and never the universal ones; a float32 engine runs the universal attentions and launches no bfloat16 product."""
    from llmx_amd.engine import StepEntry
    o = ops()
    tokens = tokens_for("A", 200, 2)
    for dtype in ("bfloat16", "float32"):
        engine = make_engine("A", dtype, graphs=False)
        engine.add_request("r")
        seen = []
        for entry in (StepEntry("r", tokens[:150], [149]), StepEntry("r", tokens[150:199], [48]), StepEntry("r", tokens[199:], [0])):
            o.take_launches()
            engine.step([entry])
            seen.append(o.take_launches())
        for s in seen:
            # a bfloat16 step of one row norms its rows in the products that read them, all but the head's
            assert s["layernorm"] == (1 if dtype == "bfloat16" and s is seen[2] else 7 + 6 + 1) and s["join_rows"] == 2 and s["latent_prep"] == 1 and s["head_norm_gate"] == 3
            assert s["qknorm_rope_kvwrite"] == 3 and s["scale_softcap"] == 1
            assert not any(n in s for n in ("combine_rows", "cast_rows", "gate_heads", "head_gate", "head_norm_rope_kvwrite", "scale_add"))
        assert seen[0]["delta_chunks"] == 3 and "state_scan" not in seen[0] and seen[0]["delta_prep"] == 3
        assert seen[1]["state_scan"] == 3 and seen[1]["delta_prep"] == 3
        assert seen[2]["delta_step"] == 3 and "state_scan" not in seen[2] and "delta_prep" not in seen[2]
        every = {k for s in seen for k in s}
        if dtype == "bfloat16":
            assert not any(n.startswith(("gemm_generic", "latent_attention.generic", "attention.generic")) for n in every), sorted(every)
            assert seen[0]["attention.tiles"] == 1 and any(n.startswith("attention.rules") for n in seen[0])
            assert seen[0]["latent_attention.tiles"] == 1 and seen[2]["latent_attention.rows"] == 1 and seen[2]["latent_attention.merge"] == 1
        else:
            assert "latent_attention.generic" in every and "attention.generic" in every
            assert not any(n.startswith(("gemm_skinny", "gemm_tile", "latent_attention.mfma", "latent_attention.tiles")) for n in every), sorted(every)


def test_a_failed_step_leaves_pages_and_states_as_they_were():
    from llmx_amd.cache import OutOfPages
    from llmx_amd.engine import StepEntry, StepError
    name = "A"
    tokens = tokens_for(name, 60, 1)
    engine = make_engine(name, "float32", kv_tokens=64, max_requests=2)
    engine.add_request("a")
    engine.add_request("b")
    first = engine.step([StepEntry("a", tokens[:20], [19])]).clone()
    with pytest.raises(OutOfPages):
        engine.step([StepEntry("a", tokens[20:40], [19]), StepEntry("b", tokens[:60], [])])
    with pytest.raises(StepError):
        engine.truncate("a", 5)                 # states cannot be taken back to the middle
    rest = engine.step([StepEntry("a", tokens[20:60], list(range(40)))]).clone().cpu()
    whole = run_cut(make_engine(name, "float32"), "w", tokens, [(0, 60)])
    assert torch.equal(first.cpu()[0], whole[19]) and torch.equal(rest, whole[20:])
    engine.truncate("a", 0)                     # back to nothing: the first token is a first token again
    assert torch.equal(engine.step([StepEntry("a", tokens, list(range(60)))]).cpu(), whole)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sharp_attention_and_long_memory_over_a_long_prompt(dtype, tmp_path):
    """Larger query norms let the softmax pick single keys, so a lost key shows; sinks of the keys' size; decays near 1 make the states
    remember hundreds of tokens.  Whole, portions and decoding against the plain model."""
    def edit(tensors):
        for k in tensors:
            if k.endswith("mix.q.norm"):
                tensors[k] = tensors[k] * 4.0
            if k == "l3.mix.q":
                tensors[k] = tensors[k] * 4.0
            if k.endswith("mix.sink"):
                tensors[k] = tensors[k] + 2.0
            if k.endswith("A_log"):
                tensors[k] = tensors[k] * 0.0 - 8.0
    folder = write_folder(CONFIGS["A"], 77, str(tmp_path / "sharp"), edit)
    engine = make_engine("A", dtype, folder=folder)
    config, tensors = load_plain(folder)
    length = 520
    tokens = tokens_for("A", length, 4)
    want = plain.forward(config, tensors, tokens)
    cuttings = {"whole": [(0, length)], "portions": portions(length, 9), "decoded": [(0, length - 90)] + [(i, i + 1) for i in range(length - 90, length)]}
    for what, cuts in cuttings.items():
        rows = run_cut(engine, what, tokens, cuts)
        if dtype == "float32":
            close(rows, want, 1e-4, what)
        else:
            rms = float((rows.double() - torch.as_tensor(want)).pow(2).mean().sqrt() / torch.as_tensor(want).pow(2).mean().sqrt())
            assert rms < 5e-2, f"{what}: {rms}"
    if dtype == "float32":      # the first token is still felt at the end
        b = plain.forward(config, tensors, [(tokens[0] + 1) % 300] + tokens[1:])[-1]
        assert float(np.abs(want[-1] - b).max()) > 1e-3 * float(np.abs(want[-1]).max())


def test_a_scheduler_serves_the_design():
    """`generate` (scheduler, step function, device sampler) with prompts of unequal length and a small step budget, so that
    prompts are cut into portions beside decoding requests; float32 picks the plain implementation's tokens."""
    from llmx_amd import SamplingParams, generate
    name = "A"
    config, tensors = load_plain(model_folder(name))
    prompts = [tokens_for(name, n, 40 + n) for n in (3, 29, 11, 1, 18)]
    engine = make_engine(name, "float32", kv_tokens=512, max_requests=3)
    got = generate(engine, prompts, SamplingParams(max_tokens=10, temp=0.0), max_seqs=3, max_step_tokens=16)
    for p, g in zip(prompts, got):
        assert g == greedy(config, tensors, p, 10)
    got16 = generate(make_engine(name, "bfloat16", kv_tokens=512, max_requests=3), prompts, SamplingParams(max_tokens=10, temp=0.0), max_seqs=3, max_step_tokens=16)
    near = 0
    for p, g in zip(prompts, got16):
        assert len(g) == 10
        rows = plain.forward(config, tensors, p + g[:-1])[len(p) - 1:]
        near += sum(rows[i, t] >= rows[i].max() - 0.1 * np.abs(rows[i]).max() for i, t in enumerate(g))
    assert near >= 45


def test_trace_replay_and_command_line(tmp_path):
    """bin/trace_run as a subprocess on a model folder: a prompt portion beside decoded tokens, requests that end and whose seats
    are taken again; the logits files are the plain model's rows.  `llmx logits` reads the same folder."""
    name = "C"
    a, b, c = tokens_for(name, 40, 1), tokens_for(name, 9, 2), tokens_for(name, 30, 3)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:33], "want": [0, 32]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[33:34], "want": [0]}, {"id": "b", "tokens": b, "want": [8]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "c", "tokens": c[:2], "want": []}], "end": []},
        {"step": 3, "entries": [{"id": "c", "tokens": c[2:], "want": [27]}, {"id": "a", "tokens": a[34:], "want": [5]}], "end": ["a", "c"]},
    ]
    out = tmp_path / "out"
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", model_folder(name), "--dtype", "float32", "--out", str(out),
                          "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    V = CONFIGS[name]["vocab"]
    want = {"a": plain_logits(name, 40, 1), "b": plain_logits(name, 9, 2), "c": plain_logits(name, 30, 3)}
    rows = {0: [("a", 0), ("a", 32)], 1: [("a", 33), ("b", 8)], 3: [("c", 29), ("a", 39)]}
    assert not (out / "2.f32").exists()
    for step, places in rows.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, V))
        assert got.shape[0] == len(places)
        for r, (rid, p) in enumerate(places):
            close(got[r], want[rid][p], F32_TOL)
    cli = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "llmx"), "logits", model_folder(name), " ".join(map(str, b)), "--dtype", "f32", "--top", "1"],
                         capture_output=True, text=True, timeout=600)
    assert cli.returncode == 0, cli.stderr[-2000:]
    assert int(cli.stdout.splitlines()[-1].split()[0]) == int(torch.argmax(want["b"][8]))


def test_command_line_generates_from_a_configuration_with_random_weights(tmp_path):
    """`llmx generate --config JSON --random SEED` for this design: weights generated on the device, the scheduler's loop,
    the device sampler."""
    cfg = tmp_path / "config.json"
    cfg.write_text(json.dumps(copy.deepcopy(CONFIGS["A"])))
    outs = []
    for _ in range(2):
        run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "llmx"), "generate", "--config", str(cfg), "--random", "5", "--std", "0.06",
                              "3 1 4 1 5 9 2 6", "-n", "9", "--temp", "0"], capture_output=True, text=True, timeout=600)
        assert run.returncode == 0, run.stderr[-2000:]
        ids = [int(t) for t in run.stdout.split()]
        assert len(ids) == 9 and all(0 <= t < CONFIGS["A"]["vocab"] for t in ids)
        outs.append(ids)
    assert outs[0] == outs[1]
