"""Neruzen in the engine against the plain implementation (tests/plain_neruzen.py), mechanism by mechanism and whole.

Kernels alone: the bigram embedding and the token shift over entries and state slots, the latent attention's preparation,
windowed attention over shuffled pages with one query made to fit a single key on both sides of a window's, a page's and a
segment's edge, the recurrence row by row, step by step and chunk by chunk, the norm over all heads, routing by groups.  Then
the engine under every way of cutting the same tokens into steps: in float32 against the plain implementation within F32_TOL
(and bit for bit among cuttings whose portions are too short for the chunked recurrence), in bfloat16 against the plain
implementation with the expert picks of that very run within BF16_TOL; pages and request seats that are used again; long
decoding; greedy generation through `generate`; the trace replay tool and the command line.
"""

from __future__ import annotations

import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_neruzen as plain
from neruzen_cases import CONFIGS, PAGES, Picks, greedy, load_plain, model_folder, plain_logits, portions, tokens_for, write_folder

pytestmark = pytest.mark.gpu

F32_TOL = 5e-5      # |engine - plain| over all logits relative to the largest |logit|: float32 sums in another order
CUT_TOL = 3e-5      # two cuttings of the same tokens where one runs the recurrence by chunks, float32
# the serving path against the plain implementation (float64, nothing rounded), with the engine's expert picks: the largest
# difference and the root mean square of all, relative to the logits'.  Met: 2.5e-2 and 1.1e-2; in B a head's read-out is
# hardly more than (q . k) v, whose sign alone is left after its norm, so where q . k is close to 0 a rounding turns a head
# over: single rows differ by up to 1.5e-1, all together by 1.6e-2
BF16_TOL = {"A": 5e-2, "B": 3e-1, "C": 5e-2, "D": 3e-2}
BF16_RMS = {"A": 1.6e-2, "B": 3e-2, "C": 1.8e-2, "D": 1.2e-2}
PICK_SLACK = 4e-7   # a pick's score lies among the best of the engine's own router logits within this
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [torch.float32, torch.bfloat16]
DTYPE_IDS = ["float32", "bfloat16"]


def ops():
    from llmx_amd import ops as o
    return o


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a)).to(device="cuda", dtype=dtype).contiguous()


def close(got, want, tol, what=""):
    got, want = (torch.as_tensor(np.asarray(t.cpu() if isinstance(t, torch.Tensor) else t)).double() for t in (got, want))
    err = float((got - want).abs().max()) / max(float(want.abs().max()), 1e-30)
    assert err <= tol, f"{what}: relative error {err:.3e} above {tol:.1e}"
    return err


# ---------------------------------------------------------------------------
# kernels alone: what a row takes from the token before it
def _step(counts, slots_read, slots_write):
    """Device arrays of a step with these rows an entry: (row_entry, entry_rows, slot_read, slot_write)."""
    starts = np.concatenate([[0], np.cumsum(counts)[:-1]])
    return (dev(np.repeat(np.arange(len(counts)), counts), torch.int32), dev(np.stack([starts, counts], axis=1), torch.int32),
            dev(slots_read, torch.int32), dev(slots_write, torch.int32))


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("bigram", [(50, 7, 3), (1, 5, 2), (97, 10 ** 12 + 39, 2 ** 31 + 5)], ids=["small", "one_bucket", "large_multipliers"])
def test_bigram_embedding_over_entries_and_steps(dtype, bigram):
    o = ops()
    buckets, a, b = bigram
    rng = np.random.default_rng(buckets)
    vocab, width = 2000, 300
    table, second = dev(rng.normal(size=(vocab, width)), dtype), dev(rng.normal(size=(buckets + 1, width)), dtype)
    seqs = [[int(t) for t in rng.integers(0, vocab, size=n)] for n in (11, 4, 1)]
    W = {"embed": table.double().cpu().numpy(), "bigram": second.double().cpu().numpy()}
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": a, "mul_cur": b}}}
    want = [plain.embed(s, W, cfg) for s in seqs]
    state = torch.zeros(8, 1, device="cuda", dtype=torch.int32)
    state[6] = 77                          # a slot of no request
    got = [[], [], []]
    fed, held = [0, 0, 0], [0, 1, 2]
    for counts in ([5, 1, 1], [1, 3, 0], [3, 0, 0], [1, 0, 0], [1, 0, 0]):
        live = [i for i in range(3) if counts[i]]
        n = [counts[i] for i in live]
        to = [(held[i] + 3) % 6 for i in live]
        entry, rows, sr, sw = _step(n, [held[i] for i in live], to)
        ids = dev(sum((seqs[i][fed[i]:fed[i] + counts[i]] for i in live), []), torch.int32)
        out = torch.empty(sum(n), width, device="cuda")
        o.embed_bigram(table, second, ids, state, sr, sw, entry, rows, out, buckets, a, b)
        at = 0
        for i, slot in zip(live, to):
            got[i].append(out[at:at + counts[i]].cpu())
            at += counts[i]
            fed[i] += counts[i]
            held[i] = slot
    assert fed == [11, 4, 1] and int(state[6]) == 77
    for i in range(3):
        close(torch.cat(got[i]), want[i], 1e-6, f"sequence {i}")


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("width", [54, 1500, 2048, 3000, 5000, 9000])
def test_token_shift_with_and_without_the_norm(dtype, width):
    """Entries of unequal length in steps of few rows and of more than a thousand (four rows a workgroup where they fit), the
    last row carried over in the state; the fused form has the bits of the norm kernel followed by the shift."""
    o = ops()
    rng = np.random.default_rng(width)
    lengths = [1100, 3, 40]
    xs = [rng.normal(size=(n, width)).astype(np.float32) for n in lengths]
    w, s = rng.uniform(0.5, 1.5, size=width), rng.uniform(0.0, 1.0, size=width)
    wd, sd = dev(w), dev(s)
    hs = [plain.rms_norm(x.astype(np.float64), wd.double().cpu().numpy(), 1e-5) for x in xs]
    want = [plain.token_shift(h, sd.double().cpu().numpy()) for h in hs]
    state = torch.zeros(6, width + 3, device="cuda")
    got, h_got = [[], [], []], [[], [], []]
    fed, held = [0, 0, 0], [0, 1, 2]
    for counts in ([1063, 1, 1], [1, 2, 38], [35, 0, 1], [1, 0, 0]):
        live = [i for i in range(3) if counts[i]]
        n = [counts[i] for i in live]
        to = [(held[i] + 3) % 6 for i in live]
        entry, rows, sr, sw = _step(n, [held[i] for i in live], to)
        T = sum(n)
        x = dev(np.concatenate([xs[i][fed[i]:fed[i] + counts[i]] for i in live]))
        shifted, h, h32 = (torch.empty(T, width, device="cuda", dtype=d) for d in (dtype, dtype, torch.float32))
        before = state.clone()
        o.token_shift(x, sd, state, sr, sw, entry, rows, shifted, norm=(wd, 1e-5), out=h, out32=h32)
        h_ref, h32_ref, again = (torch.empty_like(t) for t in (h, h32, shifted))
        o.rmsnorm(x, wd, 1e-5, h_ref, h32_ref)
        assert torch.equal(h, h_ref) and torch.equal(h32, h32_ref)
        o.token_shift(h32_ref, sd, before, sr, sw, entry, rows, again)
        assert torch.equal(again, shifted) and torch.equal(before, state)
        at = 0
        for i, slot in zip(live, to):
            got[i].append(shifted[at:at + counts[i]].float().cpu())
            h_got[i].append(h32[at:at + counts[i]].cpu())
            at += counts[i]
            fed[i] += counts[i]
            held[i] = slot
    assert fed == lengths
    tol = 1e-6 if dtype == torch.float32 else 5e-3
    for i in range(3):
        close(torch.cat(got[i]), want[i], tol, f"entry {i}")
        close(torch.cat(h_got[i]), hs[i], 1e-6, f"entry {i}, unshifted")


# ---------------------------------------------------------------------------
# kernels alone: latent attention
@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("sizes", [(3, 24, 16, 48, 40, 16), (2, 5, 6, 10, 7, 4), (16, 8, 64, 512, 96, 64), (4, 16, 8, 48, 300, 0)],
                         ids=["even", "ragged", "wide", "no_rotation"])
def test_latent_norms_cache_rows_and_queries(dtype, sizes):
    H, D, R, C, Cq, dims = sizes
    o = ops()
    from llmx_amd.parts.position import scaled_table
    rng = np.random.default_rng(C)
    T, page, eps = 37, 8, 1e-6
    width = o.latent_cache_width(C, R)
    proj, q = dev(rng.normal(size=(T, Cq + C + R + 3))), dev(rng.normal(size=(T, H * (D + R) + 5)))
    wq, wc = dev(rng.uniform(0.5, 1.5, Cq)), dev(rng.uniform(0.5, 1.5, C))
    order = list(range(8))
    random.Random(3).shuffle(order)
    tables = dev([order], torch.int32)
    past = 11
    pos, entry = dev(np.arange(past, past + T), torch.int32), dev(np.zeros(T), torch.int32)
    cos_sin = dev(scaled_table(64, dims, 300.0, None, True))
    cache, cache_t = torch.zeros(8, page, width, device="cuda", dtype=dtype), torch.zeros(8, C, page, device="cuda", dtype=dtype)
    c_q = torch.empty(T, Cq, device="cuda", dtype=dtype)
    o.latent_down(proj, wq, c_q, wc, cos_sin, pos, entry, tables, cache, eps, Cq, R, C, cache_t=cache_t, pairing=o.ROPE_HALVES)
    p64, rot = proj.double().cpu().numpy(), {"base": 300.0, "dims": dims}
    tol = 2e-6 if dtype == torch.float32 else 5e-3
    close(c_q.float(), plain.rms_norm(p64[:, :Cq], wq.double().cpu().numpy(), eps), tol, "query latent")
    lat = plain.rms_norm(p64[:, Cq:Cq + C], wc.double().cpu().numpy(), eps)
    key = plain.rotate_halves(p64[:, Cq + C:Cq + C + R], np.arange(past, past + T), rot)
    flat = torch.stack([cache[order[p // page], p % page] for p in range(past, past + T)]).float().cpu()
    close(flat[:, :C], lat, tol, "latent")
    close(flat[:, C:C + R], key, tol, "key part")
    assert not flat[:, C + R:].any()
    assert torch.equal(cache_t.transpose(1, 2), cache[:, :, :C])
    for row_major in (False, True):
        lead = (T, H) if row_major else (H, T)
        plain_part, rot_part = torch.empty(*lead, D, device="cuda", dtype=dtype), torch.empty(*lead, R, device="cuda", dtype=dtype)
        o.latent_queries(q, cos_sin, pos, plain_part, rot_part, H, D, R, o.ROPE_HALVES, row_major)
        if not row_major:
            plain_part, rot_part = plain_part.transpose(0, 1), rot_part.transpose(0, 1)
        q64 = q[:, :H * (D + R)].double().cpu().numpy().reshape(T, H, D + R)
        close(plain_part.float(), q64[..., :D], tol, "unrotated queries")
        close(rot_part.float(), plain.rotate_halves(q64[..., D:], np.arange(past, past + T), rot), tol, "rotated queries")


def _window_case(dtype, H, C, R, page, length, window, runs, sharp=None, row_major=True, tiles=True, seed=0):
    """Windowed attention over latents in shuffled pages, beside an unrelated request: queries and cached rows are random;
    sharp = (row, key): the row's queries are made to fit that key alone, whether the row may see it or not.  Pages that
    no row of a run can see are named -1 in the table, as the cache manager leaves them.  runs: [(first row, end), ...]."""
    o = ops()
    rng = np.random.default_rng(seed + H * 1000 + C + length)
    c, r = rng.normal(size=(length, C)), rng.normal(size=(length, R))
    ql, qr = rng.normal(size=(length, H, C)) * 0.3, rng.normal(size=(length, H, R)) * 0.3
    if sharp is not None:
        row, key = sharp
        ql[row] = c[key] * 4.0
        qr[row] = r[key] * 4.0
    cores = o.latent_attention_mfma_ok(dtype, C, R, page, o.latent_cache_width(C, R))
    width = o.latent_cache_width(C, R) if cores else C + R
    n_pages = -(-length // page)
    order = list(range(n_pages + 4))
    random.Random(length).shuffle(order)
    cache = torch.zeros(n_pages + 4, page, width, device="cuda", dtype=dtype)
    cache_t = torch.zeros(n_pages + 4, C, page, device="cuda", dtype=dtype)
    cd, rd = dev(c, dtype), dev(r, dtype)
    at = torch.tensor([order[p // page] * page + p % page for p in range(length)], device="cuda")
    cache.view(-1, width)[at, :C] = cd
    cache.view(-1, width)[at, C:C + R] = rd
    cache_t.copy_(cache[:, :, :C].transpose(1, 2))
    qld, qrd = dev(ql, dtype), dev(qr, dtype)
    scale = 0.4 / (C + R) ** 0.5 * 3
    out = torch.zeros(length, H, C)
    ran = {}
    for a, b in runs:
        n = b - a
        table = [order[i] if (i + 1) * page > a - window + 1 else -1 for i in range(n_pages)]
        tables = dev([[-1] * n_pages, table], torch.int32)
        pos, entry = dev(np.arange(a, b), torch.int32), dev(np.ones(n), torch.int32)
        x, y = qld[a:b], qrd[a:b]
        if not row_major:
            x, y = x.transpose(0, 1), y.transpose(0, 1)
        x, y = x.contiguous(), y.contiguous()
        mixed = torch.zeros_like(x)
        plan = o.latent_plan([0, n], H, "cuda", contexts=[0, b], tiles=tiles, window=window) if cores else None
        o.take_launches()
        o.latent_attention(x, y, cache, pos, entry, tables, mixed, scale, window=window, cache_t=cache_t if cores else None, plan=plan, row_major=row_major)
        for k, v in o.take_launches().items():
            ran[k] = ran.get(k, 0) + v
        out[a:b] = (mixed if row_major else mixed.transpose(0, 1)).float().cpu()
    c64, r64 = cd.double().cpu().numpy(), rd.double().cpu().numpy()
    q64, t64 = qld.double().cpu().numpy(), qrd.double().cpu().numpy()
    want = np.zeros((length, H, C))
    mask = plain.window_mask(length, window)
    for h in range(H):
        s = (q64[:, h] @ c64.T + t64[:, h] @ r64.T) * scale
        want[:, h] = plain.softmax_rows(np.where(mask, s, -np.inf)) @ c64
    return out, torch.as_tensor(want), ran, cores


ATT_TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("case", [(4, 48, 8, 16, 150, 40), (3, 10, 6, 4, 60, 5), (16, 32, 32, 16, 300, 101), (20, 96, 32, 16, 200, 64), (2, 64, 16, 16, 140, 65),
                                  (5, 128, 64, 32, 400, 129), (16, 512, 64, 16, 700, 300), (8, 16, 8, 8, 90, 1), (1, 16, 0, 48, 500, 2), (6, 64, 8, 16, 200, 1000),
                                  (7, 256, 64, 16, 330, 170)],
                         ids=lambda c: "x".join(map(str, c)))
def test_windowed_attention_over_shuffled_pages(dtype, case):
    H, C, R, page, length, window = case
    whole, want, ran, cores = _window_case(dtype, H, C, R, page, length, window, [(0, length)])
    close(whole, want, ATT_TOL[dtype], "a prompt")
    assert ("latent_attention.tiles" in ran) == cores and ("latent_attention.generic" in ran) != cores
    tail = length - 20
    decoded, _, ran, _ = _window_case(dtype, H, C, R, page, length, window, [(0, tail)] + [(i, i + 1) for i in range(tail, length)])
    close(decoded, want, ATT_TOL[dtype], "a decoded tail")
    if cores and window > 2 * ops().LATENT_SPLIT_WINDOW_KEYS:
        assert ran["latent_attention.merge"] == 20
    cuts = list(range(0, length - 2, 23)) + [length]
    pieces, _, _, _ = _window_case(dtype, H, C, R, page, length, window, list(zip(cuts, cuts[1:])))
    assert torch.equal(pieces, whole)          # portions of several rows give a row the whole prompt's bits
    other, _, _, _ = _window_case(dtype, H, C, R, page, length, window, [(0, length)], row_major=False, tiles=False)
    assert torch.equal(other, whole)           # the one-wave form and the other layout too


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("decoded", [False, True], ids=["prompt", "decoded"])
def test_one_key_on_both_sides_of_every_edge(dtype, decoded):
    """The row's queries fit one key: the first and last of the window and their neighbours outside and inside, page and segment
    borders, the row itself; windows that end on, before and behind such borders."""
    length = 300
    for window in (1, 64, 65, 87, 200):
        row = 281
        lo = row - window + 1
        for key in sorted({max(0, lo - 2), max(0, lo - 1), lo, lo + 1, row - 1, row, 255, 256, 192}):
            if key > row:
                continue
            for C, R, page in ((32, 32, 16), (48, 8, 16), (10, 6, 4)):
                runs = [(row, row + 1)] if decoded else [(row - 9, row + 10)]
                got, want, _, _ = _window_case(dtype, 4, C, R, page, length, window, runs, sharp=(row, key))
                close(got[row], want[row], ATT_TOL[dtype] * 2, f"window {window}, key {key}, latent {C}")
    if dtype == torch.float32 and not decoded:       # the sharp key does carry the weight where it is seen, and none where it is not
        _, inside, _, _ = _window_case(dtype, 4, 32, 32, 16, length, 64, [(281, 282)], sharp=(281, 218))
        _, outside, _, _ = _window_case(dtype, 4, 32, 32, 16, length, 64, [(281, 282)], sharp=(281, 217))
        assert float((inside[281] - outside[281]).abs().max()) > 0.5


# ---------------------------------------------------------------------------
# kernels alone: the recurrence
def _operands(o, kind, dims, T, first=0):
    from llmx_amd.parts.position import scaled_table
    if kind == "silu":
        return o.StateOperands(o.OPERANDS_SILU)
    if kind == "rotated":
        return o.StateOperands(o.OPERANDS_ROTATED, dev(scaled_table(600, dims, 40.0, None, True)), dev(np.arange(first, first + T), torch.int32))
    return None


@pytest.mark.parametrize("sizes", [(2, 16, 24, 8), (1, 7, 9, 6), (3, 64, 16, 64), (2, 80, 40, 12), (2, 128, 128, 128), (1, 200, 33, 40), (1, 256, 100, 0), (1, 20, 1, 4)],
                         ids=lambda s: "x".join(map(str, s)))
@pytest.mark.parametrize("kind", ["plain", "silu", "rotated"])
def test_recurrence_by_rows_by_steps_and_by_chunks(kind, sizes):
    """One request's rows all three ways, carried on between state slots: rows in short portions (the scan), single tokens (the
    step layout: the scan's bits), a long run (chunks on the matrix cores), and each after another; against the plain sums."""
    o = ops()
    H, D, V, dims = sizes
    rng = np.random.default_rng(D * 7 + V)
    T = 333
    decay = [(0.9, 0.995, 0.3)[i % 3] for i in range(H)]
    rows = rng.normal(size=(T, H * (2 * D + V) + 5)).astype(np.float32)
    pre = dev(rows)
    cols = (slice(0, H * D), slice(H * D, 2 * H * D), slice(2 * H * D, 2 * H * D + H * V))
    q, k, v = (rows[:, c].astype(np.float64) for c in cols)
    if kind == "silu":
        q, k, v = plain.silu(q), plain.silu(k), plain.silu(v)
    q, k = q.reshape(T, H, D), k.reshape(T, H, D)
    if kind == "rotated":
        q, k = (plain.rotate_halves(x, np.arange(T), {"base": 40.0, "dims": dims}) for x in (q, k))
    want, S = plain.decayed_outer_products(q, k, v.reshape(T, H, V), np.float32(decay))
    want, scale = want.reshape(T, H * V) * 0.5, 0.5
    stride = o.state_matrix_size(H, D, V) + 4
    decays = torch.tensor(decay, device="cuda").repeat_interleave(D).view(1, -1)
    powers = o.decay_powers(decay, "cuda")

    def run(cuts, form):
        state = torch.zeros(3, stride, device="cuda")
        state[2] = 5.0
        out = torch.zeros(T, H * V, device="cuda")
        held = 0
        for a, b in cuts:
            n = b - a
            part = [pre[a:b][:, c] for c in cols]
            y = torch.full((n, H * V), 9.0, device="cuda")
            _, er, sr, sw = _step([n], [held], [1 - held])
            held = 1 - held
            opnd = _operands(o, kind, dims, n, a)
            if form(n) == "chunks":
                plan = o.DecayedPlan([n], o.lib().llmx_decayed_state_rows(), "cuda")
                o.decayed_state_chunks(*part, powers, state, sr, sw, y, scale, H, D, V, plan, opnd)
            else:
                o.state_scan(*part, decays.expand(n, H * D), None, state, sr, sw, er, y, scale, H, H, D, V,
                             max_rows=n if form(n) == "step" else max(n, 2), operands=opnd)
            out[a:b] = y
        assert bool((state[2] == 5.0).all())
        return out.cpu(), o.state_matrix_plain(state[held], H, D, V).cpu()

    singles = [(i, i + 1) for i in range(T)]
    scanned, s_scan = run([(0, 100), (100, 103), (103, T)], lambda n: "scan")
    stepped, s_step = run(singles, lambda n: "step")
    close(scanned, want, 2e-5, "row by row")
    close(s_scan, S, 2e-5, "state")
    assert torch.equal(stepped, scanned) and torch.equal(s_step, s_scan)
    chunked, s_chunk = run([(0, T)], lambda n: "chunks")
    close(chunked, want, 2e-5, "chunk by chunk")
    close(s_chunk, S, 2e-5, "state after chunks")
    mixed, s_mixed = run([(0, 5), (5, 140), (140, 141), (141, 142), (142, 330), (330, T)], lambda n: "chunks" if n >= 128 else "step" if n == 1 else "scan")
    close(mixed, want, 2e-5, "in turns")
    close(s_mixed, S, 2e-5, "state after turns")


def test_long_and_short_entries_share_a_step():
    """A step with two long entries, a short one and a single token: each kernel takes its entries and leaves the others' rows,
    states and slots alone; every entry has the bits it has alone."""
    o = ops()
    H, D, V = 2, 32, 24
    rng = np.random.default_rng(1)
    counts = [150, 1, 300, 40]
    T = sum(counts)
    pre = dev(rng.normal(size=(T, H * (2 * D + V))))
    parts = lambda x: (x[:, :H * D], x[:, H * D:2 * H * D], x[:, 2 * H * D:])
    decay = [0.99, 0.7]
    decays, powers = torch.tensor(decay, device="cuda").repeat_interleave(D).view(1, -1), o.decay_powers(decay, "cuda")
    start = dev(rng.normal(size=(9, o.state_matrix_size(H, D, V))))

    def run(x, n, sr, sw):
        state, out = start.clone(), torch.full((x.shape[0], H * V), 7.0, device="cuda")
        _, er, sr, sw = _step(n, sr, sw)
        plan = o.decayed_plan(n, "cuda")
        if plan is not None:
            o.decayed_state_chunks(*parts(x), powers, state, sr, sw, out, 1.0, H, D, V, plan)
        if plan is None or plan.short_entries:
            o.state_scan(*parts(x), decays.expand(x.shape[0], H * D), None, state, sr, sw, er, out, 1.0, H, H, D, V, max_rows=max(n),
                         max_rows_here=o.DECAYED_CHUNKS_MIN_ROWS - 1 if plan is not None else 0)
        return out, state

    together, state = run(pre, counts, [0, 1, 2, 3], [4, 5, 6, 7])
    at = 0
    for i, n in enumerate(counts):
        alone, s = run(pre[at:at + n].contiguous(), [n], [i], [4 + i])
        assert torch.equal(alone, together[at:at + n]) and torch.equal(s[4 + i], state[4 + i]), f"entry {i}"
        at += n
    assert torch.equal(state[:4], start[:4]) and torch.equal(state[8], start[8])


@pytest.mark.parametrize("dtype", DTYPES, ids=DTYPE_IDS)
@pytest.mark.parametrize("width", [40, 512, 513, 2048, 5000])
def test_norm_over_all_heads_with_a_gate(dtype, width):
    o = ops()
    rng = np.random.default_rng(width)
    T = 9
    x, z, w = rng.normal(size=(T, width)) * 3, rng.normal(size=(T, width + 7)), rng.uniform(0.5, 1.5, size=width)
    out = torch.empty(T, width, device="cuda", dtype=dtype)
    o.head_norm_gate(dev(x), dev(w), dev(z)[:, :width], out, 1e-6, 1, width, o.GATE_SIGMOID)
    close(out.float(), plain.rms_norm(x, w, 1e-6) * plain.sigmoid(z[:, :width]), 2e-6 if dtype == torch.float32 else 5e-3, "weight and sigmoid")
    o.head_norm_gate(dev(x), None, dev(z)[:, :width], out, 1e-6, 1, width, o.GATE_SILU)
    close(out.float(), plain.rms_unit(x, 1e-6) * plain.silu(z[:, :width]), 2e-6 if dtype == torch.float32 else 5e-3, "silu")


# ---------------------------------------------------------------------------
# kernels alone: routing
@pytest.mark.parametrize("case", [(8, 2, 1, 4), (6, 3, 2, 2), (16, 4, 2, 4), (64, 8, 3, 6), (256, 8, 4, 8), (300, 10, 2, 5), (1024, 32, 5, 9), (5, 5, 2, 2), (12, 1, 1, 3),
                                  (8, 4, 4, 8), (160, 160, 7, 7)], ids=lambda c: "x".join(map(str, c)))
def test_routing_by_groups_picks_and_weights(case):
    o = ops()
    X, G, keep, k = case
    rng = np.random.default_rng(X + k)
    rows = 40
    z = rng.normal(size=(rows, X)) * 2
    z[0] = 0.0                                           # all alike: the lowest numbers of the lowest groups
    z[1, : X // 2] = z[1, X - X // 2:]                   # ties between groups
    z = z.astype(np.float32)
    cfg = {"router": {"experts": X, "top": k, "groups": {"count": G, "keep": keep}}}
    want_ids, want_w, _ = plain.route(z.astype(np.float64), {"r.router": np.eye(X)}, "r.", cfg)
    ids, w = torch.empty(rows, k, device="cuda", dtype=torch.int32), torch.empty(rows, k, device="cuda")
    o.route_topk(dev(z), None, ids, w, k, o.SCORE_SOFTMAX, "always", 1.0, groups=(G, keep))
    assert np.array_equal(ids.cpu().numpy(), want_ids)
    close(w, want_w, 2e-6, "weights")
    # few rows: routing and grouping in one launch, the same bits; no groups: the same as one group
    n = 12
    arrays = lambda: [torch.empty(s, device="cuda", dtype=torch.int32) for s in (X, X + 1, n * k, X, 1)]
    ids1, w1 = torch.empty(n, k, device="cuda", dtype=torch.int32), torch.empty(n, k, device="cuda")
    o.route_topk_align(dev(z[:n]), None, ids1, w1, k, o.SCORE_SOFTMAX, "always", 1.0, *arrays(), groups=(G, keep))
    assert torch.equal(ids1, ids[:n]) and torch.equal(w1, w[:n])
    # one slot more: expert number X with weight 1, grouped with the others
    more, w_more = torch.empty(rows, k + 1, device="cuda", dtype=torch.int32), torch.empty(rows, k + 1, device="cuda")
    for r in (n, rows):
        counts, offsets, pairs, active, n_active = (torch.empty(s, device="cuda", dtype=torch.int32) for s in (X + 1, X + 2, r * (k + 1), X + 1, 1))
        if X < 1024:
            o.route_topk_align(dev(z[:r]), None, more[:r], w_more[:r], k, o.SCORE_SOFTMAX, "always", 1.0, counts, offsets, pairs, active, n_active, groups=(G, keep))
            assert torch.equal(more[:r, :k], ids[:r]) and bool((more[:r, k] == X).all()) and bool((w_more[:r, k] == 1).all())
            assert int(counts[X]) == r and pairs[int(offsets[X]):].tolist() == [t * (k + 1) + k for t in range(r)]
            assert all(more[:r].flatten()[pairs[int(offsets[e]):int(offsets[e + 1])].long()].eq(e).all() for e in range(X + 1))
    one, none = torch.empty_like(ids), torch.empty_like(ids)
    o.route_topk(dev(z), None, one, w, k, o.SCORE_SOFTMAX, "always", 1.0, groups=(1, 1))
    o.route_topk(dev(z), None, none, w, k, o.SCORE_SOFTMAX, "always", 1.0)
    assert torch.equal(one, none)
    with pytest.raises(o.KernelError):
        o.route_topk(dev(z), None, one, w, k, o.SCORE_SOFTMAX, "always", 1.0, groups=(X + 1, 1))


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


def with_picks(engine, run):
    """(run(), the expert picks and router logits of every routed layer by request and position)."""
    engine.observer = Picks()
    try:
        return run(), engine.observer
    finally:
        engine.observer = None


def check_picks(config, picks, rid, length):
    """The engine's picks of a request, after checking every row's against the engine's own router logits: no expert twice, all
    from `keep` groups, and each score among the best of those groups."""
    logits, ids = picks.logits_of(rid, length), picks.of(rid, length)
    for i, got in ids.items():
        r = config["layers"][i]["mlp"]["router"]
        per = r["experts"] // r["groups"]["count"]
        s = plain.softmax_rows(logits[i].astype(np.float64))
        for t in range(length):
            assert len(set(got[t].tolist())) == r["top"]
            used = {e // per for e in got[t].tolist()}
            assert len(used) <= r["groups"]["keep"]
            best = np.sort([s[t, g * per:(g + 1) * per].max() for g in range(r["groups"]["count"])])[::-1]
            assert all(s[t, g * per:(g + 1) * per].max() >= best[r["groups"]["keep"] - 1] - PICK_SLACK for g in used)
            open_to = [e for e in range(r["experts"]) if s[t, (e // per) * per:(e // per + 1) * per].max() >= best[r["groups"]["keep"] - 1] + PICK_SLACK]
            worst = s[t, got[t]].min()
            assert all(s[t, e] <= worst + PICK_SLACK for e in open_to if e not in got[t])
    return ids


def against_plain(name, dtype, tokens, got, picks=None, rid=None, folder=None, tol=None):
    """float32 against the plain implementation; bfloat16 too, with the picks of the run that gave `got` (a near tie of two
    scores may fall the other way after rounding, and then another expert runs)."""
    config, tensors = load_plain(folder or model_folder(name))
    if dtype == "float32":
        close(got, plain.forward(config, tensors, tokens), tol or F32_TOL, "against the plain implementation")
        return
    ids = check_picks(config, picks, rid, len(tokens))
    want = torch.as_tensor(plain.forward(config, tensors, tokens, picks=ids))
    rms = float((got.double() - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
    close(got, want, BF16_TOL[name], "against the plain implementation with the engine's picks")
    assert rms <= BF16_RMS[name], f"root mean square of the differences {rms:.3e} of the logits'"


LENGTHS = (1, 2, 9, 33, 75, 127, 130, 200)


def test_whole_prompts_and_every_layer(setup):
    name, dtype, engine = setup
    for seed, length in enumerate(LENGTHS):
        tokens = tokens_for(name, length, seed)
        if dtype == "float32":
            close(run_cut(engine, "w", tokens, [(0, length)]), plain_logits(name, length, seed), F32_TOL, f"{length} tokens")
        else:
            got, picks = with_picks(engine, lambda: run_cut(engine, "w", tokens, [(0, length)]))
            against_plain(name, dtype, tokens, got, picks, "w")
    if dtype != "float32":
        return
    config, tensors = load_plain(model_folder(name))
    tokens = tokens_for(name, 140, 99)
    layers, seen = [], []
    plain.forward(config, tensors, tokens, layers_out=layers)
    engine.observer = lambda step, kind, **t: seen.append(t["residual"].clone()) if kind == "layer" else None
    try:
        run_cut(engine, "layers", tokens, [(0, 140)])
    finally:
        engine.observer = None
    assert len(seen) == len(layers) == len(config["layers"])
    for i, (got, want) in enumerate(zip(seen, layers)):
        close(got, want, F32_TOL, f"residual after layer {i}")


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
    rows = {}
    for what, cuts in cuttings.items():
        if dtype == "bfloat16":
            rows[what], picks = with_picks(engine, lambda: run_cut(engine, what, tokens, cuts))
            against_plain(name, dtype, tokens, rows[what], picks, what)
        else:
            rows[what] = run_cut(engine, what, tokens, cuts)
    if dtype == "float32":
        close(rows["whole"], plain_logits(name, length, seed), F32_TOL)
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
        if dtype == "float32":
            close(want, plain_logits(name, n, 20 + i), F32_TOL)
    assert all(engine.cache.pages_in_use(g) == 0 for g in range(len(engine.cache.groups)))
    assert engine.cache.slots.in_use == 0


def test_long_decoding_and_graph_replays(setup):
    """A short prompt, then 230 tokens one by one past every window: an engine that replays decode steps as graphs against one
    that does not, and against the plain implementation."""
    name, dtype, engine = setup
    length, seed = 250, 8
    tokens = tokens_for(name, length, seed)
    cuts = [(0, 20)] + [(i, i + 1) for i in range(20, length)]
    before = engine.graph_replays
    got = run_cut(engine, "long", tokens, cuts)
    assert engine.graphs and engine.graph_replays - before > 150
    eager = make_engine(name, dtype, graphs=False)
    again, picks = with_picks(eager, lambda: run_cut(eager, "long", tokens, cuts))
    assert torch.equal(again, got)
    against_plain(name, dtype, tokens, got, picks, "long")


def test_windows_give_pages_back_while_a_request_runs():
    """A long prompt in portions in an engine whose windowed pools could not hold it whole; what is read afterwards is right."""
    from llmx_amd.engine import Engine, StepEntry
    name, length = "A", 390
    engine = Engine.load(model_folder(name), dtype="float32", kv_tokens=400, page_tokens=16, max_requests=1, step_tokens=30)
    tokens = tokens_for(name, length, 6)
    engine.add_request("r")
    rows = []
    for a in range(0, length, 30):
        rows.append(engine.step([StepEntry("r", tokens[a:a + 30], list(range(min(30, length - a))))]).clone().cpu())
        used = {g.window: engine.cache.pages_in_use(i) for i, g in enumerate(engine.cache.groups)}
        assert used[40] <= 4 and used[101] <= 8
    assert all(g.n_pages < 25 for g in engine.cache.groups)
    engine.end_request("r")
    close(torch.cat(rows), plain_logits(name, length, 6), F32_TOL)


def test_which_kernels_a_serving_step_takes():
    """The launch witness: a bfloat16 step at sizes the matrix cores take (configuration A) runs the design's kernels and never
    the universal ones; a float32 engine runs the universal attention and launches no bfloat16 product."""
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
            assert s["embed_bigram"] == 1 and s["rmsnorm_shift"] == 4 and s["latent_prep"] == 4 and s["head_norm_gate"] == 2 and s["moe_combine"] == 3
            assert s["rmsnorm"] == 1 and "scale_add" not in s and "combine_rows" not in s and "token_shift" not in s and "head_gate" not in s
        # the shared expert of layer 3 is as wide as the routed ones and goes through their launches, layer 0's has its own
        if dtype == "bfloat16":
            assert seen[2]["gemm_skinny.grouped"] == 3 * 2 + 2 * 2
        assert seen[0]["decayed_state.chunks"] == 2 and "state_scan" not in seen[0]
        assert seen[1]["state_scan"] == 2 and seen[2]["state_step"] == 2
        assert seen[0]["route_topk"] == 3 and seen[2]["route_topk_align"] == 3
        every = {k: sum(s.get(k, 0) for s in seen) for s in seen for k in s}
        if dtype == "bfloat16":
            assert not any(n.startswith(("gemm_generic", "latent_attention.generic")) for n in every), sorted(every)
            assert seen[0]["latent_attention.tiles"] == 2 and seen[2]["latent_attention.rows"] == 2 and seen[2]["latent_attention.merge"] == 2
        else:
            assert every["latent_attention.generic"] == 6
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
    """Larger query weights let the softmax pick single keys, so a key lost at a page's or a window's edge shows; a decay near 1
    makes the states remember hundreds of tokens.  Whole, portions and decoding against the plain model."""
    import copy
    config = copy.deepcopy(CONFIGS["A"])
    config["layers"][1]["mixer"]["decay"] = [0.9995, 0.999, 0.9999]

    def edit(tensors):
        for k in tensors:
            if k.endswith("dq.norm"):
                tensors[k] = tensors[k] * 5.0
    folder = write_folder(config, 57, str(tmp_path / "sharp"), edit)
    engine = make_engine("A", dtype, folder=folder)
    length = 520
    tokens = tokens_for("A", length, 4)
    cuttings = {"whole": [(0, length)], "portions": portions(length, 9), "decoded": [(0, length - 90)] + [(i, i + 1) for i in range(length - 90, length)]}
    for what, cuts in cuttings.items():
        rows, picks = with_picks(engine, lambda: run_cut(engine, what, tokens, cuts))
        against_plain("A", dtype, tokens, rows, picks, what, folder=folder, tol=1e-4)
    if dtype == "float32":      # the states do remember: another first token changes the last row
        plain_config, tensors = load_plain(folder)
        a = plain.forward(plain_config, tensors, tokens)[-1]
        b = plain.forward(plain_config, tensors, [(tokens[0] + 1) % 320] + tokens[1:])[-1]
        assert float(np.abs(a - b).max()) > 1e-3 * float(np.abs(a).max())


def test_greedy_generation_through_the_scheduler():
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
    # bfloat16: every token is the plain implementation's best, given the tokens before it, within rounding
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
    cfg.write_text(json.dumps(CONFIGS["A"]))
    outs = []
    for _ in range(2):
        run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "llmx"), "generate", "--config", str(cfg), "--random", "5", "--std", "0.06",
                              "3 1 4 1 5 9 2 6", "-n", "9", "--temp", "0"], capture_output=True, text=True, timeout=600)
        assert run.returncode == 0, run.stderr[-2000:]
        ids = [int(t) for t in run.stdout.split()]
        assert len(ids) == 9 and all(0 <= t < CONFIGS["A"]["vocab"] for t in ids)
        outs.append(ids)
    assert outs[0] == outs[1]
