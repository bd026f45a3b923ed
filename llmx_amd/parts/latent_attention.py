"""Causal softmax attention over one cached latent a token (keys and values are low-rank expansions of it).

Per row, from the input h:  q = W_q h, or through a latent of its own q = W_uq rmsnorm(W_dq h), head by head [dim unrotated |
rot_dim rotated];  W_dkv h = [latent of kv_rank | one key part of rot_dim]: the latent is RMS-normed (weight `dkv.norm`) and
is, with the rotated key part that all heads share, all that is cached.  Head n's key for a token is [W_uk,n c | k_rot], its
value W_uv,n c; score = (q_plain . W_uk,n c + q_rot . k_rot) * scale, softmax over the request's keys up to the row (the last
`window` of them; with a sink the denominator also holds exp(sink_n), a learned number a head), and the head's result is multiplied by sigmoid(W_g h)_n, where there is a gate, before the output
projection.

Neither keys nor values are ever expanded: q_lat = W_uk,n^T q_plain (a grouped product, one group a head) turns the
score into (q_lat . c + q_rot . k_rot) * scale over the cached rows themselves, the attention returns the weighted sum of
latents, and W_uv,n is applied to that (a second grouped product; without a gate it stores the rows that the output
projection reads).
"""

from __future__ import annotations

import torch

from .. import ops
from .base import BuildContext, LayerCache, Mixer, build_part, register
from .spec import CacheTensor, PagedNeed, PartSpec, TensorSpec

MAX_LATENT = 2048          # the attention kernels keep a row's weighted sum of latents in a wave's registers
MAX_LATENT_KEY = 4096      # latent + rotated key part: a query row in a workgroup's LDS


class LatentAttention(Mixer):
    """params: hidden, heads, dim (unrotated query/key dims a head), rot_dim (rotated dims a head), vdim, kv_rank, scale (the
    factor on the scores), eps (of the latents' norms), gate ("head_sigmoid" | None), position (PartSpec of a rotary encoding
    whose dims are at most rot_dim), window (None: every earlier key), q_rank (None: one query projection), sink (True: a logit
    a head in the softmax's denominator).
    Tensors <prefix>q (or dq, dq.norm, uq), dkv, dkv.norm, uk, uv, g, sink, o."""
    graph_safe = True

    def __init__(self, params, prefix, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        p = params
        self.hidden = int(p["hidden"])
        self.heads = int(p["heads"])
        self.dim = int(p["dim"])
        self.rot_dim = int(p["rot_dim"])
        self.vdim = int(p["vdim"])
        self.rank = int(p["kv_rank"])
        self.eps = float(p["eps"])
        self.scale = float(p["scale"])
        self.window = int(p["window"]) if p.get("window") else None
        self.q_rank = int(p["q_rank"]) if p.get("q_rank") else 0
        self.sink = bool(p.get("sink", False))
        self.gate = p.get("gate", "head_sigmoid")
        if self.gate not in ("head_sigmoid", None):
            raise ValueError(f"latent attention: gate {self.gate!r} is not 'head_sigmoid' or None")
        if min(self.heads, self.dim, self.vdim, self.rank) < 1 or self.rot_dim < 0:
            raise ValueError("latent attention: heads, dim, vdim and kv_rank are at least 1 and rot_dim is not negative")
        if self.rank > MAX_LATENT or self.rank + self.rot_dim > MAX_LATENT_KEY:
            raise ValueError(f"latent attention: kv_rank {self.rank} with rot_dim {self.rot_dim}; the attention kernels take a latent of at "
                             f"most {MAX_LATENT} and at most {MAX_LATENT_KEY} with the rotated part")
        if not self.scale > 0.0:
            raise ValueError(f"latent attention: the softmax scale must be positive, not {self.scale}")
        self.position = build_part("position", p.get("position") or PartSpec("none"), ctx)
        self.pairing = ops.ROPE_HALVES if self.position.rotation()[1] and self.position.pairing == "halves" else ops.ROPE_INTERLEAVED
        if self.position.rotation()[1] > self.rot_dim:
            raise ValueError(f"latent attention: {self.position.rotation()[1]} rotated dims do not fit the rotated part of {self.rot_dim}")
        self.q_width = self.heads * (self.dim + self.rot_dim)
        self.down_width = self.rank + self.rot_dim
        self.gate_width = self.heads if self.gate else 0
        # the fused in-projection: queries (or their latent) | latent and key part | gate
        self.first_width = self.q_rank or self.q_width
        # without a gate the heads' rows lie row by row, so that the last grouped product stores what the output projection reads
        self.row_major = self.gate is None
        self.sink_logits = None
        self.w_in = self.w_o = self.latent_norm = self.q_norm = self.w_uq = self.w_uk_t = self.w_uv = None

    def _matrix_cores(self) -> bool:
        """Whether this engine's steps run the attention on the matrix cores, which read the latents once more, transposed."""
        page = self.ctx.page_tokens
        return bool(page) and self.ctx.device.type == "cuda" \
            and ops.latent_attention_mfma_ok(self.ctx.act_dtype, self.rank, self.rot_dim, page, ops.latent_cache_width(self.rank, self.rot_dim))

    def cache_need(self):
        cores = self._matrix_cores()
        # a page: [tokens, kv_rank + rot_dim], padded for the matrix cores with zeros that nothing ever writes
        width = ops.latent_cache_width(self.rank, self.rot_dim) if cores else self.down_width
        tensors = [CacheTensor("latent", (width,), None, 0)]
        if cores:
            tensors.append(CacheTensor("latent_t", (self.rank,), None, 1))     # the latents once more: [kv_rank, tokens]
        return PagedNeed(tuple(tensors), self.window)

    def tensor_specs(self, available):
        E, q, d, g = self.hidden, self.first_width, self.down_width, self.gate_width
        fused, shape = self.name("in"), (q + d + g, E)      # one product for the projections that read h: q (or dq) | dkv | g
        specs = [TensorSpec(self.name("dq" if self.q_rank else "q"), (q, E), into=(fused, shape, (slice(0, q),))),
                 TensorSpec(self.name("dkv"), (d, E), into=(fused, shape, (slice(q, q + d),))),
                 TensorSpec(self.name("dkv.norm"), (self.rank,), "norm"),
                 TensorSpec(self.name("uk"), (self.heads * self.dim, self.rank)),
                 TensorSpec(self.name("uv"), (self.heads * self.vdim, self.rank)),
                 TensorSpec(self.name("o"), (E, self.heads * self.vdim))]
        if self.q_rank:
            specs += [TensorSpec(self.name("dq.norm"), (self.q_rank,), "norm"), TensorSpec(self.name("uq"), (self.q_width, self.q_rank))]
        if self.sink:
            specs.append(TensorSpec(self.name("sink"), (self.heads,), "bias", dtype="float32", init=("uniform", -1.0, 1.0)))
        if g:
            specs.append(TensorSpec(self.name("g"), (g, E), into=(fused, shape, (slice(q + d, q + d + g),))))
        return specs

    def load(self, tensors):
        self.w_in = tensors[self.name("in")]
        self.w_o = tensors[self.name("o")]
        self.latent_norm = tensors[self.name("dkv.norm")]
        if self.sink:
            self.sink_logits = tensors[self.name("sink")]
        if self.q_rank:
            self.q_norm, self.w_uq = tensors[self.name("dq.norm")], tensors[self.name("uq")]
        # q_lat = W_uk,n^T q_plain: the grouped product wants each head's matrix as [out = kv_rank, in = dim]
        self.w_uk_t = tensors[self.name("uk")].view(self.heads, self.dim, self.rank).transpose(1, 2).contiguous()
        self.w_uv = tensors[self.name("uv")].view(self.heads, self.vdim, self.rank)

    def _groups(self, step):
        return ops.head_groups(self.heads, step.rows, step.device, self.row_major)

    def _plan(self, step):
        if not self._matrix_cores():
            return None
        window = self.window or 0
        return step.shared(("latent.plan", self.heads, window), lambda: ops.latent_plan(
            [e.n for e in step.entries], self.heads, step.device, contexts=[e.past + e.n for e in step.entries], window=window))

    def graph_key(self, step):
        # a recorded step reads the groups' lists and the plan's items; the key keeps them alive
        return self._groups(step), self._plan(step)

    def takes_deferred_norm(self, step):
        return ops.gemm_takes_normed_rows(step.rows, self.w_in, torch.float32)

    def forward(self, step, h, out, accumulate, cache: LayerCache, h32=None):
        T, H, act = step.rows, self.heads, step.act_dtype
        lead = (T, H) if self.row_major else (H, T)
        proj = step.buf("latent.proj", (T, self.first_width + self.down_width + self.gate_width), torch.float32)
        ops.gemm(h, self.w_in, proj, scratch=step.buf)
        q_plain = step.buf("latent.q_plain", (*lead, self.dim), act)
        q_rot = step.buf("latent.q_rot", (*lead, self.rot_dim), act)
        latents = cache.tensors["latent"]
        cache_t = cache.tensors.get("latent_t")
        tables = step.tables(cache.group)
        cos_sin = self.position.rotation()[0]
        if self.q_rank:
            c_q = step.buf("latent.c_q", (T, self.q_rank), act)
            ops.latent_down(proj, self.q_norm, c_q, self.latent_norm, cos_sin, step.positions, step.row_entry, tables, latents, self.eps,
                            self.q_rank, self.rot_dim, self.rank, write_cache=cache.writes, cache_t=cache_t, pairing=self.pairing)
            q = step.buf("latent.q", (T, self.q_width), torch.float32)
            ops.gemm(c_q, self.w_uq, q, scratch=step.buf)
            ops.latent_queries(q, cos_sin, step.positions, q_plain, q_rot, H, self.dim, self.rot_dim, self.pairing, self.row_major)
        else:
            ops.latent_prep(proj, self.latent_norm, cos_sin, step.positions, step.row_entry, tables, q_plain, q_rot, latents, self.eps, H,
                            self.dim, self.rot_dim, self.rank, write_cache=cache.writes, cache_t=cache_t, pairing=self.pairing,
                            row_major=self.row_major)
        offsets, pairs, active, n_active = self._groups(step)
        q_lat = step.buf("latent.q_lat", (*lead, self.rank), act)
        ops.grouped_gemm(q_plain.view(H * T, self.dim), self.w_uk_t, q_lat.view(H * T, self.rank), offsets, pairs, 1, ops.EPI_STORE,
                         active, n_active, token_rows=T)
        mixed = step.buf("latent.mixed", (*lead, self.rank), act)
        ops.latent_attention(q_lat, q_rot, latents, step.positions, step.row_entry, tables, mixed, self.scale, window=self.window or 0,
                             scratch=step.buf, cache_t=cache_t, plan=self._plan(step), row_major=self.row_major, sink=self.sink_logits)
        joined = step.buf("latent.joined", (T, H * self.vdim), act)
        values = joined.view(H * T, self.vdim) if self.row_major else step.buf("latent.values", (H * T, self.vdim), torch.float32)
        ops.grouped_gemm(mixed.view(H * T, self.rank), self.w_uv, values, offsets, pairs, 1, ops.EPI_STORE, active, n_active, token_rows=T)
        if not self.row_major:
            ops.head_gate(values.view(H, T, self.vdim), proj[:, self.first_width + self.down_width:], joined)
        ops.gemm(joined, self.w_o, out, ops.EPI_ADD if accumulate else ops.EPI_STORE, scratch=step.buf)


register("mixer", "latent_attention", LatentAttention)
