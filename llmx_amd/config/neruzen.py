"""Neruzen's typed configuration, read from its own config.json keys.

A decoder whose layers are listed one by one.  A layer has one RMS norm; its feed-forward reads the normed rows, its mixer the
same rows token-shifted, and both results join the residual.  The mixer is "latent_attention" (softmax attention over a
sliding window of cached latents, queries through a latent of their own), "lightning" (linear attention over silu projections
with a constant decay a head, one norm over all heads, a sigmoid gate) or "retention" (linear attention over rotated queries
and keys with a constant decay a head, unit-RMS heads, a silu gate); the feed-forward is routed experts of gated units picked
by groups, beside a shared expert, or absent.  A second embedding table is indexed by the token and the one before it.
config.json gives every size and every constant that differs between models of the design:

  architecture "Neruzen"; vocab; width; norm.eps; embedding.bigram {buckets, mul_prev, mul_cur}; layers[]: type, mixer
  (latent_attention: heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, mask {size}, rot {base, dims};
   lightning: heads, dim, vdim, decay [a number a head]; retention: the same and rot {base, dims}),
  mlp (null | {kind "moe", expert {ff}, router {experts, top, groups {count, keep} (optional)}, shared {ff} (optional)}).
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional, Tuple

from ..limits import MAX_EXPERTS, MAX_TOP_K
from .reader import ConfigError, KeyReader

ARCHITECTURE = "Neruzen"
#: keys a model folder's config.json may carry that say nothing about the arithmetic
WITHOUT_EFFECT = ("name", "seed", "comment", "description", "dtype", "torch_dtype")
LAYER_TYPES = ("latent_attention", "lightning", "retention")
MAX_STATE_DIM = 256     # key channels of a head that the recurrence's kernels keep in registers


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int


@dataclass(frozen=True)
class BigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int
    rot: Rotation


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Rotation


@dataclass(frozen=True)
class ExpertsConfig:
    ff: int
    experts: int
    top: int
    group_count: int = 1
    group_keep: int = 1
    shared_ff: Optional[int] = None     # None: no shared expert


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any                          # LatentAttentionConfig | LightningConfig | RetentionConfig
    mlp: Optional[ExpertsConfig] = None


@dataclass(frozen=True)
class NeruzenConfig:
    vocab: int
    width: int
    norm_eps: float
    bigram: BigramConfig
    layers: Tuple[LayerConfig, ...]

    architecture = ARCHITECTURE

    def __post_init__(self):
        object.__setattr__(self, "layers", tuple(self.layers))
        check(self)

    @classmethod
    def from_json(cls, values: Mapping[str, Any]) -> "NeruzenConfig":
        r = KeyReader(values)
        name = r.raw("architecture")
        if name != ARCHITECTURE:
            raise r.unsupported("architecture", f"{name!r}; expected {ARCHITECTURE!r}")
        norm = r.child("norm")
        eps = norm.real("eps", lo=0.0)
        norm.finish((), ARCHITECTURE)
        embedding = r.child("embedding")
        b = embedding.child("bigram")
        bigram = BigramConfig(buckets=b.integer("buckets"), mul_prev=b.integer("mul_prev", lo=0, hi=1 << 62),
                              mul_cur=b.integer("mul_cur", lo=0, hi=1 << 62))
        b.finish((), ARCHITECTURE)
        embedding.finish((), ARCHITECTURE)
        raw_layers = r.raw("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise r.unsupported("layers", "a list of at least one layer is expected")
        layers = tuple(_read_layer(entry, i) for i, entry in enumerate(raw_layers))
        cfg = cls(vocab=r.integer("vocab"), width=r.integer("width"), norm_eps=eps, bigram=bigram, layers=layers)
        r.finish(WITHOUT_EFFECT, ARCHITECTURE)
        return cfg

    @property
    def vocab_size(self) -> int:
        """The vocabulary under the name the command line asks every configuration for."""
        return self.vocab

    def to_json(self) -> dict:
        b = self.bigram
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"bigram": {"buckets": b.buckets, "mul_prev": b.mul_prev, "mul_cur": b.mul_cur}},
                "layers": [_layer_json(layer) for layer in self.layers]}


def _read_rotation(m: KeyReader) -> Rotation:
    rot = m.child("rot")
    out = Rotation(base=rot.real("base", positive=True), dims=rot.integer("dims", lo=0))
    rot.finish((), ARCHITECTURE)
    return out


def _read_decay(m: KeyReader) -> Tuple[float, ...]:
    decay = m.raw("decay")
    if not isinstance(decay, list) or not all(isinstance(g, (int, float)) and not isinstance(g, bool) for g in decay):
        raise m.unsupported("decay", "a list of numbers, one a head")
    return tuple(float(g) for g in decay)


def _read_mixer(kind: str, m: KeyReader):
    if kind == "latent_attention":
        mask = m.child("mask")
        window = mask.integer("size")
        mask.finish((), ARCHITECTURE)
        return LatentAttentionConfig(heads=m.integer("heads"), dim=m.integer("dim"), rot_dim=m.integer("rot_dim", lo=0), vdim=m.integer("vdim"),
                                     q_rank=m.integer("q_rank"), kv_rank=m.integer("kv_rank"), scale=m.real("scale", positive=True), window=window,
                                     rot=_read_rotation(m))
    sizes = dict(heads=m.integer("heads"), dim=m.integer("dim"), vdim=m.integer("vdim"), decay=_read_decay(m))
    return LightningConfig(**sizes) if kind == "lightning" else RetentionConfig(rot=_read_rotation(m), **sizes)


def _read_experts(mlp: KeyReader) -> ExpertsConfig:
    mlp.choice("kind", ("moe",))
    expert, router = mlp.child("expert"), mlp.child("router")
    groups, shared = router.child("groups", required=False), mlp.child("shared", required=False)
    out = ExpertsConfig(ff=expert.integer("ff"), experts=router.integer("experts"), top=router.integer("top"),
                        group_count=1 if groups is None else groups.integer("count"), group_keep=1 if groups is None else groups.integer("keep"),
                        shared_ff=None if shared is None else shared.integer("ff"))
    for part in (expert, router, groups, shared, mlp):
        if part is not None:
            part.finish((), ARCHITECTURE)
    return out


def _read_layer(entry, i: int) -> LayerConfig:
    r = KeyReader(entry, where=f"layers[{i}]")
    kind = r.choice("type", LAYER_TYPES)
    m = r.child("mixer")
    mixer = _read_mixer(kind, m)
    m.finish((), ARCHITECTURE)
    mlp = r.child("mlp", required=False)
    ff = None if mlp is None else _read_experts(mlp)
    r.finish(("name", "comment"), ARCHITECTURE)
    return LayerConfig(kind, mixer, ff)


def _layer_json(layer: LayerConfig) -> dict:
    a = layer.mixer
    mixer = {"heads": a.heads, "dim": a.dim, "vdim": a.vdim}
    if layer.type == "latent_attention":
        mixer.update({"rot_dim": a.rot_dim, "q_rank": a.q_rank, "kv_rank": a.kv_rank, "scale": a.scale, "mask": {"size": a.window}})
    else:
        mixer["decay"] = list(a.decay)
    if layer.type != "lightning":
        mixer["rot"] = {"base": a.rot.base, "dims": a.rot.dims}
    m = layer.mlp
    mlp = None
    if m is not None:
        mlp = {"kind": "moe", "expert": {"ff": m.ff},
               "router": {"experts": m.experts, "top": m.top, "groups": {"count": m.group_count, "keep": m.group_keep}}}
        if m.shared_ff is not None:
            mlp["shared"] = {"ff": m.shared_ff}
    return {"type": layer.type, "mixer": mixer, "mlp": mlp}


def check(c: NeruzenConfig) -> None:
    """The rules a configuration keeps wherever it came from."""
    def bad(key, why):
        return ConfigError(f"config: unsupported value for {key} ({why})")

    def rotation(where, rot, dim, of):
        if rot.dims % 2 or not 0 <= rot.dims <= dim:
            raise bad(f"{where}.rot.dims", f"the rotated dims are even and at most {of}")
        if rot.base <= 0.0:
            raise bad(f"{where}.rot.base", "positive")

    if c.vocab < 1 or c.width < 1:
        raise bad("width", "vocab and width are at least 1")
    if not 0 < c.bigram.buckets < (1 << 31) or c.bigram.mul_prev < 0 or c.bigram.mul_cur < 0:
        raise bad("embedding.bigram", "between 1 and 2^31 - 1 buckets and no negative multiplier")
    if not c.layers:
        raise bad("layers", "at least one layer")
    for i, layer in enumerate(c.layers):
        where = f"layers[{i}]"
        if layer.type not in LAYER_TYPES:
            raise bad(f"{where}.type", f"{layer.type!r}; this engine computes {list(LAYER_TYPES)}")
        a = layer.mixer
        want = {"latent_attention": LatentAttentionConfig, "lightning": LightningConfig, "retention": RetentionConfig}[layer.type]
        if not isinstance(a, want):
            raise bad(f"{where}.mixer", f"not the sizes of a mixer of type {layer.type!r}")
        if layer.type == "latent_attention":
            rotation(f"{where}.mixer", a.rot, a.rot_dim, "rot_dim")
            if a.window < 1:
                raise bad(f"{where}.mixer.mask.size", "at least 1")
        else:
            if a.dim > MAX_STATE_DIM:
                raise bad(f"{where}.mixer.dim", f"at most {MAX_STATE_DIM}")
            if len(a.decay) != a.heads or not all(0.0 <= g <= 1.0 for g in a.decay):
                raise bad(f"{where}.mixer.decay", "a number between 0 and 1 for every head")
            if layer.type == "retention":
                rotation(f"{where}.mixer", a.rot, a.dim, "dim")
        m = layer.mlp
        if m is None:
            continue
        if m.ff < 1 or (m.shared_ff is not None and m.shared_ff < 1):
            raise bad(f"{where}.mlp", "inner widths of at least 1")
        if not 0 < m.top <= m.experts:
            raise bad(f"{where}.mlp.router.top", "between 1 and the expert count")
        if m.experts > MAX_EXPERTS or m.top > MAX_TOP_K:
            raise bad(f"{where}.mlp.router", f"at most {MAX_EXPERTS} experts and {MAX_TOP_K} picks")
        if m.group_count < 1 or m.experts % m.group_count:
            raise bad(f"{where}.mlp.router.groups.count", "the experts form equal groups")
        if not 0 < m.group_keep <= m.group_count or m.top > m.group_keep * (m.experts // m.group_count):
            raise bad(f"{where}.mlp.router.groups.keep", "between 1 and the group count, with enough experts for the picks")
