"""Vivulorn's typed configuration, read from its own config.json keys.

A decoder whose layers are listed one by one, each with a mixer ("delta": a gated delta rule with one decay a head;
"latent_attention": attention over one cached latent a token, with a sink a head; "attention": softmax attention with norms over
whole projections, YaRN-blended rotation and a gate a value) and a dense feed-forward or none.  A run of layers is repeated with
the same weights, every pass with a cache of its own.  config.json gives every size and every constant that differs between
models of the design:

  architecture "Vivulorn"; vocab; width; norm.eps; embedding.scale; logit_softcap; layers[]: type, mixer (attention: heads,
  kv_heads, dim, vdim, scale, rot {base, dims, scaling {factor, original, fast, slow}}; latent_attention: heads, dim, rot_dim,
  vdim, kv_rank, scale, rot {base, dims}; delta: heads, kv_heads, dim, vdim, conv), mlp (null | {kind "dense", ff});
  loop {start, stop, times}.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .nenotar import RotaryScaling
from .reader import ConfigError, KeyReader

ARCHITECTURE = "Vivulorn"
#: keys a model folder's config.json may carry that say nothing about the arithmetic
WITHOUT_EFFECT = ("name", "seed", "comment", "description", "dtype", "torch_dtype")
LAYER_TYPES = ("attention", "latent_attention", "delta")


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    rot_scaling: Optional[RotaryScaling] = None


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: Any                      # AttentionConfig | LatentAttentionConfig | DeltaConfig
    ff: Optional[int] = None        # the dense feed-forward's inner width; None: the layer has none


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class VivulornConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: Tuple[LayerConfig, ...]
    loop: Optional[LoopConfig] = None
    logit_softcap: Optional[float] = None

    architecture = ARCHITECTURE

    def __post_init__(self):
        object.__setattr__(self, "layers", tuple(self.layers))
        check(self)

    @classmethod
    def from_json(cls, values: Mapping[str, Any]) -> "VivulornConfig":
        r = KeyReader(values)
        name = r.raw("architecture")
        if name != ARCHITECTURE:
            raise r.unsupported("architecture", f"{name!r}; expected {ARCHITECTURE!r}")
        norm, embedding = r.child("norm"), r.child("embedding", required=False)
        eps = norm.real("eps", lo=0.0)
        scale = embedding.real("scale", default=1.0) if embedding is not None else 1.0
        norm.finish((), ARCHITECTURE)
        if embedding is not None:
            embedding.finish((), ARCHITECTURE)
        raw_layers = r.raw("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise r.unsupported("layers", "a list of at least one layer is expected")
        layers = tuple(_read_layer(entry, i) for i, entry in enumerate(raw_layers))
        raw_loop = r.child("loop", required=False)
        loop = None
        if raw_loop is not None:
            loop = LoopConfig(start=raw_loop.integer("start", lo=0), stop=raw_loop.integer("stop"), times=raw_loop.integer("times"))
            raw_loop.finish((), ARCHITECTURE)
        cfg = cls(vocab=r.integer("vocab"), width=r.integer("width"), norm_eps=eps, embedding_scale=scale, layers=layers, loop=loop,
                  logit_softcap=r.real("logit_softcap", default=None, positive=True))
        r.finish(WITHOUT_EFFECT, ARCHITECTURE)
        return cfg

    @property
    def vocab_size(self) -> int:
        """The vocabulary under the name the command line asks every configuration for."""
        return self.vocab

    def passes(self) -> List[Tuple[int, bool]]:
        """(layer, whether a pass of the repeated run starts with it), in the order the layers run."""
        if self.loop is None:
            return [(i, False) for i in range(len(self.layers))]
        a, b, times = self.loop.start, self.loop.stop, self.loop.times
        return ([(i, False) for i in range(a)] + [(i, i == a) for _ in range(times) for i in range(a, b)]
                + [(i, False) for i in range(b, len(self.layers))])

    def to_json(self) -> dict:
        out = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "layers": [_layer_json(layer) for layer in self.layers]}
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        return out


def _read_layer(entry, i: int) -> LayerConfig:
    r = KeyReader(entry, where=f"layers[{i}]")
    kind = r.choice("type", LAYER_TYPES)
    m = r.child("mixer")
    if kind == "delta":
        mixer: Any = DeltaConfig(heads=m.integer("heads"), kv_heads=m.integer("kv_heads"), dim=m.integer("dim"), vdim=m.integer("vdim"),
                                 conv=m.integer("conv"))
    elif kind == "attention":
        rot = m.child("rot")
        sc = rot.child("scaling", required=False)
        scaling = None
        if sc is not None:
            scaling = RotaryScaling(factor=sc.real("factor", positive=True), original=sc.real("original", positive=True),
                                    fast=sc.real("fast", positive=True), slow=sc.real("slow", positive=True))
            sc.finish((), ARCHITECTURE)
        mixer = AttentionConfig(heads=m.integer("heads"), kv_heads=m.integer("kv_heads"), dim=m.integer("dim"), vdim=m.integer("vdim"),
                                scale=m.real("scale", positive=True), rot_base=rot.real("base", positive=True),
                                rot_dims=rot.integer("dims", lo=0), rot_scaling=scaling)
        rot.finish((), ARCHITECTURE)
    else:
        rot = m.child("rot")
        mixer = LatentAttentionConfig(heads=m.integer("heads"), dim=m.integer("dim"), rot_dim=m.integer("rot_dim"), vdim=m.integer("vdim"),
                                      kv_rank=m.integer("kv_rank"), scale=m.real("scale", positive=True), rot_base=rot.real("base", positive=True))
        if rot.integer("dims") != mixer.rot_dim:
            raise rot.unsupported("dims", f"the rotated part of {mixer.rot_dim} turns whole")
        rot.held("scaling", None)
        rot.finish((), ARCHITECTURE)
    m.finish((), ARCHITECTURE)
    mlp = r.child("mlp", required=False)
    ff = None
    if mlp is not None:
        mlp.choice("kind", ("dense",))
        ff = mlp.integer("ff")
        mlp.finish((), ARCHITECTURE)
    r.finish(("name", "comment"), ARCHITECTURE)
    return LayerConfig(kind, mixer, ff)


def _layer_json(layer: LayerConfig) -> dict:
    m = layer.mixer
    if layer.type == "delta":
        mixer: Dict[str, Any] = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}
    elif layer.type == "attention":
        rot: Dict[str, Any] = {"base": m.rot_base, "dims": m.rot_dims}
        if m.rot_scaling is not None:
            s = m.rot_scaling
            rot["scaling"] = {"factor": s.factor, "original": s.original, "fast": s.fast, "slow": s.slow}
        mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale, "rot": rot}
    else:
        mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank, "scale": m.scale,
                 "rot": {"base": m.rot_base, "dims": m.rot_dim}}
    return {"type": layer.type, "mixer": mixer, "mlp": None if layer.ff is None else {"kind": "dense", "ff": layer.ff}}


def check(c: VivulornConfig) -> None:
    """The rules a configuration keeps wherever it came from."""
    def bad(key, why):
        return ConfigError(f"config: unsupported value for {key} ({why})")
    if c.vocab < 1 or c.width < 1:
        raise bad("width", "vocab and width are at least 1")
    if not c.layers:
        raise bad("layers", "at least one layer")
    for i, layer in enumerate(c.layers):
        where = f"layers[{i}]"
        if layer.type not in LAYER_TYPES:
            raise bad(f"{where}.type", f"{layer.type!r}; this engine computes {list(LAYER_TYPES)}")
        m = layer.mixer
        expected = {"attention": AttentionConfig, "latent_attention": LatentAttentionConfig, "delta": DeltaConfig}[layer.type]
        if not isinstance(m, expected):
            raise bad(f"{where}.mixer", f"not the sizes of a mixer of type {layer.type!r}")
        if layer.type != "latent_attention" and m.heads % m.kv_heads:
            raise bad(f"{where}.mixer.kv_heads", "the head count must be divisible by it")
        if layer.type == "attention":
            if m.rot_dims % 2 or m.rot_dims > m.dim:
                raise bad(f"{where}.mixer.rot.dims", "the rotated dims are even and at most dim")
            if m.rot_scaling is not None and m.rot_base <= 1.0:
                raise bad(f"{where}.mixer.rot.base", "above 1 where the frequencies are blended")
        elif layer.type == "latent_attention":
            if m.rot_dim % 2:
                raise bad(f"{where}.mixer.rot_dim", "the rotated dims are even")
        elif m.dim > 256:
            raise bad(f"{where}.mixer.dim", "at most 256")
        if layer.ff is not None and layer.ff < 1:
            raise bad(f"{where}.mlp.ff", "at least 1")
    if c.loop is not None and (not 0 <= c.loop.start < c.loop.stop <= len(c.layers) or c.loop.times < 1):
        raise bad("loop", f"a run of layers inside the model's {len(c.layers)}, at least once")
