"""Vivulorn assembled from parts.

Embedding times a scale; per layer the "prenorm" arrangement with layer norms of weight and bias: a mixer among softmax
attention (norms over the whole q and k projections, YaRN-blended halved rotary pairs, a gate a value), latent attention
(interleaved pairs, a sink a head, no gate) and the gated delta rule with one decay a head, then a dense feed-forward with biases
and the exact gelu, or none.  A run of layers repeats: every pass opens with a product of the residual and the embedding's rows
and has cache numbers of its own.  A final layer norm; the head is the embedding's table, its logits soft-capped.
Tensor names: embed, loop.in, l<i>.norm1, l<i>.norm2 (+ .b), l<i>.mix.*, l<i>.mlp.up, .down (+ .b), final.norm (+ .b).
"""

from __future__ import annotations

from ..config.vivulorn import ARCHITECTURE, VivulornConfig
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, RunEntry
from .registry import register_architecture

NO_POSITION_LIMIT = 1 << 30     # the design states no longest context: the cache's size is the limit

_ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "output_gate": "g"}


def _mixer(c: VivulornConfig, i: int) -> PartSpec:
    layer = c.layers[i]
    m, p = layer.mixer, f"l{i}.mix."
    if layer.type == "attention":
        s = m.rot_scaling
        position = PartSpec("rotary_scaled", {"dims": m.rot_dims, "base": m.rot_base, "pairing": "halves", "exact_angles": True,
                                              "scaling": None if s is None else {"factor": s.factor, "original": s.original, "fast": s.fast,
                                                                                 "slow": s.slow}})
        return PartSpec("attention", {"hidden": c.width, "heads": m.heads, "kv_heads": m.kv_heads, "head_dim": m.dim, "v_dim": m.vdim,
                                      "qk_norm": "projection", "eps": c.norm_eps, "scale": m.scale, "output_gate": True, "position": position,
                                      "names": _ATTENTION_NAMES}, p)
    if layer.type == "latent_attention":
        position = PartSpec("rotary_scaled", {"dims": m.rot_dim, "base": m.rot_base, "pairing": "interleaved", "exact_angles": True})
        return PartSpec("latent_attention", {"hidden": c.width, "heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim,
                                             "kv_rank": m.kv_rank, "scale": m.scale, "eps": c.norm_eps, "gate": None, "sink": True,
                                             "position": position, "window": None}, p)
    return PartSpec("head_delta_rule", {"hidden": c.width, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
                                        "conv": m.conv, "eps": c.norm_eps}, p)


def assemble(c: VivulornConfig) -> ModelSpec:
    E = c.width

    def norm(name):
        return PartSpec("layernorm", {"width": E, "eps": c.norm_eps, "tensor": "", "bias": ".b"}, name)

    blocks = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        ffn = ffn_norm = None
        if layer.ff is not None:
            ffn_norm = norm(p + "norm2")
            ffn = PartSpec("dense_act", {"hidden": E, "intermediate": layer.ff, "activation": "gelu"}, p + "mlp.")
        blocks.append(BlockSpec(mixer_norm=norm(p + "norm1"), mixer=_mixer(c, i), ffn_norm=ffn_norm, ffn=ffn, arrangement="prenorm"))
    return ModelSpec(
        architecture=ARCHITECTURE,
        vocab_size=c.vocab,
        hidden_size=E,
        max_positions=NO_POSITION_LIMIT,
        embedding=PartSpec("token_embedding", {"vocab": c.vocab, "hidden": E, "scale": c.embedding_scale, "tensor": ""}, "embed"),
        blocks=blocks,
        run_order=[RunEntry(layer=i, cache=n, before=0 if opens else None) for n, (i, opens) in enumerate(c.passes())],
        final_norm=norm("final.norm"),
        head=PartSpec("linear", {"vocab": c.vocab, "hidden": E, "tied": True, "softcap": c.logit_softcap}, "head"),
        inputs=[PartSpec("pass_projection", {"hidden": E}, "loop.in")] if c.loop is not None else [],
    )


register_architecture(ARCHITECTURE, VivulornConfig, assemble, replace=True)
