"""Neruzen assembled from parts.

A bigram embedding (the token's row plus a row of a second table chosen by the token and the one before); per layer the
"parallel" arrangement with one RMS norm, h = norm1(x), x += mixer(shift(h)) + ff(h): a mixer of token-shifted rows among
latent attention over a window (queries through a latent of their own, halved rotary pairs, no gate), linear attention with
constant decays over silu projections (one norm over all heads, a sigmoid gate) and over rotated queries and keys (unit-RMS
heads, a silu gate); routed silu-gated experts picked by groups (softmax scores, weights normalized) beside a shared expert,
or no feed-forward; a final RMS norm and an untied head.
Tensor names: embed, bigram, l<i>.norm1, l<i>.shift, l<i>.mix.*, l<i>.mlp.*, final.norm, head.
"""

from __future__ import annotations

from ..config.neruzen import ARCHITECTURE, NeruzenConfig
from ..parts.spec import BlockSpec, ModelSpec, PartSpec, RunEntry
from .registry import register_architecture

NO_POSITION_LIMIT = 1 << 30     # the design states no longest context: the cache's size is the limit

_EXPERT_NAMES = {"router": "router", "expert_gate": "e{e}.gate", "expert_up": "e{e}.up", "expert_down": "e{e}.down",
                 "fused_gate_up": "gate_up", "fused_down": "down", "shared_gate": "shared.gate", "shared_up": "shared.up",
                 "shared_down": "shared.down"}


def _rotation(rot) -> PartSpec:
    return PartSpec("rotary_scaled", {"dims": rot.dims, "base": rot.base, "pairing": "halves", "exact_angles": True})


def _mixer(c: NeruzenConfig, i: int) -> PartSpec:
    layer = c.layers[i]
    m, p = layer.mixer, f"l{i}.mix."
    common = {"hidden": c.width, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "eps": c.norm_eps}
    if layer.type == "latent_attention":
        return PartSpec("latent_attention", dict(common, rot_dim=m.rot_dim, q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, gate=None,
                                                 position=_rotation(m.rot), window=m.window), p)
    if layer.type == "lightning":
        return PartSpec("decayed_linear_attention", dict(common, decay=m.decay, operands="silu", norm="joint", gate="sigmoid"), p)
    return PartSpec("decayed_linear_attention", dict(common, decay=m.decay, operands="rotated", position=_rotation(m.rot),
                                                     key_scale=float(m.dim) ** -0.5, norm="head", gate="silu"), p)


def assemble(c: NeruzenConfig) -> ModelSpec:
    E = c.width

    def norm(name):
        return PartSpec("rmsnorm", {"width": E, "eps": c.norm_eps, "tensor": ""}, name)

    blocks = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        ffn = None
        if layer.mlp is not None:
            m = layer.mlp
            ffn = PartSpec("routed_experts", {"hidden": E, "experts": m.experts, "top_k": m.top, "intermediate": m.ff, "score": "softmax",
                                              "normalize": "always", "groups": {"count": m.group_count, "keep": m.group_keep}, "unit": "swiglu",
                                              "shared": None if m.shared_ff is None else {"intermediate": m.shared_ff},
                                              "names": _EXPERT_NAMES, "files": "per_expert"}, p + "mlp.")
        # one norm: the feed-forward has none of its own and reads the rows that the mixer's shift starts from
        mixer = PartSpec("token_shift", {"hidden": E, "mixer": _mixer(c, i)}, p + "shift")
        blocks.append(BlockSpec(mixer_norm=norm(p + "norm1"), mixer=mixer, ffn_norm=None, ffn=ffn, arrangement="parallel"))
    b = c.bigram
    return ModelSpec(
        architecture=ARCHITECTURE,
        vocab_size=c.vocab,
        hidden_size=E,
        max_positions=NO_POSITION_LIMIT,
        embedding=PartSpec("bigram_embedding", {"vocab": c.vocab, "hidden": E, "tensor": "",
                                                "bigram": {"tensor": "bigram", "buckets": b.buckets, "mul_prev": b.mul_prev, "mul_cur": b.mul_cur}}, "embed"),
        blocks=blocks,
        run_order=[RunEntry(layer=i, cache=i) for i in range(len(blocks))],
        final_norm=norm("final.norm"),
        head=PartSpec("linear", {"vocab": c.vocab, "hidden": E, "tied": False, "tensor": ""}, "head"),
    )


register_architecture(ARCHITECTURE, NeruzenConfig, assemble, replace=True)
