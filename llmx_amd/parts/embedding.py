"""Token embedding and the language-model head.

x[t] = table[id[t]] widened to float32, times the embedding's scale where the model has one (/root/reference/src/model/arch/blocks.hpp:95-97); logits = rows . W^T in
float32 for the wanted rows only (:267-272).  A tied head reads the embedding's table.  A bigram embedding adds a second
table's row, chosen by the token and the one before it.
"""

from __future__ import annotations

import torch

from .. import ops
from .base import Embedding, Head, LayerCache, register
from .spec import StateNeed, TensorSpec


class TokenEmbedding(Embedding):
    """params: vocab, hidden; scale (the rows are multiplied by it, 1 by default); tensor (the name's last part, "weight"
    by default); side_tables: {full tensor name: width}, further tables with a row a token that other parts read by
    name (a part of each layer's own token input, for instance): the embedding lists them, once for the model.
    Tensor <prefix><tensor> (vocab, hidden)."""
    graph_safe = True

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.vocab = int(params["vocab"])
        self.hidden = int(params["hidden"])
        self.scale = float(params.get("scale", 1.0))
        self.tensor = str(params.get("tensor", "weight"))
        self.side_tables = {str(k): int(v) for k, v in (params.get("side_tables") or {}).items()}
        self.weight = None

    def tensor_specs(self, available):
        return [TensorSpec(self.name(self.tensor), (self.vocab, self.hidden), "table")] + \
               [TensorSpec(name, (self.vocab, width), "table") for name, width in self.side_tables.items()]

    def load(self, tensors):
        self.weight = tensors[self.name(self.tensor)]

    def table(self):
        return self.weight

    def forward(self, step, out):
        ops.embed_gather(self.weight, step.token_ids, out, self.scale)


class BigramEmbedding(TokenEmbedding):
    """A token embedding with a second table's row added: row (previous token * mul_prev + token * mul_cur) mod buckets, and the
    table's last row for a request's first token.  params: those of TokenEmbedding, and bigram {tensor (its full name), buckets,
    mul_prev, mul_cur}.  Tensors: the embedding's, and <bigram tensor> (buckets + 1, hidden).  State: the last token."""
    steps_between_slots = True      # reads the state at step.entry_held_slots, writes it at step.entry_slots

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        b = params["bigram"]
        self.bigram_name = str(b["tensor"])
        self.buckets, self.mul_prev, self.mul_cur = int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])
        if self.buckets < 1:
            raise ValueError("bigram embedding: at least one bucket")
        self.bigram = None

    def cache_need(self):
        return StateNeed((1,), "int32")

    def tensor_specs(self, available):
        return super().tensor_specs(available) + [TensorSpec(self.bigram_name, (self.buckets + 1, self.hidden), "table")]

    def load(self, tensors):
        super().load(tensors)
        self.bigram = tensors[self.bigram_name]

    def forward(self, step, out, cache: LayerCache):
        ops.embed_bigram(self.weight, self.bigram, step.token_ids, cache.state, step.entry_held_slots, step.entry_slots, step.row_entry,
                         step.entry_rows, out, self.buckets, self.mul_prev, self.mul_cur, self.scale)


class LinearHead(Head):
    """params: vocab, hidden, tied (bool); tensor (the name's last part, "weight" by default); logit_scale (the logits are
    multiplied by it, 1 by default) and softcap (c > 0: logits <- c tanh(logits / c), after the scale; None: none).
    Tensor <prefix><tensor> (vocab, hidden) unless tied."""
    graph_safe = True

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.vocab = int(params["vocab"])
        self.hidden = int(params["hidden"])
        self.tied = bool(params.get("tied", False))
        self.tensor = str(params.get("tensor", "weight"))
        self.logit_scale = float(params.get("logit_scale", 1.0))
        self.softcap = float(params["softcap"]) if params.get("softcap") else 0.0
        if self.softcap < 0.0:
            raise ValueError("head: a softcap is positive")
        self.weight = None

    def tensor_specs(self, available):
        return [] if self.tied else [TensorSpec(self.name(self.tensor), (self.vocab, self.hidden), "table")]

    def load(self, tensors):
        if not self.tied:
            self.weight = tensors[self.name(self.tensor)]

    def tie(self, table: torch.Tensor) -> None:
        self.weight = table

    def forward(self, step, rows, logits):
        ops.gemm(rows, self.weight, logits)
        if self.logit_scale != 1.0 or self.softcap > 0.0:
            ops.scale_softcap(logits, self.logit_scale, self.softcap)


register("embedding", "token_embedding", TokenEmbedding)
register("embedding", "bigram_embedding", BigramEmbedding)
register("head", "linear", LinearHead)
