"""A mixer that reads token-shifted rows.

    shifted_t = h_t + (h_(t-1) - h_t) * s        element by element; h_(-1) = 0 before a request's first token
    result = mixer(shifted)

h are the normed rows as the norm gives them (unrounded), s one learned factor a coordinate.  The last h of a request is part
of its state (float32), beside whatever the wrapped mixer keeps: the engine sees a composite need.
"""

from __future__ import annotations

import torch

from .. import ops
from .base import LayerCache, Mixer, Part, build_part, register
from .norm import RMSNorm
from .spec import CompositeNeed, StateNeed, TensorSpec


class TokenShift(Part):
    """The factors and the state of a shift.  Tensor: the prefix itself, (hidden,)."""
    graph_safe = True
    steps_between_slots = True      # reads the state at step.entry_held_slots, writes it at step.entry_slots

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.hidden = int(params["hidden"])
        self.weight = None

    def cache_need(self):
        return StateNeed((self.hidden,), "float32")

    def tensor_specs(self, available):
        return [TensorSpec(self.prefix, (self.hidden,), "norm", init=("uniform", 0.0, 1.0))]

    def load(self, tensors):
        self.weight = tensors[self.prefix]


class ShiftedMixer(Mixer):
    """params: hidden, mixer (PartSpec); the prefix is the shift's tensor name.  A built model lists the wrapped mixer and the
    shift as parts of their own after this one (`members()`).  An arrangement whose norm is an RMS norm may run the norm and the
    shift in one launch (`normed_and_shifted`) and hand the wrapped mixer its rows itself (`inner`)."""
    graph_safe = True
    wants_f32_input = True
    steps_between_slots = True      # the members say so themselves

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.hidden = int(params["hidden"])
        self.inner = build_part("mixer", params["mixer"], ctx)
        if self.inner.wants_f32_input:
            raise ValueError("token shift: the wrapped mixer reads rows in the activation type")
        self.shift = TokenShift({"hidden": self.hidden}, prefix, ctx)
        self.graph_safe = bool(getattr(self.inner, "graph_safe", False))

    def members(self):
        return [self.inner, self.shift]

    def cache_need(self):
        return CompositeNeed((self.inner.cache_need(), self.shift.cache_need()))

    def fuses(self, norm) -> bool:
        return isinstance(norm, RMSNorm)

    def normed_and_shifted(self, step, norm: RMSNorm, x, cache: LayerCache, out=None, out32=None) -> torch.Tensor:
        """The shifted rows of h = norm(x) in the activation type; `out` / `out32` receive h itself."""
        shifted = step.buf("shift.rows", tuple(x.shape), step.act_dtype)
        ops.token_shift(x, self.shift.weight, cache.members[1].state, step.entry_held_slots, step.entry_slots, step.row_entry, step.entry_rows,
                        shifted, norm=(norm.weight, norm.eps), out=out, out32=out32)
        return shifted

    def forward(self, step, h, out, accumulate, cache: LayerCache, h32=None):
        shifted = step.buf("shift.rows", tuple(h32.shape), step.act_dtype)
        ops.token_shift(h32, self.shift.weight, cache.members[1].state, step.entry_held_slots, step.entry_slots, step.row_entry, step.entry_rows, shifted)
        self.inner.forward(step, shifted, out, accumulate, cache.members[0])


register("mixer", "token_shift", ShiftedMixer)
