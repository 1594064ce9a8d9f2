"""What a mixer reads of the residual stream, mixed channel by channel with the previous token's row:

    shift(x)_t = x_t + (x_(t-1) - x_t) * mu        (zeros before a sequence's start)

mu [hidden].  The previous row is the stream's own (float32, before the mixing); the last row that a request brought is its
state, so a prompt may be cut anywhere.  It is a part of a layer like a mixer (it owns state), but what it makes is read by
the mixer: it is laid down as a reader of the stream, where other arrangements have a norm (`plan.normed`).
"""
from __future__ import annotations

from typing import List, Sequence

from ..cache.needs import StateNeed
from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import Mixer, Runtime, register_mixer

SHIFT_STATE = "token_shift"


@register_mixer("token_shift")
class TokenShift(Mixer):
    def state_needs(self) -> Sequence[StateNeed]:
        return (StateNeed(SHIFT_STATE, (self.hidden,)),)

    def tensor_decls(self) -> List[TensorDecl]:
        return [TensorDecl(self.spec.tensors["mu"], (self.hidden,), FLOAT32, init="unit")]

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        self.mu = weights[self.spec.tensors["mu"]].contiguous()

    def small_tensors(self):
        return [self.mu]

    def state_bytes(self) -> int:
        return 2 * 4 * self.hidden

    def emit(self, plan, cache) -> int:
        """-> the number of a reader of the stream (to be used as a norm's)."""
        return plan.shifted_rows(mu=self.mu, state=cache.states[SHIFT_STATE])
