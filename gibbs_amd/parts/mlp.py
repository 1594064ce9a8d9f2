"""Dense feed-forward without a gate: down(act(up(h))).

`activation: "poly_norm"`: act(z) = a N(z) + b N(z^2) + c N(z^3) + e, powers element by element, N the division of
a token's vector of values by its root mean square (`eps` inside the root), and [a, b, c, e] a tensor of the
checkpoint (`act`).  The three mean squares are float32 sums in either precision of a run.

Other activations have no tensors: one of `ops.ACTIVATIONS`, or "relu_squared", the square of relu.  The up product and its
activation are one kernel in steps of few rows."""
from __future__ import annotations

from typing import List

from .. import ops

from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import FeedForward, Runtime, register_feed_forward


@register_feed_forward("mlp")
class MlpFeedForward(FeedForward):
    def __init__(self, spec, hidden):
        super().__init__(spec, hidden)
        self.inter = int(spec.params["inter"])
        self.activation = spec.params.get("activation", "poly_norm")
        self.eps = float(spec.params.get("eps", 0.0))
        self.poly = self.activation == "poly_norm"
        if not self.poly and self.activation not in ops.PLAIN_ACTIVATIONS:
            raise ValueError(f"feed-forward activation {self.activation!r} is not implemented ('poly_norm' or one of {sorted(ops.PLAIN_ACTIVATIONS)})")

    def tensor_decls(self) -> List[TensorDecl]:
        t = self.spec.tensors
        decls = [TensorDecl(t["up"], (self.inter, self.hidden)), TensorDecl(t["down"], (self.hidden, self.inter))]
        return decls + ([TensorDecl(t["act"], (4,), FLOAT32, init="gain")] if self.poly else [])

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        self.w_up, self.w_down = weights[t["up"]], weights[t["down"]]
        self.coef = weights[t["act"]] if self.poly else None
        self.p_up = self.p_down = None

    def matrices(self):
        return [self.w_up, self.w_down]

    def product_shapes(self):
        return [(self.inter, self.hidden), (self.hidden, self.inter)]

    def small_tensors(self):
        return [self.coef] if self.poly else []

    def pack_matrices(self) -> None:
        if not self.poly:
            self.p_up, self.p_down = ops.PackedWeight(self.w_up), ops.PackedWeight(self.w_down)

    def emit(self, plan) -> int:
        if not self.poly:
            return plan.act_mlp(w_up=self.w_up, p_up=self.p_up, w_down=self.w_down, p_down=self.p_down, inter=self.inter,
                                activation=ops.PLAIN_ACTIVATIONS[self.activation])
        return plan.mlp(w_up=self.w_up, w_down=self.w_down, inter=self.inter, coef=self.coef, eps=self.eps)
