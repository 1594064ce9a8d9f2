"""Gated outer-product mixer (HGRN2): a decayed state per head in which the complement of the decay stands for the key.

With h the mixer's input, per head, q = silu(W_q h) [dim], v = W_v h [vdim] and a forget gate per channel that never falls
below a learned bound, f = l + (1 - l) sigmoid(W_f h + b); with a state S [dim, vdim] that starts at zero and ' for transposed:

    S = diag(f) S + (1 - f) v';    y = S' q

Each head's y is divided by its root mean square (eps inside the root), multiplied by a gain [vdim] that the heads share, and
the heads are projected back.  S lives in the request's slot as float32; the gate, 1 - f (taken as (1 - l) sigmoid(-z), which
does not cancel), the rule and the norm are float32 in both precisions of a run.  The kernels are csrc/gated_outer.hip's and,
for the walk over ragged portions, csrc/recurrent.hip's.
"""
from __future__ import annotations

from typing import List, Sequence

import torch

from ..cache.needs import StateNeed
from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import Mixer, Runtime, register_mixer

RULE_STATE = "gated_outer_rule"


@register_mixer("gated_outer")
class GatedOuterMixer(Mixer):
    def __init__(self, spec, hidden, layer_index):
        super().__init__(spec, hidden, layer_index)
        p = spec.params
        self.heads, self.dim, self.vdim, self.norm_eps = int(p["heads"]), int(p["dim"]), int(p["vdim"]), float(p["norm_eps"])
        if self.heads < 1 or not 0 < self.dim <= 256 or self.vdim < 1:
            raise ValueError(f"{self.heads} heads with states of {self.dim} x {self.vdim} (at least 1; at most 256 channels)")

    def state_needs(self) -> Sequence[StateNeed]:
        return (StateNeed(RULE_STATE, (self.heads, self.dim, self.vdim)),)

    def tensor_decls(self) -> List[TensorDecl]:
        t, W = self.spec.tensors, self.hidden
        qk, hv = self.heads * self.dim, self.heads * self.vdim
        return [TensorDecl(t["q"], (qk, W)), TensorDecl(t["f"], (qk, W)), TensorDecl(t["f_bias"], (qk,), FLOAT32, init="bias"),
                TensorDecl(t["lower"], (qk,), FLOAT32, init="unit"), TensorDecl(t["v"], (hv, W)),
                TensorDecl(t["norm"], (self.vdim,), FLOAT32, init="gain"), TensorDecl(t["o"], (W, hv))]

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        # one product for everything that reads the rows: [q | f | v]
        self.w_in = torch.cat([weights[t["q"]], weights[t["f"]], weights[t["v"]]], dim=0).contiguous()
        self.w_out = weights[t["o"]].contiguous()
        self.f_bias, self.lower, self.gain = weights[t["f_bias"]], weights[t["lower"]], weights[t["norm"]]

    def matrices(self):
        return [self.w_in, self.w_out]

    def product_shapes(self):
        hv = self.heads * self.vdim
        return [(2 * self.heads * self.dim + hv, self.hidden), (self.hidden, hv)]

    def small_tensors(self):
        return [self.f_bias, self.lower, self.gain]

    def state_bytes(self) -> int:
        """Bytes of state that a decoded token reads and writes."""
        return 2 * 4 * self.heads * self.dim * self.vdim

    def emit(self, plan, cache) -> int:
        return plan.gated_outer(self, rule_state=cache.states[RULE_STATE])
