"""Gated linear attention mixer: an outer-product state per head whose rows decay by a gate per key channel.

With h the mixer's input, per head, q = W_q h / sqrt(dim), k = W_k h [dim], v = W_v h [vdim] and a decay per key channel
f = sigmoid(z)^(1 / tau), z = W_a2 (W_a1 h) + b (a low-rank pair); with a state S [dim, vdim] that starts at zero and ' for
transposed:

    S = diag(f) S + k v';    y = S' q

Each head's y is divided by its root mean square (eps inside the root), multiplied by a gain [vdim] that the heads share; the
heads side by side are multiplied by silu(W_g h) and projected back.  S lives in the request's slot as float32; the decay, the
rule, the norm and the output gate are float32 in both precisions of a run.  The kernels are csrc/gated_linear.hip's.
"""
from __future__ import annotations

from typing import List, Sequence

import torch

from .. import ops
from ..cache.needs import StateNeed
from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import Mixer, Runtime, register_mixer
from .segments import stacked_rows

RULE_STATE = "gated_linear_rule"


@register_mixer("gated_linear")
class GatedLinearMixer(Mixer):
    def __init__(self, spec, hidden, layer_index):
        super().__init__(spec, hidden, layer_index)
        p = spec.params
        self.heads, self.dim, self.vdim, self.rank = int(p["heads"]), int(p["dim"]), int(p["vdim"]), int(p["rank"])
        self.tau, self.norm_eps = float(p["tau"]), float(p["norm_eps"])
        self.q_scale = self.dim ** -0.5
        if min(self.heads, self.dim, self.vdim, self.rank) < 1 or not self.tau > 0:
            raise ValueError(f"{self.heads} heads with states of {self.dim} x {self.vdim}, a decay of rank {self.rank} with tau {self.tau}")

    def state_needs(self) -> Sequence[StateNeed]:
        return (StateNeed(RULE_STATE, (self.heads, self.dim, self.vdim)),)

    def tensor_decls(self) -> List[TensorDecl]:
        t, W = self.spec.tensors, self.hidden
        qk, hv = self.heads * self.dim, self.heads * self.vdim
        return [TensorDecl(t["q"], (qk, W)), TensorDecl(t["k"], (qk, W)), TensorDecl(t["v"], (hv, W)), TensorDecl(t["g"], (hv, W)),
                TensorDecl(t["a1"], (self.rank, W)), TensorDecl(t["a2"], (qk, self.rank)), TensorDecl(t["a2_bias"], (qk,), FLOAT32, init="bias"),
                TensorDecl(t["norm"], (self.vdim,), FLOAT32, init="gain"), TensorDecl(t["o"], (W, hv))]

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        self.w_in, (self.off_q, self.off_k, self.off_v, self.off_g, self.off_z) = stacked_rows([weights[t[n]] for n in ("q", "k", "v", "g", "a1")])
        self.w_out, self.w_z = weights[t["o"]].contiguous(), weights[t["a2"]].contiguous()
        self.z_bias, self.gain = weights[t["a2_bias"]], weights[t["norm"]]
        self.p_in = self.p_out = None

    def matrices(self):
        return [self.w_in, self.w_z, self.w_out]

    def product_shapes(self):
        qk, hv = self.heads * self.dim, self.heads * self.vdim
        return [(2 * qk + 2 * hv + self.rank, self.hidden), (qk, self.rank), (self.hidden, hv)]

    def small_tensors(self):
        return [self.z_bias, self.gain]

    def state_bytes(self) -> int:
        """Bytes of state that a decoded token reads and writes."""
        return 2 * 4 * self.heads * self.dim * self.vdim

    def pack_matrices(self) -> None:
        self.p_in, self.p_out = ops.PackedWeight(self.w_in), ops.PackedWeight(self.w_out)

    def emit(self, plan, cache) -> int:
        return plan.gated_linear(self, rule_state=cache.states[RULE_STATE])
