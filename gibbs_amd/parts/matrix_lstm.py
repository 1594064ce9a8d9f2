"""Matrix memory of xLSTM (mLSTM): an outer-product state per head with exponential gates, a normaliser and a running maximum.

With h the mixer's input, per head, q = W_q h / sqrt(dim), k = W_k h [dim], v = W_v h [vdim], and two gates of one number each,
a = cap tanh((w_i . h + b_i) / cap) and log f = log sigmoid(cap tanh((w_f . h + b_f) / cap)); with S [dim, vdim], n [dim] and m
from zero:

    m' = max(log f + m, a);   keep = exp(log f + m - m');   take = exp(a - m')
    S = keep S + take k v';   n = keep n + take k;   m = m';   o = S' q / (max(|n . q|, exp(-m)) + 1e-6)

Each head's o is divided by its root mean square (eps inside the root); the heads side by side are multiplied by a gain
[heads * vdim] and by sigmoid(W_g h), and projected back.  S, n and m live in the request's slot as float32; the gates (their
projections are float32 sums that are not rounded), the rule and the norm are float32 in both precisions of a run.  The
kernels are csrc/matrix_lstm.hip's.
"""
from __future__ import annotations

from typing import List, Sequence

import torch

from .. import ops
from ..cache.needs import StateNeed
from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import Mixer, Runtime, register_mixer
from .segments import stacked_rows

RULE_STATE, NORM_STATE = "matrix_lstm_rule", "matrix_lstm_norm"


@register_mixer("matrix_lstm")
class MatrixLstmMixer(Mixer):
    def __init__(self, spec, hidden, layer_index):
        super().__init__(spec, hidden, layer_index)
        p = spec.params
        self.heads, self.dim, self.vdim = int(p["heads"]), int(p["dim"]), int(p["vdim"])
        self.gate_cap, self.norm_eps = float(p["gate_cap"]), float(p["norm_eps"])
        self.q_scale = self.dim ** -0.5
        if min(self.heads, self.dim, self.vdim) < 1 or not self.gate_cap > 0:
            raise ValueError(f"{self.heads} heads with states of {self.dim} x {self.vdim}, gates capped at {self.gate_cap}")

    def state_needs(self) -> Sequence[StateNeed]:
        # (n of every head, then m of every head; in whole 16 bytes, so that the next layer's state stays aligned)
        return (StateNeed(RULE_STATE, (self.heads, self.dim, self.vdim)), StateNeed(NORM_STATE, (-(-self.heads * (self.dim + 1) // 4) * 4,)))

    def tensor_decls(self) -> List[TensorDecl]:
        t, W, H = self.spec.tensors, self.hidden, self.heads
        qk, hv = H * self.dim, H * self.vdim
        return [TensorDecl(t["q"], (qk, W)), TensorDecl(t["k"], (qk, W)), TensorDecl(t["v"], (hv, W)), TensorDecl(t["g"], (hv, W)),
                TensorDecl(t["i"], (H, W)), TensorDecl(t["i_bias"], (H,), FLOAT32, init="bias"), TensorDecl(t["f"], (H, W)),
                TensorDecl(t["f_bias"], (H,), FLOAT32, init="bias"), TensorDecl(t["norm"], (hv,), FLOAT32, init="gain"), TensorDecl(t["o"], (W, hv))]

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        self.w_in, (self.off_q, self.off_k, self.off_v, self.off_g) = stacked_rows([weights[t[n]] for n in ("q", "k", "v", "g")])
        self.w_gates = torch.cat([weights[t["i"]], weights[t["f"]]], dim=0).contiguous()
        self.b_gates = torch.cat([weights[t["i_bias"]], weights[t["f_bias"]]]).contiguous()
        self.w_out, self.gain = weights[t["o"]].contiguous(), weights[t["norm"]]
        self.p_in = self.p_out = None

    def matrices(self):
        return [self.w_in, self.w_gates, self.w_out]

    def product_shapes(self):
        qk, hv = self.heads * self.dim, self.heads * self.vdim
        return [(2 * qk + 2 * hv + 2 * self.heads, self.hidden), (self.hidden, hv)]

    def small_tensors(self):
        return [self.b_gates, self.gain]

    def state_bytes(self) -> int:
        """Bytes of state that a decoded token reads and writes."""
        return 2 * 4 * self.heads * (self.dim * self.vdim + self.dim + 1)

    def pack_matrices(self) -> None:
        self.p_in, self.p_out = ops.PackedWeight(self.w_in), ops.PackedWeight(self.w_out)

    def emit(self, plan, cache) -> int:
        return plan.matrix_lstm(self, rule_state=cache.states[RULE_STATE], norm_state=cache.states[NORM_STATE])
