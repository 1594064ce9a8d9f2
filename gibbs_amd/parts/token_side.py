"""A sublayer that adds a row of a second token table, gated by the stream: proj(gelu(gate x) * e), e the `dim` entries of the
row's token that belong to this layer.

The table [vocab, layers * dim] is one tensor of the checkpoint that every layer of the model reads its columns of (`shared`: the
layer that declares it); it is kept whole on the device, and a step reads a row of it per token.  The product with the gate, its
activation and the table's entries are one kernel in steps of few rows, a product and an elementwise pass beyond.  It is a
feed-forward like the others (it reads rows one by one), beside its batch's token ids."""
from __future__ import annotations

from typing import List

import torch

from .. import ops
from ..weights.loader import TensorDecl, WeightStore
from .base import FeedForward, Runtime, register_feed_forward


@register_feed_forward("token_side")
class TokenSideFeedForward(FeedForward):
    def __init__(self, spec, hidden):
        super().__init__(spec, hidden)
        p = spec.params
        self.dim, self.column, self.columns, self.vocab = int(p["dim"]), int(p["column"]), int(p["columns"]), int(p["vocab"])
        self.activation = p.get("activation", "gelu_tanh")
        self.declares_table = bool(p.get("declares_table", False))
        if self.dim < 1 or not 0 <= self.column <= self.columns - self.dim:
            raise ValueError(f"{self.dim} entries from column {self.column} of a table of {self.columns}")
        if self.activation not in ops.ACTIVATIONS:
            raise ValueError(f"activation {self.activation!r} is not implemented")

    def tensor_decls(self) -> List[TensorDecl]:
        t = self.spec.tensors
        own = [TensorDecl(t["gate"], (self.dim, self.hidden)), TensorDecl(t["proj"], (self.hidden, self.dim))]
        return own + ([TensorDecl(t["table"], (self.vocab, self.columns))] if self.declares_table else [])

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        self.w_gate, self.table = weights[t["gate"]].contiguous(), weights[t["table"]]
        # (the inner size of the second product in steps of 8: columns of zeros, which meet zeros)
        self.stored = -(-self.dim // 8) * 8
        self.w_proj = torch.nn.functional.pad(weights[t["proj"]], (0, self.stored - self.dim)).contiguous()
        self.p_gate = self.p_proj = None

    def matrices(self):
        return [self.w_gate, self.w_proj]

    def product_shapes(self):
        return [(self.dim, self.hidden), (self.hidden, self.dim)]

    def pack_matrices(self) -> None:
        self.p_gate, self.p_proj = ops.PackedWeight(self.w_gate), ops.PackedWeight(self.w_proj)

    def emit(self, plan) -> int:
        return plan.act_mlp(w_up=self.w_gate, p_up=self.p_gate, w_down=self.w_proj, p_down=self.p_proj, inter=self.dim,
                            activation=ops.ACTIVATIONS[self.activation], table=self.table, column=self.column)
