"""Differential attention: two attention maps per head over the same values, one taken off the other.

With H query heads and G key/value heads, W_q h has H x [map 1 | map 2] and W_k h G x [map 1 | map 2] entries of `head_dim`
each, W_v h G x `v_head_dim`.  Every map of q and k is divided by its root mean square, multiplied by a gain [head_dim] that
all heads and maps share, and turned by the position encoding (a rotation, or none).  Map c of head h is an ordinary causal
softmax attention of q_(h,c) over k_(g,c), g = h // (H / G), with scores times `scale`, over all earlier positions, the last
`window` of them, or the row's own stretch of `chunk` positions counted from 0.  With the maps' outputs a_1, a_2 and

    lambda = exp(sum lq1 lk1) - exp(sum lq2 lk2) + diff        (vectors of head_dim, one number for the layer)

a head's output is o = a_1 - lambda a_2, divided by its root mean square over its v_head_dim values, times 1 - diff, times
sigmoid(W_g h)_h, one number per head (tensor `gate_proj` [H, hidden], if there is one); then the out-projection.

The cache holds, per position and key/value head, the row [map 1 | map 2] of keys and one row of values.  A map is laid out
as a query head of its own whose query is zero where the other map's key lies: 2 H query heads over G heads of keys of size
2 head_dim, so both maps' scores come from one pass over the keys and one over the values, in the framework's attention
kernels.  Norms, angles, scores, the softmax, lambda and the combination are float32.
"""
from __future__ import annotations

from typing import List, Optional

import torch

from ..cache.needs import CacheNeed
from ..weights.loader import FLOAT32, TensorDecl, WeightStore
from .base import Mixer, Runtime, build_position, register_mixer

MAPS = 2


@register_mixer("differential_attention")
class DifferentialAttentionMixer(Mixer):
    def __init__(self, spec, hidden, layer_index):
        super().__init__(spec, hidden, layer_index)
        p = spec.params
        self.heads, self.kv_heads, self.head_dim, self.v_head_dim = (int(p[k]) for k in ("heads", "kv_heads", "head_dim", "v_head_dim"))
        self.scale, self.diff, self.norm_eps = float(p["scale"]), float(p["diff"]), float(p["norm_eps"])
        self.window = None if p.get("window") is None else int(p["window"])
        self.chunk = int(p.get("chunk") or 0)
        self.gated = spec.tensors.get("gate_proj") is not None
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads are not a multiple of {self.kv_heads} kv heads")
        if self.chunk and self.window is not None:
            raise ValueError("an attention sees a window or chunks, not both")
        if self.window is not None and self.window <= 0:
            raise ValueError(f"attention window {self.window} must be positive")
        if max(MAPS * self.head_dim, self.v_head_dim) > 512:
            raise ValueError(f"keys of {MAPS} x {self.head_dim} and values of {self.v_head_dim} are more than the attention kernels take (512)")
        self.position = build_position(spec.position, self.head_dim)

    # ------------------------------------------------------------------ what it asks for
    def stored_dims(self):
        """(key, value) head sizes as cached: the mixer's own, or, once it is bound for a bfloat16 run, one common size in
        steps of 16 with zeros behind each head's channels, which the matrix-core attention kernels take."""
        pad = getattr(self, "padded_dim", None)
        return (pad, pad) if pad else (MAPS * self.head_dim, self.v_head_dim)

    def cache_need(self) -> Optional[CacheNeed]:
        kd, vd = self.stored_dims()
        return CacheNeed(self.kv_heads, kd, self.window, None if vd == kd else vd)

    def attention_flops(self, keys: float) -> float:
        return 2.0 * keys * MAPS * self.heads * (self.head_dim + self.v_head_dim)

    def tensor_decls(self) -> List[TensorDecl]:
        t, W, H, G, D, V = self.spec.tensors, self.hidden, self.heads, self.kv_heads, self.head_dim, self.v_head_dim
        decls = [TensorDecl(t["q_proj"], (H * MAPS * D, W)), TensorDecl(t["k_proj"], (G * MAPS * D, W)), TensorDecl(t["v_proj"], (G * V, W)),
                 TensorDecl(t["out_proj"], (W, H * V)), TensorDecl(t["q_norm"], (D,), FLOAT32, init="gain"),
                 TensorDecl(t["k_norm"], (D,), FLOAT32, init="gain")]
        decls += [TensorDecl(n, (D,), FLOAT32, init="bias") for n in t["lambda"]]
        if self.gated:
            decls.append(TensorDecl(t["gate_proj"], (H, W)))
        if self.position is not None:
            decls += self.position.tensor_decls()
        return decls

    def bind(self, weights: WeightStore, rt: Runtime) -> None:
        self.rt = rt
        t = self.spec.tensors
        self.padded_dim = None
        pad = -(-max(MAPS * self.head_dim, self.v_head_dim) // 16) * 16
        if rt.act_dtype == torch.bfloat16 and pad <= 128:
            self.padded_dim = pad
        # one product for everything that reads the rows: [q | k | v | gate], the gate's rows up to a multiple of 8 (zero rows)
        rows = [weights[t["q_proj"]], weights[t["k_proj"]], weights[t["v_proj"]]]
        self.gate_off = sum(r.shape[0] for r in rows) if self.gated else -1
        if self.gated:
            rows.append(weights[t["gate_proj"]])
        fill = -sum(r.shape[0] for r in rows) % 8
        if fill:
            rows.append(torch.zeros((fill, self.hidden), dtype=rows[0].dtype, device=rows[0].device))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.w_out = weights[t["out_proj"]].contiguous()
        self.q_gain, self.k_gain = weights[t["q_norm"]], weights[t["k_norm"]]
        lq1, lk1, lq2, lk2 = (weights[n] for n in t["lambda"])
        self.lam = (torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) + self.diff).to(torch.float32).reshape(1).contiguous()
        self.rot = None
        if self.position is not None:
            self.position.bind(weights, rt)
            self.rot = self.position.rotation()
            if self.rot is None:
                raise ValueError("differential attention takes a rotation as its position encoding")

    def matrices(self):
        return [self.w_in, self.w_out]

    def product_shapes(self):
        H, G, D, V = self.heads, self.kv_heads, self.head_dim, self.v_head_dim
        return [(MAPS * (H + G) * D + G * V + (H if self.gated else 0), self.hidden), (self.hidden, H * V)]

    def small_tensors(self):
        return [self.q_gain, self.k_gain, self.lam] + ([] if self.position is None else list(self.position.small_tensors()))

    def emit(self, plan, cache) -> int:
        kd, vd = self.stored_dims()
        if cache.kpages is None or cache.kpages.shape[-1] != kd or cache.vpages.shape[-1] != vd:
            raise ValueError("the differential attention's pages do not have its head sizes")
        return plan.differential_attention(self, kpages=cache.kpages, vpages=cache.vpages, group=cache.group, stored=(kd, vd))
