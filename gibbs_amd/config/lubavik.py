"""Typed configuration of Lubavik: a decoder whose sublayers read the residual stream itself and are normed on their way back
into it, and whose layers each add a row of a second token table.

  layer       x += norm1(mixer(x)), then x += norm2(ff(x)), then x += side_norm(W_proj (gelu(W_gate x) * e)) with e the layer's
              `token_side.dim` entries of the token's row in a second table.  norm1, norm2 and the model's last norm are RMS
              norms whose weight is stored around zero (the gain is 1 + w); side_norm's is plain
  attention   grouped heads; q and k normed over their whole projections before the rotation of the first `rot.dims` channels
              (pairs (i, i + dims/2)); every earlier position is seen; a learned sink per head; a layer with `kv_from` projects
              queries only and reads that layer's cached keys and values
  parallel    two mixers of the same rows, left_scale * left + right_scale * right.  Left: attention with biases on all of its
              projections, q and k normed per head, neighbouring channels turned, a row sees its own stretch of `mask.size`
              positions counted from 0.  Right: gated linear attention, a state per head whose key channels decay by
              sigmoid(z)^(1/tau), z from a low-rank pair
  mlstm       the matrix memory of xLSTM: exponential gates capped at `gate_cap`, a normaliser and a running maximum
  feed-forward  dense, down(relu(up h)^2); or experts: scores by a softmax over all router outputs, the `top` largest, weights
              the chosen scores over their sum times `router.scale`; a shared expert is added for every token
  output      the model's norm, then the head

config.json gives every size and constant but one, which the checkpoint's shapes give: the rank of the decay's low-rank pair.
What the design fixes (the activations, the pairing of the two rotations, which norms and gates a mixer has) is written here or in
the parts.  A layer without a feed-forward whose checkpoint nevertheless holds that sublayer's norm has it declared, so that
loading accounts for every tensor, and never reads it.
"""
from __future__ import annotations

import copy
from typing import Any, Dict, Mapping, Optional, Sequence, Tuple

from .base import ArchConfig, ConfigError, require
from .spec import FeedForwardSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec

MAX_POSITIONS = 1 << 20
EXPERT_ACTIVATION, DENSE_ACTIVATION, SIDE_ACTIVATION = "silu", "relu_squared", "gelu_tanh"
MIXER_TYPES = ("attention", "parallel", "mlstm")
DECAY_RANK = 16             # of a model without a checkpoint to read it from


class LubavikConfig(ArchConfig):
    architecture = "Lubavik"

    def __init__(self, cfg: Dict[str, Any], ranks: Optional[Mapping[int, int]] = None, unread: Sequence[Tuple[str, Tuple[int, ...]]] = ()):
        self.cfg = cfg
        self.ranks = dict(ranks or {})  # layer -> rank of the decay's low-rank pair
        self.unread = tuple(unread)     # (name, shape) of checkpoint tensors of sublayers that a layer does not have

    def __eq__(self, other) -> bool:
        return isinstance(other, LubavikConfig) and (self.cfg, self.ranks) == (other.cfg, other.ranks)

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any], tensors: Optional[Mapping[str, Sequence[int]]] = None) -> "LubavikConfig":
        c = copy.deepcopy(dict(cfg))
        tensors = dict(tensors or {})
        width, vocab = int(require(c, "width")), int(require(c, "vocab"))
        for name in ("embed", "head"):
            if name in tensors and tuple(int(s) for s in tensors[name]) != (vocab, width):
                raise ConfigError(f"config.json says {name} is {[vocab, width]}, the checkpoint holds {list(tensors[name])}")
        float(require(c, "norm.eps"))
        if c.get("token_side") is not None and int(require(c, "token_side.dim")) < 1:
            raise ConfigError(f"token_side.dim = {c['token_side']['dim']}")
        layers = require(c, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a non-empty list")
        ranks, unread = {}, []
        for i, layer in enumerate(layers):
            kind, m = layer.get("type"), layer.get("mixer")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is none of {list(MIXER_TYPES)}")
            if not isinstance(m, dict):
                raise ConfigError(f"layer {i}: no mixer sizes")
            if kind == "attention":
                cls._check_attention(i, m)
                cls._check_source(i, m, layers)
            elif kind == "parallel":
                left, right = require(m, "left"), require(m, "right")
                cls._check_attention(i, left)
                if left.get("kv_from") is not None:
                    raise ConfigError(f"layer {i}: the left mixer of a parallel pair has keys and values of its own (kv_from)")
                cls._check_state(i, right)
                if not float(require(right, "tau")) > 0:
                    raise ConfigError(f"layer {i}: tau = {right['tau']}")
                float(require(m, "left_scale"))
                float(require(m, "right_scale"))
                pair = tensors.get(f"l{i}.mix.right.a1")
                ranks[i] = DECAY_RANK if pair is None else int(pair[0])
            else:
                cls._check_state(i, m)
                if not float(require(m, "gate_cap")) > 0:
                    raise ConfigError(f"layer {i}: gate_cap = {m['gate_cap']}")
            mlp = layer.get("mlp")
            if mlp is None:
                unread += [(n, tuple(int(s) for s in tensors[n])) for n in (f"l{i}.norm2",) if n in tensors]
            elif mlp.get("kind") == "dense":
                if int(require(mlp, "ff")) < 1:
                    raise ConfigError(f"layer {i}: ff = {mlp['ff']}")
            elif mlp.get("kind") == "moe":
                experts, top = int(require(mlp, "router.experts")), int(require(mlp, "router.top"))
                if int(require(mlp, "expert.ff")) < 1 or experts < 1 or not 1 <= top <= experts:
                    raise ConfigError(f"layer {i}: {top} of {experts} experts a token")
                if mlp.get("shared") is not None and int(require(mlp, "shared.ff")) < 1:
                    raise ConfigError(f"layer {i}: shared.ff = {mlp['shared']['ff']}")
            else:
                raise ConfigError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} is neither 'dense' nor 'moe'")
        return cls(c, ranks, unread)

    @staticmethod
    def _check_attention(i: int, m: Mapping[str, Any]) -> None:
        for key in ("heads", "kv_heads", "dim", "vdim"):
            if int(require(m, key)) < 1:
                raise ConfigError(f"layer {i}: {key} = {m[key]}")
        float(require(m, "scale"))
        if int(m["heads"]) % int(m["kv_heads"]):
            raise ConfigError(f"layer {i}: {m['heads']} heads are not a multiple of {m['kv_heads']} kv heads")
        rot = m.get("rot") or {}
        dims = int(rot.get("dims", 0))
        if dims % 2 or not 0 <= dims <= int(m["dim"]):
            raise ConfigError(f"layer {i}: {dims} rotated dimensions of a head of {m['dim']}")
        if dims:
            float(require(rot, "base"))
        size = (m.get("mask") or {}).get("size")
        if size is not None and int(size) < 1:
            raise ConfigError(f"layer {i}: mask.size = {size}")

    @staticmethod
    def _check_source(i: int, m: Mapping[str, Any], layers: Sequence[Mapping[str, Any]]) -> None:
        if m.get("kv_from") is None:
            return
        src = int(m["kv_from"])
        owner = layers[src] if 0 <= src < i else {}
        if owner.get("type") != "attention" or (owner.get("mixer") or {}).get("kv_from") is not None:
            raise ConfigError(f"layer {i}: kv_from {src} is no earlier attention layer with keys and values of its own")
        for key in ("kv_heads", "dim", "vdim"):
            if int(owner["mixer"][key]) != int(m[key]):
                raise ConfigError(f"layer {i}: {key} {m[key]} differs from layer {src}'s, whose keys and values it reads")

    @staticmethod
    def _check_state(i: int, m: Mapping[str, Any]) -> None:
        for key in ("heads", "dim", "vdim"):
            if int(require(m, key)) < 1:
                raise ConfigError(f"layer {i}: {key} = {m[key]}")

    def to_dict(self) -> dict:
        return copy.deepcopy(self.cfg)

    def derived(self) -> dict:
        kinds = [layer["type"] for layer in self.cfg["layers"]]
        shared = {str(i): int(layer["mixer"]["kv_from"]) for i, layer in enumerate(self.cfg["layers"]) if layer["mixer"].get("kv_from") is not None}
        return {"max_positions": MAX_POSITIONS, "layers_by_type": {k: kinds.count(k) for k in MIXER_TYPES}, "reads_cache_of": shared,
                "decay_ranks": {str(i): r for i, r in self.ranks.items()}}

    # ------------------------------------------------------------------ the model it describes
    @staticmethod
    def _rotation(m: Mapping[str, Any], variant: str) -> Optional[PositionSpec]:
        rot = m.get("rot") or {}
        if int(rot.get("dims", 0)) == 0:
            return None
        return PositionSpec("rope", {"theta": float(rot["base"]), "rotary_dim": int(rot["dims"]), "variant": variant, "precision": "f64"})

    @staticmethod
    def _attention_params(m: Mapping[str, Any], eps: float) -> dict:
        size = (m.get("mask") or {}).get("size")
        return {"heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]), "v_head_dim": int(m["vdim"]),
                "scale": float(m["scale"]), "chunk": 0 if size is None else int(size), "qk_norm_eps": eps}

    def _attention(self, p: str, m: Mapping[str, Any], eps: float) -> MixerSpec:
        params = dict(self._attention_params(m, eps), chunk=0, qk_norm="whole", sink=True)
        names = {"q_proj": p + "q", "out_proj": p + "o", "q_norm": p + "q.norm", "sink": p + "sink"}
        if m.get("kv_from") is not None:
            params["kv_source"] = int(m["kv_from"])
        else:
            names.update(k_proj=p + "k", v_proj=p + "v", k_norm=p + "k.norm")
        return MixerSpec("attention", params, names, position=self._rotation(m, "half_split"))

    def _chunked(self, p: str, m: Mapping[str, Any], eps: float) -> MixerSpec:
        params = dict(self._attention_params(m, eps), qk_norm="before", bias=True, out_bias=True)
        names = {"q_proj": p + "q", "k_proj": p + "k", "v_proj": p + "v", "out_proj": p + "o", "q_norm": p + "q.norm", "k_norm": p + "k.norm",
                 "q_bias": p + "q.b", "k_bias": p + "k.b", "v_bias": p + "v.b", "o_bias": p + "o.b"}
        return MixerSpec("attention", params, names, position=self._rotation(m, "interleaved"))

    def _linear(self, p: str, m: Mapping[str, Any], eps: float, rank: int) -> MixerSpec:
        params = {"heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "rank": rank, "tau": float(m["tau"]), "norm_eps": eps}
        names = {n: p + n for n in ("q", "k", "v", "g", "a1", "a2", "norm", "o")}
        return MixerSpec("gated_linear", params, dict(names, a2_bias=p + "a2.b"))

    def _memory(self, p: str, m: Mapping[str, Any], eps: float) -> MixerSpec:
        params = {"heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "gate_cap": float(m["gate_cap"]), "norm_eps": eps}
        names = {n: p + n for n in ("q", "k", "v", "g", "i", "f", "norm", "o")}
        return MixerSpec("matrix_lstm", params, dict(names, i_bias=p + "i.b", f_bias=p + "f.b"))

    def _feed_forward(self, p: str, mlp: Mapping[str, Any]) -> FeedForwardSpec:
        if mlp["kind"] == "dense":
            return FeedForwardSpec("mlp", {"inter": int(mlp["ff"]), "activation": DENSE_ACTIVATION}, {"up": p + "up", "down": p + "down"})
        n, shared = int(mlp["router"]["experts"]), mlp.get("shared")
        params = {"experts": n, "top": int(mlp["router"]["top"]), "inter": int(mlp["expert"]["ff"]), "activation": EXPERT_ACTIVATION,
                  "scores": "softmax_all", "weight_scale": float(mlp["router"].get("scale", 1.0)),
                  "shared": None if shared is None else {"inter": int(shared["ff"]), "activation": EXPERT_ACTIVATION, "gate": False}}
        names = {"router": p + "router", "gate": tuple(f"{p}e{e}.gate" for e in range(n)), "up": tuple(f"{p}e{e}.up" for e in range(n)),
                 "down": tuple(f"{p}e{e}.down" for e in range(n))}
        if shared is not None:
            names.update(shared_gate=p + "shared.gate", shared_up=p + "shared.up", shared_down=p + "shared.down")
        return FeedForwardSpec("moe", params, names)

    def model_spec(self) -> ModelSpec:
        c = self.cfg
        eps, count = float(c["norm"]["eps"]), len(c["layers"])
        norm = lambda name: NormSpec("rms", eps, name, offset=1.0)
        side = c.get("token_side")
        layers = []
        for i, layer in enumerate(c["layers"]):
            name, m, params = f"l{i}", layer["mixer"], {}
            p = f"{name}.mix."
            if layer["type"] == "attention":
                parts = [("mixer", self._attention(p, m, eps))]
            elif layer["type"] == "parallel":
                parts = [("left", self._chunked(p + "left.", m["left"], eps)), ("right", self._linear(p + "right.", m["right"], eps, self.ranks[i]))]
                params = {"left_scale": float(m["left_scale"]), "right_scale": float(m["right_scale"])}
            else:
                parts = [("mixer", self._memory(p, m, eps))]
            parts.append(("norm1", norm(f"{name}.norm1")))
            if layer.get("mlp") is not None:
                parts += [("ffn", self._feed_forward(f"{name}.mlp.", layer["mlp"])), ("norm2", norm(f"{name}.norm2"))]
            if side is not None:
                d = int(side["dim"])
                parts += [("side", FeedForwardSpec("token_side", {"dim": d, "column": i * d, "columns": count * d, "vocab": int(c["vocab"]),
                                                                  "activation": SIDE_ACTIVATION, "declares_table": i == 0},
                                                   {"table": "side.embed", "gate": f"{name}.side.gate", "proj": f"{name}.side.proj"})),
                          ("side_norm", NormSpec("rms", eps, f"{name}.side.norm"))]
            layers.append(LayerSpec(name, "post_norm", parts=parts, params=params))
        return ModelSpec(
            architecture=self.architecture, hidden=int(c["width"]), vocab=int(c["vocab"]), layers=tuple(layers), order=tuple(range(count)),
            embedding="embed", final_norm=norm("final.norm"), head="head", max_position=MAX_POSITIONS, unread_tensors=self.unread)
