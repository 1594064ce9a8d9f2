"""Typed configuration of Gumozen: a decoder whose sublayers read the residual stream itself and are normed on their way back
into it.

  embedding   the table's row, RMS-normed with a gain of its own
  layer       x += ls1 * norm1(mixer(shift(x))), then x += ls2 * norm2(ff(x)): RMS norms on the sublayers' results, times a
              scale per channel; what the mixer reads is mixed channel by channel with the previous token's row,
              shift(x)_t = x_t + (x_(t-1) - x_t) * mu (the previous row is part of a request's state)
  attention   differential: two maps per head over the same values, each a softmax of its own over the row's stretch of
              `mask.size` positions counted from 0; q and k normed per head and map, then the first `rot.dims` channels turned
              (pairs (i, i + dims/2), frequencies with the smooth three-band scaling of `rot.scaling`); o = a_1 - lambda a_2,
              divided by its root mean square, times 1 - `diff`, times one sigmoid gate per head
  hgrn2       a recurrence per head with a decay per channel, f = l + (1 - l) sigmoid(W_f h + b), and its complement as the key:
              S = diag(f) S + (1 - f) v', read-out S' q normed per head
  latent_attention  queries through a normed latent, keys and values of all heads from a small normed latent that is cached;
              no positions; a layer with `kv_from` reads an earlier layer's cached latent with its own up-projections
  feed-forward  a mixture of experts: scores sigmoid(W_router h), the `top` largest chosen, an expert applied to its score
              times h
  output      the model's norm, then the head

config.json gives every size and constant; what the design fixes (the activations, the pairing of the rotation, which norms
and gates a mixer has) is written here or in the parts.  A layer without a feed-forward whose checkpoint nevertheless holds
that sublayer's norm and scale has them declared, so that loading accounts for every tensor, and never reads them.
"""
from __future__ import annotations

import copy
from typing import Any, Dict, Mapping, Optional, Sequence, Tuple

from .base import ArchConfig, ConfigError, require
from .spec import FeedForwardSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec

MAX_POSITIONS = 1 << 20
ACTIVATION = "silu"
MIXER_TYPES = ("attention", "hgrn2", "latent_attention")
SCALING_KEYS = ("factor", "low", "high", "original")


class GumozenConfig(ArchConfig):
    architecture = "Gumozen"

    def __init__(self, cfg: Dict[str, Any], unread: Sequence[Tuple[str, Tuple[int, ...]]] = ()):
        self.cfg = cfg
        self.unread = tuple(unread)     # (name, shape) of checkpoint tensors of sublayers that a layer does not have

    def __eq__(self, other) -> bool:
        return isinstance(other, GumozenConfig) and self.cfg == other.cfg

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, cfg: Mapping[str, Any], tensors: Optional[Mapping[str, Sequence[int]]] = None) -> "GumozenConfig":
        c = copy.deepcopy(dict(cfg))
        width, vocab = int(require(c, "width")), int(require(c, "vocab"))
        for name in ("embed", "head"):
            if tensors is not None and name in tensors and tuple(int(s) for s in tensors[name]) != (vocab, width):
                raise ConfigError(f"config.json says {name} is {[vocab, width]}, the checkpoint holds {list(tensors[name])}")
        float(require(c, "norm.eps"))
        layers = require(c, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: layers must be a non-empty list")
        unread = []
        for i, layer in enumerate(layers):
            kind, m = layer.get("type"), layer.get("mixer")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is none of {list(MIXER_TYPES)}")
            if not isinstance(m, dict):
                raise ConfigError(f"layer {i}: no mixer sizes")
            sizes = {"attention": ("heads", "kv_heads", "dim", "vdim"), "hgrn2": ("heads", "dim", "vdim"),
                     "latent_attention": ("heads", "dim", "vdim", "kv_rank", "q_rank")}[kind]
            for key in sizes:
                if int(require(m, key)) < 1:
                    raise ConfigError(f"layer {i}: {key} = {m[key]}")
            if kind == "attention":
                cls._check_attention(i, m)
            elif kind == "latent_attention":
                float(require(m, "scale"))
                src = m.get("kv_from")
                if src is not None:
                    src = int(src)
                    owner = layers[src] if 0 <= src < i else {}
                    if owner.get("type") != "latent_attention" or (owner.get("mixer") or {}).get("kv_from") is not None:
                        raise ConfigError(f"layer {i}: kv_from {src} is no earlier latent-attention layer with a latent of its own")
                    if int(owner["mixer"]["kv_rank"]) != int(m["kv_rank"]):
                        raise ConfigError(f"layer {i}: kv_rank {m['kv_rank']} differs from layer {src}'s, whose latent it reads")
            mlp = layer.get("mlp")
            if mlp is None:
                if tensors is not None:
                    unread += [(n, tuple(int(s) for s in tensors[n])) for n in (f"l{i}.norm2", f"l{i}.ls2") if n in tensors]
                continue
            if mlp.get("kind") != "moe":
                raise ConfigError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} is not 'moe'")
            experts, top = int(require(mlp, "router.experts")), int(require(mlp, "router.top"))
            if int(require(mlp, "expert.ff")) < 1 or experts < 1 or not 1 <= top <= experts:
                raise ConfigError(f"layer {i}: {top} of {experts} experts a token")
        return cls(c, unread)

    @staticmethod
    def _check_attention(i: int, m: Mapping[str, Any]) -> None:
        float(require(m, "scale"))
        float(require(m, "diff"))
        if int(m["heads"]) % int(m["kv_heads"]):
            raise ConfigError(f"layer {i}: {m['heads']} heads are not a multiple of {m['kv_heads']} kv heads")
        rot = m.get("rot") or {}
        dims = int(rot.get("dims", 0))
        if dims % 2 or not 0 <= dims <= int(m["dim"]):
            raise ConfigError(f"layer {i}: {dims} rotated dimensions of a map of {m['dim']}")
        if dims:
            float(require(rot, "base"))
        if rot.get("scaling") is not None:
            factor, low, high, original = (float(require(rot["scaling"], k)) for k in SCALING_KEYS)
            if not (factor > 0 and 0 < low < high and original > 0):
                raise ConfigError(f"layer {i}: rot.scaling {rot['scaling']}")
        size = (m.get("mask") or {}).get("size")
        if size is not None and int(size) < 1:
            raise ConfigError(f"layer {i}: mask.size = {size}")

    def to_dict(self) -> dict:
        return copy.deepcopy(self.cfg)

    def derived(self) -> dict:
        kinds = [layer["type"] for layer in self.cfg["layers"]]
        shared = {str(i): int(layer["mixer"]["kv_from"]) for i, layer in enumerate(self.cfg["layers"]) if layer["mixer"].get("kv_from") is not None}
        return {"max_positions": MAX_POSITIONS, "layers_by_type": {k: kinds.count(k) for k in MIXER_TYPES}, "reads_latent_of": shared}

    # ------------------------------------------------------------------ the model it describes
    def _attention(self, i: int, m: Mapping[str, Any], eps: float) -> MixerSpec:
        p = f"l{i}.mix."
        size = (m.get("mask") or {}).get("size")
        params = {"heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]), "v_head_dim": int(m["vdim"]),
                  "scale": float(m["scale"]), "chunk": 0 if size is None else int(size), "diff": float(m["diff"]), "norm_eps": eps}
        names = {"q_proj": p + "q", "k_proj": p + "k", "v_proj": p + "v", "out_proj": p + "o", "q_norm": p + "q.norm", "k_norm": p + "k.norm",
                 "gate_proj": p + "g", "lambda": tuple(p + n for n in ("lq1", "lk1", "lq2", "lk2"))}
        rot = m.get("rot") or {}
        position = None
        if int(rot.get("dims", 0)) > 0:
            rope = {"theta": float(rot["base"]), "rotary_dim": int(rot["dims"]), "variant": "half_split", "precision": "f64"}
            if rot.get("scaling") is not None:
                rope["bands"] = {k: float(rot["scaling"][k]) for k in SCALING_KEYS}
            position = PositionSpec("rope", rope)
        return MixerSpec("differential_attention", params, names, position=position)

    def _latent(self, i: int, m: Mapping[str, Any], eps: float) -> MixerSpec:
        p = f"l{i}.mix."
        params = {"heads": int(m["heads"]), "dim": int(m["dim"]), "rot_dim": 0, "vdim": int(m["vdim"]), "kv_rank": int(m["kv_rank"]),
                  "q_rank": int(m["q_rank"]), "scale": float(m["scale"]), "norm_eps": eps}
        names = {"dq": p + "dq", "dq_norm": p + "dq.norm", "uq": p + "uq", "uk": p + "uk", "uv": p + "uv", "o": p + "o"}
        if m.get("kv_from") is not None:
            params["kv_source"] = int(m["kv_from"])
        else:
            names.update(dkv=p + "dkv", dkv_norm=p + "dkv.norm")
        return MixerSpec("latent_attention", params, names)

    def _recurrence(self, i: int, m: Mapping[str, Any], eps: float) -> MixerSpec:
        p = f"l{i}.mix."
        params = {"heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "norm_eps": eps}
        names = {"q": p + "q", "f": p + "f", "f_bias": p + "f.b", "lower": p + "lower", "v": p + "v", "norm": p + "norm", "o": p + "o"}
        return MixerSpec("gated_outer", params, names)

    def _experts(self, i: int, mlp: Mapping[str, Any]) -> FeedForwardSpec:
        p = f"l{i}.mlp."
        n = int(mlp["router"]["experts"])
        params = {"experts": n, "top": int(mlp["router"]["top"]), "inter": int(mlp["expert"]["ff"]), "activation": ACTIVATION,
                  "scores": "sigmoid", "weigh": "input"}
        names = {"router": p + "router", "gate": tuple(f"{p}e{e}.gate" for e in range(n)), "up": tuple(f"{p}e{e}.up" for e in range(n)),
                 "down": tuple(f"{p}e{e}.down" for e in range(n))}
        return FeedForwardSpec("moe", params, names)

    def model_spec(self) -> ModelSpec:
        c = self.cfg
        eps = float(c["norm"]["eps"])
        make = {"attention": self._attention, "hgrn2": self._recurrence, "latent_attention": self._latent}
        layers = []
        for i, layer in enumerate(c["layers"]):
            name = f"l{i}"
            parts = [("mixer_input", MixerSpec("token_shift", {}, {"mu": f"{name}.shift"})), ("mixer", make[layer["type"]](i, layer["mixer"], eps)),
                     ("norm1", NormSpec("rms", eps, f"{name}.norm1", scale=f"{name}.ls1"))]
            if layer.get("mlp") is not None:
                parts += [("ffn", self._experts(i, layer["mlp"])), ("norm2", NormSpec("rms", eps, f"{name}.norm2", scale=f"{name}.ls2"))]
            layers.append(LayerSpec(name, "post_norm", parts=parts))
        return ModelSpec(
            architecture=self.architecture, hidden=int(c["width"]), vocab=int(c["vocab"]), layers=tuple(layers), order=tuple(range(len(layers))),
            embedding="embed", final_norm=NormSpec("rms", eps, "final.norm"), head="head", max_position=MAX_POSITIONS,
            embedding_norm=NormSpec("rms", eps, "embed.norm"), unread_tensors=self.unread)
