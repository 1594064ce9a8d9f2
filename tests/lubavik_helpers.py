"""Small Lubavik configurations that differ in every size and option, model folders made from them through the
framework's random-weights mode, and the plain implementation's logits for them."""
from __future__ import annotations

import json
import os

import numpy as np

from tests.gumozen_helpers import edited, load_model_dir, tokens  # noqa: F401  (the same reading and editing of model folders)
from tests.plain import lubavik_plain as Z


def _rot(m, rot):
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return m


def attention(heads, kv, dim, vdim, scale, rot=None, kv_from=None):
    m = _rot({"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}, rot)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def chunked(heads, kv, dim, vdim, scale, size=None, rot=None):
    m = _rot({"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}, rot)
    if size is not None:
        m["mask"] = {"size": size}
    return m


def linear(heads, dim, vdim, tau):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def parallel(left, right, left_scale=1.0, right_scale=1.0):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def mlstm(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None, scale=1.0):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


def model(vocab, width, layers, side, eps=1e-5):
    return {"architecture": "Lubavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side}, "layers": layers}


# A: no size a multiple of 8 where it can be avoided (the plain kernels in both precisions); two attention layers read the first
# one's keys and values; scores that stand out (scales well above 1 / sqrt(dim)), so that single keys far back carry weight; a
# layer without a feed-forward; weights of the pair apart; three experts of seven, with and without a shared one.
LUBAVIK_A = model(211, 100, [
    with_mlp(attention(6, 3, 10, 14, 0.7, rot=(1000.0, 6)), moe(7, 3, 30, shared=22, scale=1.7)),
    with_mlp(parallel(chunked(4, 2, 6, 9, 0.6, size=13, rot=(100.0, 4)), linear(3, 9, 15, 4.0), 0.9, 1.6), dense(45)),
    with_mlp(attention(9, 3, 10, 14, 0.5, kv_from=0, rot=(1000.0, 6)), None),
    with_mlp(mlstm(3, 11, 14, 3.0), moe(5, 2, 18)),
    with_mlp(attention(3, 3, 10, 14, 0.8, kv_from=0), moe(4, 1, 20, shared=9, scale=0.6)),
], side=5)
# B: sizes that the matrix-core kernels take (keys of 16 and values of 48: stored at one padded size in bfloat16), the first layer
# recurrent, an odd number of experts a token, a rotation of part of a head.
LUBAVIK_B = model(256, 128, [
    with_mlp(mlstm(2, 64, 32, 9.0), dense(200)),
    with_mlp(attention(8, 2, 16, 48, 0.3, rot=(10000.0, 8)), moe(8, 3, 64, shared=32, scale=2.0)),
    with_mlp(parallel(chunked(4, 4, 32, 16, 0.25, size=40, rot=(500.0, 32)), linear(2, 24, 40, 12.0), 1.4, 0.6), moe(6, 2, 40, shared=24)),
    with_mlp(attention(4, 2, 16, 48, 0.5, kv_from=1, rot=(10000.0, 8)), dense(96)),
    with_mlp(mlstm(4, 16, 24, 5.0), moe(8, 2, 32)),
], side=16, eps=1e-6)
# C: sizes in steps of 8 that are no multiples of 16, chunks of five, one head, every expert chosen, no rotation, weights of the pair at 1.
LUBAVIK_C = model(97, 72, [
    with_mlp(parallel(chunked(3, 1, 40, 24, 0.15, size=5), linear(1, 8, 24, 1.0)), moe(3, 3, 16, shared=8)),
    with_mlp(attention(1, 1, 24, 8, 0.2), None),
    with_mlp(mlstm(1, 8, 8, 20.0), dense(24)),
    with_mlp(attention(3, 1, 24, 8, 0.4, kv_from=1), moe(1, 1, 40, scale=3.0)),
], side=24)
# D: heads of real sizes (64 over values of 128; states of 128 x 64, 24 x 136 and 40 x 300), chunks of one position and of 64, one expert.
LUBAVIK_D = model(64, 48, [
    with_mlp(parallel(chunked(2, 1, 64, 128, 0.125, size=64, rot=(1e4, 64)), linear(1, 128, 64, 16.0), 0.5, 2.0), moe(1, 1, 24)),
    with_mlp(mlstm(1, 128, 64, 15.0), moe(2, 1, 24, shared=16)),
    with_mlp(attention(2, 2, 64, 64, 0.125, rot=(1e6, 64)), dense(64)),
    with_mlp(parallel(chunked(2, 2, 12, 20, 0.3, size=1), linear(2, 24, 136, 8.0), 1.0, -0.5), None),
    with_mlp(mlstm(2, 40, 300, 6.0), dense(16)),
], side=8)
MODELS = {"A": LUBAVIK_A, "B": LUBAVIK_B, "C": LUBAVIK_C, "D": LUBAVIK_D}
RANKS = {"A": 3, "B": 8, "C": 11, "D": 16}


def single_layer(layer, mlp=None, width=100, side=7) -> dict:
    """A model of one layer with the mixer of `layer` and the feed-forward `mlp`."""
    return model(131, width, [with_mlp(layer, mlp)], side)


def ranked_config(cfg: dict, rank: int):
    """The configuration of a model whose decays' low-rank pairs have rank `rank` (a checkpoint's shapes give it)."""
    from gibbs_amd.config import config_from_dict
    shapes = {f"l{i}.mix.right.a1": (rank, cfg["width"]) for i, l in enumerate(cfg["layers"]) if l["type"] == "parallel"}
    return config_from_dict(cfg, tensors=shapes)


def make_model_dir(folder: str, cfg: dict, name: str, seed: int = 0, std: float = 0.1, bias_std: float = 0.5, gain_std: float = 0.3, rank: int = 6) -> str:
    """Writes a model of configuration `cfg` through the framework's random-weights mode: matrices in bfloat16, so that
    both precisions of the engine and the plain implementation start from the same values; gains, biases and sinks spread widely
    so that leaving one out shows, and the second table's rows of the stream's own size.  A head's read-out is divided by its
    root mean square: where k . q of the tokens that a state holds nearly cancels, the rounding of the operands decides what the
    row is, in any precision.  So the recurrences' keys are made to resemble their queries, and their input gates not too sharp: the
    row's own token then speaks for itself."""
    from gibbs_amd.parts import DecoderModel
    from gibbs_amd.weights import write_random_model
    config = ranked_config(cfg, rank)
    decls = DecoderModel(config.model_spec()).tensor_decls()
    path = os.path.join(folder, f"lubavik_{name}_{seed}")
    write_random_model(path, config, decls, seed=seed, dtype="bfloat16", std=std, gain_std=gain_std, bias_std=bias_std)

    def edit(w):
        w["embed"] *= 5.0
        if "side.embed" in w:
            w["side.embed"] *= 10.0
        for name in list(w):
            if name.endswith(".mix.i"):
                w[name] *= 0.3
            if name.endswith((".mix.i", ".right.a1")):
                p = name.rsplit(".", 1)[0]
                w[p + ".k"] = 0.8 * w[p + ".q"] + 0.4 * w[p + ".k"]
    return edited(path, folder, "made", edit)


def settle_choices(model_dir: str, folder: str) -> str:
    """A copy of a model folder whose routers always choose clearly: channel 0 of the stream is the same clear value for every
    token (the embedding's, which no sublayer adds to), and a router's outputs lie far apart along it (in a shuffled order), the
    rest of its matrix a fiftieth of what it was: every token of a layer takes the same experts, with weights that still differ
    from token to token.  Another precision cannot choose differently on such a model, so all of its rows can be held to a bound."""
    rng = np.random.default_rng(11)

    def edit(w):
        w["embed"][:, 0] = 1.0
        for name in sorted(w):
            if name.endswith((".norm1", ".norm2")):
                w[name][0] = -1.0
            if name.endswith(".side.norm"):
                w[name][0] = 0.0
            if name.endswith(".mlp.router"):
                n = w[name].shape[0]
                w[name] *= 0.02
                w[name][:, 0] = w[name].new_tensor((rng.permutation(n) - n / 2) * 0.5)
    return edited(model_dir, folder, "settled", edit)


def clear_tokens(model_dir: str, seed: int, n: int, vocab: int, clear: float, tries: int = 6) -> list:
    """Of a few random sequences, the one whose first unclear choice of experts (`plain_margins` below `clear`) comes latest:
    what follows such a token in a sequence may depend on a choice that another precision makes differently."""
    best, best_at = None, -1
    for k in range(tries):
        ids = tokens(seed * 1000 + k, n, vocab)
        unclear = np.nonzero(plain_margins(model_dir, ids) < clear)[0]
        at = int(unclear[0]) if unclear.size else n
        if at > best_at:
            best, best_at = ids, at
        if at == n:
            break
    return best


_models: dict = {}
_logits: dict = {}
_margins: dict = {}


def plain_logits(model_dir: str, ids) -> np.ndarray:
    key = (model_dir, tuple(ids))
    if key not in _logits:
        if model_dir not in _models:
            _models[model_dir] = load_model_dir(model_dir)
        cfg, w = _models[model_dir]
        margins = []
        _logits[key] = Z.forward(cfg, w, list(ids), margins_out=margins)
        _margins[key] = np.min(margins, axis=0) if margins else np.full(len(ids), np.inf)
    return _logits[key]


def plain_margins(model_dir: str, ids) -> np.ndarray:
    """Per token, how clear the least clear choice of experts among the model's layers is (`Z.route_margin`)."""
    plain_logits(model_dir, ids)
    return _margins[(model_dir, tuple(ids))]


_amplified: dict = {}


def amplification(model_dir: str, ids) -> np.ndarray:
    """Per row, how much more the logits move (relative L2) than the weights do, under the larger of two random relative perturbations
    of all weights of 1e-6; about ten for an ordinary row.  A read-out that nearly cancels, a feed-forward with few active
    channels and the norms behind them make a few rows in a hundred amplify rounding by hundreds: no two computations of such a
    row agree as closely as of others."""
    key = (model_dir, tuple(ids))
    if key not in _amplified:
        plain = plain_logits(model_dir, ids)
        cfg, w = _models[model_dir]
        moved = []
        for seed in range(2):
            rng = np.random.default_rng(seed)
            moved.append(Z.forward(cfg, {k: v * (1.0 + 1e-6 * rng.normal(size=v.shape)) for k, v in w.items()}, list(ids)))
        _amplified[key] = np.max([np.sqrt(((m - plain) ** 2).sum(-1) / (plain ** 2).sum(-1)) for m in moved], axis=0) / 1e-6
    return _amplified[key]
