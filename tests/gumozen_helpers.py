"""Small Gumozen configurations that differ in every size and option, model folders made from them through the
framework's random-weights mode, and the plain implementation's logits for them."""
from __future__ import annotations

import json
import os

import numpy as np

from tests.plain import gumozen_plain as Z


def differential(heads, kv, dim, vdim, scale, diff, size=None, rot=None, scaling=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if size is not None:
        m["mask"] = {"size": size}
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "attention", "mixer": m}


def recurrence(heads, dim, vdim):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def latent(heads, dim, vdim, kv_rank, q_rank, scale, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


def model(vocab, width, layers, eps=1e-5):
    return {"architecture": "Gumozen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# A: no size a multiple of 8 where it can be avoided (the plain kernels in both precisions); two latent layers read the first
# one's latent, with other head counts and value sizes; scores that stand out (scales well above 1 / sqrt(dim)), so that single
# keys far back carry weight; a layer without a feed-forward; three experts of seven.
GUMOZEN_A = model(211, 100, [
    with_mlp(latent(5, 6, 9, 11, 13, 1.2), moe(7, 3, 30)),
    with_mlp(differential(6, 3, 10, 14, 0.9, 0.35, size=13, rot=(1000.0, 6), scaling=(4.0, 1.0, 4.0, 64)), moe(5, 2, 22)),
    with_mlp(recurrence(3, 7, 10), None),
    with_mlp(latent(3, 10, 7, 11, 17, 0.8, kv_from=0), moe(4, 1, 45)),
    with_mlp(differential(4, 4, 6, 9, 1.1, 0.6), moe(3, 2, 18)),
    with_mlp(latent(2, 5, 12, 11, 9, 1.5, kv_from=0), moe(2, 1, 20)),
])
# B: sizes that the matrix-core kernels take (keys of 2 x 16, values of 48: stored at one padded size in bfloat16), the first
# layer recurrent, an odd number of experts a token.
GUMOZEN_B = model(256, 128, [
    with_mlp(recurrence(2, 64, 32), moe(8, 3, 64)),
    with_mlp(differential(4, 2, 16, 48, 0.3, 0.2, size=40, rot=(10000.0, 16), scaling=(8.0, 1.0, 4.0, 128)), moe(8, 2, 32)),
    with_mlp(latent(4, 32, 16, 48, 56, 0.2), moe(4, 1, 64)),
    with_mlp(recurrence(4, 24, 40), moe(6, 2, 40)),
    with_mlp(latent(8, 16, 24, 48, 32, 0.25, kv_from=2), moe(4, 2, 24)),
], eps=1e-6)
# C: sizes in steps of 8 that are no multiples of 16, chunks of five, a rotation of part of a map without scaling, every expert
# chosen, values smaller than a map.
GUMOZEN_C = model(97, 72, [
    with_mlp(differential(3, 1, 40, 24, 0.15, 0.8, size=5, rot=(100.0, 8)), moe(3, 3, 16)),
    with_mlp(latent(3, 8, 8, 24, 24, 0.4), None),
    with_mlp(recurrence(9, 8, 8), moe(2, 2, 24)),
    with_mlp(latent(6, 24, 16, 24, 40, 0.2, kv_from=1), moe(1, 1, 40)),
])
# D: heads of real sizes: maps of 64 over values of 128, a recurrence of 128 x 64 and one of 24 x 136, a cached latent of 128;
# chunks of one position; one expert.
GUMOZEN_D = model(64, 48, [
    with_mlp(differential(2, 1, 64, 128, 0.125, 0.5, size=64, rot=(1e4, 64), scaling=(2.0, 1.0, 2.0, 32)), moe(1, 1, 24)),
    with_mlp(recurrence(1, 128, 64), moe(2, 1, 24)),
    with_mlp(latent(2, 64, 64, 128, 40, 0.125), moe(3, 1, 16)),
    with_mlp(differential(2, 2, 12, 20, 0.3, 0.1, size=1), moe(2, 2, 16)),
    with_mlp(recurrence(2, 24, 136), None),
])
MODELS = {"A": GUMOZEN_A, "B": GUMOZEN_B, "C": GUMOZEN_C, "D": GUMOZEN_D}


def single_layer(layer, mlp=None, width=100) -> dict:
    """A model of one layer with the mixer of `layer` and the feed-forward `mlp`."""
    return model(131, width, [with_mlp(layer, mlp)])


def make_model_dir(folder: str, cfg: dict, name: str, seed: int = 0, std: float = 0.1, bias_std: float = 0.5, gain_std: float = 0.3) -> str:
    """Writes a model of configuration `cfg` through the framework's random-weights mode: matrices in bfloat16, so that
    both precisions of the engine and the plain implementation start from the same values; gains, biases, scales and lower
    bounds spread widely so that leaving one out shows."""
    from gibbs_amd.config import config_from_dict
    from gibbs_amd.parts import DecoderModel
    from gibbs_amd.weights import write_random_model
    config = config_from_dict(cfg)
    decls = DecoderModel(config.model_spec()).tensor_decls()
    path = os.path.join(folder, f"gumozen_{name}_{seed}")
    write_random_model(path, config, decls, seed=seed, dtype="bfloat16", std=std, gain_std=gain_std, bias_std=bias_std)
    return path


def edited(model_dir: str, folder: str, suffix: str, edit) -> str:
    """A copy of a model folder whose weights (name -> float32 tensor) went through `edit`; matrices stay in bfloat16."""
    import shutil
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, os.path.basename(model_dir) + "_" + suffix)
    os.makedirs(path, exist_ok=True)
    shutil.copy(os.path.join(model_dir, "config.json"), os.path.join(path, "config.json"))
    w = load_file(os.path.join(model_dir, "model.safetensors"))
    types = {k: v.dtype for k, v in w.items()}
    w = {k: v.float() for k, v in w.items()}
    edit(w)
    save_file({k: v.to(types[k]).contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return path


def settle_choices(model_dir: str, folder: str) -> str:
    """A copy of a model folder whose routers always choose clearly: channel 0 of the stream is the same clear value for every
    token (the embedding's, which no sublayer adds to), and a router's outputs lie far apart along it (in a shuffled order), the
    rest of its matrix a fiftieth of what it was: every token of a layer takes the same experts, with weights that still differ
    from token to token.  Another precision cannot choose differently on such a model, so all of its rows can be held to a bound."""
    rng = np.random.default_rng(11)

    def edit(w):
        w["embed"][:, 0] = 0.2
        w["embed.norm"][0] = 1.0
        for name in sorted(w):
            if name.endswith((".norm1", ".norm2")):
                w[name][0] = 0.0
            if name.endswith(".mlp.router"):
                n = w[name].shape[0]
                w[name] *= 0.02
                w[name][:, 0] = w[name].new_tensor((rng.permutation(n) - n / 2) * 0.25)
    return edited(model_dir, folder, "settled", edit)


def tokens(seed: int, n: int, vocab: int) -> list:
    return np.random.default_rng(seed).integers(0, vocab, size=n).tolist()


def load_model_dir(model_dir: str):
    """(config, name -> float64 array) of a model folder, read with the safetensors package."""
    from safetensors.torch import load_file
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    w = {k: v.double().numpy() for k, v in load_file(os.path.join(model_dir, "model.safetensors")).items()}
    return cfg, w


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
