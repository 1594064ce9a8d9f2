"""Plain Gumozen forward pass: whole sequences, no cache, one function per mechanism.

Written from the design's equations in float64 (rotation angles in float32, as the design computes them).  Nothing
from the product package is imported; the engine is held against this in both of its precisions.

Notation: T tokens, W model width; a linear weight is stored [out, in] and applied as h @ W.T.  The stream starts as the
normed embedding; a layer adds two sublayers' results, each normed and scaled channel by channel on its way in, and the
sublayers read the stream itself (the mixer after mixing every token's row with the row before it).
"""
from __future__ import annotations

import numpy as np

F64 = np.float64


# --------------------------------------------------------------------------- small functions
def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def rms_unit(x, eps: float) -> np.ndarray:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def token_shift(h, mu) -> np.ndarray:
    """Row t becomes h_t + (h_(t-1) - h_t) mu, channel by channel; the row before the first is zeros."""
    before = np.vstack([np.zeros((1, h.shape[1]), dtype=F64), h[:-1]])
    return h + (before - h) * mu[None, :]


# --------------------------------------------------------------------------- rotation
def frequencies(base: float, dims: int, scaling=None) -> np.ndarray:
    """f_i = base^(-2i/dims), i = 0 .. dims/2 - 1, in float32.  `scaling` (factor, low, high, original): frequencies whose
    wavelength l = 2 pi / f is below original / high stay, above original / low they are divided by the factor, between
    the two the kept and the divided one are mixed with s = (original / l - low) / (high - low) for the kept one."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling is not None:
            factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            wavelength = 2.0 * np.pi / f
            if wavelength > original / low:
                f = f / factor
            elif not wavelength < original / high:
                s = (original / wavelength - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return np.array(out, dtype=F64).astype(np.float32)


def rotate(x, positions, freq, dims: int) -> np.ndarray:
    """Turns the pairs (i, i + dims/2) of the first `dims` entries of the last axis of x [T, heads, n] by the angle
    float32(p) * freq[i]; the other entries pass."""
    half = dims // 2
    ang = (np.asarray(positions, dtype=np.float32)[:, None] * freq[None, :]).astype(np.float32).astype(F64)
    cos, sin = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.astype(F64).copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * cos - v * sin
    out[..., half:dims] = v * cos + u * sin
    return out


# --------------------------------------------------------------------------- attention
def visible_chunk(T: int, size) -> np.ndarray:
    """[i, j]: j <= i and both in the same stretch of `size` positions counted from 0 (None: every earlier position)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i // size == j // size)


def softmax_attention(q, k, v, scale: float, visible) -> np.ndarray:
    """q [T, H, D] over k [T, G, D], v [T, G, V] where `visible` [T, T] says so; query head h reads kv head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = np.where(visible, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        e = np.exp(s - s.max(-1, keepdims=True))
        out[:, h] = (e / e.sum(-1, keepdims=True)) @ v[:, g]
    return out


def combination_weight(lq1, lk1, lq2, lk2, diff: float) -> float:
    """How much of the second map is taken off the first."""
    return float(np.exp((lq1 * lk1).sum()) - np.exp((lq2 * lk2).sum()) + diff)


def differential_attention_mixer(h, w, p: str, m: dict, positions, eps: float) -> np.ndarray:
    """Two attention maps per head over the same values, o = a_1 - lambda a_2, divided by its root mean square, times
    1 - diff, times one sigmoid gate per head."""
    H, G, D, V = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ w[p + "q"].T).reshape(T, H, 2, D)
    k = (h @ w[p + "k"].T).reshape(T, G, 2, D)
    v = (h @ w[p + "v"].T).reshape(T, G, V)
    rot = m.get("rot")
    maps = []
    for c in range(2):
        qc = rms_unit(q[:, :, c], eps) * w[p + "q.norm"]
        kc = rms_unit(k[:, :, c], eps) * w[p + "k.norm"]
        if rot is not None and int(rot.get("dims", 0)) > 0:
            freq = frequencies(rot["base"], int(rot["dims"]), rot.get("scaling"))
            qc, kc = rotate(qc, positions, freq, int(rot["dims"])), rotate(kc, positions, freq, int(rot["dims"]))
        size = (m.get("mask") or {}).get("size")
        maps.append(softmax_attention(qc, kc, v, float(m["scale"]), visible_chunk(T, None if size is None else int(size))))
    diff = float(m["diff"])
    lam = combination_weight(w[p + "lq1"], w[p + "lk1"], w[p + "lq2"], w[p + "lk2"], diff)
    o = rms_unit(maps[0] - lam * maps[1], eps) * (1.0 - diff)
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * V) @ w[p + "o"].T


def latent(h, w, p: str, eps: float) -> np.ndarray:
    """The small row per token that a latent attention's keys and values are made of."""
    return rms_unit(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]


def latent_attention_mixer(h, c, w, p: str, m: dict, eps: float) -> np.ndarray:
    """Attention without positions whose keys and values are W_uk c and W_uv c; every earlier token is seen."""
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    cq = rms_unit(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).reshape(T, H, D)
    k = (c @ w[p + "uk"].T).reshape(T, H, D)
    v = (c @ w[p + "uv"].T).reshape(T, H, V)
    o = softmax_attention(q, k, v, float(m["scale"]), visible_chunk(T, None))
    return o.reshape(T, H * V) @ w[p + "o"].T


# --------------------------------------------------------------------------- gated linear recurrence
def forget_gate(z, bias, lower) -> np.ndarray:
    """A gate per channel that never falls below `lower`."""
    return lower + (1.0 - lower) * sigmoid(z + bias)


def gated_outer_scan(q, f, v) -> np.ndarray:
    """Per head a state S [D, V] from zero: S <- diag(f_t) S + (1 - f_t) v_t', read-out S' q_t.  q, f [T, H, D], v [T, H, V]."""
    T, H, D = q.shape
    V = v.shape[2]
    o = np.zeros((T, H, V), dtype=F64)
    for h in range(H):
        S = np.zeros((D, V), dtype=F64)
        for t in range(T):
            S = f[t, h][:, None] * S + np.outer(1.0 - f[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def hgrn2_mixer(h, w, p: str, m: dict, eps: float) -> np.ndarray:
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = silu(h @ w[p + "q"].T).reshape(T, H, D)
    f = forget_gate(h @ w[p + "f"].T, w[p + "f.b"], w[p + "lower"]).reshape(T, H, D)
    v = (h @ w[p + "v"].T).reshape(T, H, V)
    o = rms_unit(gated_outer_scan(q, f, v), eps) * w[p + "norm"]
    return o.reshape(T, H * V) @ w[p + "o"].T


# --------------------------------------------------------------------------- experts
def route(h, router, top: int):
    """Scores sigmoid(router h); the `top` largest (the lower index among equals) and, as weights, their scores.
    -> (chosen [T, top], weights [T, top])."""
    s = sigmoid(h @ router.T)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1)


def route_margin(h, router, top: int) -> np.ndarray:
    """Per row, how far the last chosen expert's score lies above the best one that was not chosen (inf where every expert
    is chosen): a choice closer than the rounding of h may fall the other way in another precision."""
    s = np.sort(sigmoid(h @ router.T), axis=-1)[:, ::-1]
    return s[:, top - 1] - s[:, top] if top < s.shape[1] else np.full(h.shape[0], np.inf)


def expert(h, gate, up, down) -> np.ndarray:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def moe_ff(h, w, p: str, mlp: dict, margins_out=None) -> np.ndarray:
    """sum over the chosen experts of expert(weight * h): the weight goes in with the row."""
    top = int(mlp["router"]["top"])
    chosen, weights = route(h, w[p + "router"], top)
    if margins_out is not None:
        margins_out.append(route_margin(h, w[p + "router"], top))
    out = np.zeros_like(h, dtype=F64)
    for e in range(int(mlp["router"]["experts"])):
        for c in range(top):
            at = np.nonzero(chosen[:, c] == e)[0]
            if at.size:
                q = f"{p}e{e}."
                out[at] += expert(weights[at, c][:, None] * h[at], w[q + "gate"], w[q + "up"], w[q + "down"])
    return out


# --------------------------------------------------------------------------- the model
def forward(cfg: dict, weights: dict, tokens, return_layers: bool = False, margins_out=None):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer, [layers, T, W]).  `margins_out`: a list
    that receives every expert layer's `route_margin` per token."""
    w = {k: np.asarray(v, dtype=F64) for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    T = len(tokens)
    positions = np.arange(T)
    x = rms_unit(w["embed"][np.asarray(tokens)], eps) * w["embed.norm"]
    latents: dict = {}
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = token_shift(x, w[p + "shift"])
        if layer["type"] == "attention":
            d = differential_attention_mixer(h, w, p + "mix.", m, positions, eps)
        elif layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                latents[i] = latent(h, w, p + "mix.", eps)
            d = latent_attention_mixer(h, latents[i if m.get("kv_from") is None else int(m["kv_from"])], w, p + "mix.", m, eps)
        elif layer["type"] == "hgrn2":
            d = hgrn2_mixer(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + rms_unit(d, eps) * w[p + "norm1"] * w[p + "ls1"]
        if layer.get("mlp") is not None:
            x = x + rms_unit(moe_ff(x, w, p + "mlp.", layer["mlp"], margins_out), eps) * w[p + "norm2"] * w[p + "ls2"]
        after.append(x.copy())
    logits = (rms_unit(x, eps) * w["final.norm"]) @ w["head"].T
    return (logits, np.stack(after)) if return_layers else logits
