"""Plain Lubavik forward pass: whole sequences, no cache, one function per mechanism.

Written from the design's equations in float64 (rotation angles in float32, as the design computes them).  Nothing
from the product package is imported; the engine is held against this in both of its precisions.

Notation: T tokens, W model width; a linear weight is stored [out, in] and applied as h @ W.T.  The sublayers read the
stream itself; each result is normed on its way in, and behind the feed-forward a small row of a second token table, gated by
the stream, is added as a third sublayer.
"""
from __future__ import annotations

import numpy as np

F64 = np.float64


# --------------------------------------------------------------------------- small functions
def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z):
    return -(np.maximum(-z, 0.0) + np.log1p(np.exp(-np.abs(z))))


def rms_unit(x, eps: float) -> np.ndarray:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def norm_around_one(x, w, eps: float) -> np.ndarray:
    """The model's norm: the stored weight is what the gain differs from one by."""
    return rms_unit(x, eps) * (1.0 + w)


# --------------------------------------------------------------------------- rotation
def rotate(x, positions, base: float, dims: int, neighbours: bool) -> np.ndarray:
    """Turns pairs of the first `dims` entries of the last axis of x [T, heads, n] by the angle float32(p) * f_i, f_i =
    base^(-2i/dims): pairs (2i, 2i + 1) with `neighbours`, else (i, i + dims/2); the other entries pass."""
    half = dims // 2
    freq = np.array([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=F64).astype(np.float32)
    ang = (np.asarray(positions, dtype=np.float32)[:, None] * freq[None, :]).astype(np.float32).astype(F64)
    cos, sin = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if neighbours else (slice(0, half), slice(half, dims))
    out = x.astype(F64).copy()
    u, v = x[..., first], x[..., second]
    out[..., first] = u * cos - v * sin
    out[..., second] = v * cos + u * sin
    return out


# --------------------------------------------------------------------------- attention
def visible_chunk(T: int, size) -> np.ndarray:
    """[i, j]: j <= i and both in the same stretch of `size` positions counted from 0 (None: every earlier position)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i // size == j // size)


def softmax_attention(q, k, v, scale: float, visible, sink=None) -> np.ndarray:
    """q [T, H, D] over k [T, G, D], v [T, G, V] where `visible` [T, T] says so; query head h reads kv head h // (H / G).  `sink` [H]:
    one more term exp(sink_h) in the denominator."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = np.where(visible, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        top = s.max(-1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        e = np.exp(s - top)
        total = e.sum(-1, keepdims=True) + (np.exp(sink[h] - top) if sink is not None else 0.0)
        out[:, h] = (e / total) @ v[:, g]
    return out


def own_keys_values(h, w, p: str, m: dict, positions, eps: float):
    """Keys (normed over the whole projection, rotated) and values of an attention layer that has its own."""
    T, G, D, V = h.shape[0], int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    k = (rms_unit(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(T, G, D)
    rot = m.get("rot") or {}
    if int(rot.get("dims", 0)) > 0:
        k = rotate(k, positions, rot["base"], int(rot["dims"]), neighbours=False)
    return k, (h @ w[p + "v"].T).reshape(T, G, V)


def sink_attention_mixer(h, k, v, w, p: str, m: dict, positions, eps: float) -> np.ndarray:
    """Queries of this layer over keys and values that may be another layer's."""
    T, H, D, V = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (rms_unit(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(T, H, D)
    rot = m.get("rot") or {}
    if int(rot.get("dims", 0)) > 0:
        q = rotate(q, positions, rot["base"], int(rot["dims"]), neighbours=False)
    o = softmax_attention(q, k, v, float(m["scale"]), visible_chunk(T, None), w[p + "sink"])
    return o.reshape(T, H * V) @ w[p + "o"].T


def chunked_attention_mixer(h, w, p: str, m: dict, positions, eps: float) -> np.ndarray:
    """Projections with biases, q and k normed per head, neighbours rotated, a softmax over the row's own chunk."""
    T, H, G, D, V = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, D)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, V)
    q, k = rms_unit(q, eps) * w[p + "q.norm"], rms_unit(k, eps) * w[p + "k.norm"]
    rot = m.get("rot") or {}
    if int(rot.get("dims", 0)) > 0:
        q, k = (rotate(x, positions, rot["base"], int(rot["dims"]), neighbours=True) for x in (q, k))
    size = (m.get("mask") or {}).get("size")
    o = softmax_attention(q, k, v, float(m["scale"]), visible_chunk(T, None if size is None else int(size)))
    return o.reshape(T, H * V) @ w[p + "o"].T + w[p + "o.b"]


# --------------------------------------------------------------------------- recurrences
def decayed_outer_scan(q, k, v, alpha) -> np.ndarray:
    """Per head a state S [D, V] from zero: S <- diag(alpha_t) S + k_t v_t', read-out S' q_t.  q, k, alpha [T, H, D], v [T, H, V]."""
    T, H, D = q.shape
    o = np.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        S = np.zeros((D, v.shape[2]), dtype=F64)
        for t in range(T):
            S = alpha[t, h][:, None] * S + np.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def gated_linear_mixer(h, w, p: str, m: dict, eps: float) -> np.ndarray:
    """Linear attention whose state decays channel by channel, alpha = sigmoid(z)^(1/tau), z from a low-rank pair."""
    T, H, D, V = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[p + "q"].T).reshape(T, H, D) / np.sqrt(D)
    k = (h @ w[p + "k"].T).reshape(T, H, D)
    v = (h @ w[p + "v"].T).reshape(T, H, V)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = np.exp(log_sigmoid(z) / float(m["tau"])).reshape(T, H, D)
    o = rms_unit(decayed_outer_scan(q, k, v, alpha), eps) * w[p + "norm"]
    return (o.reshape(T, H * V) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, w, p: str, m: dict, positions, eps: float) -> np.ndarray:
    return (float(m["left_scale"]) * chunked_attention_mixer(h, w, p + "left.", m["left"], positions, eps)
            + float(m["right_scale"]) * gated_linear_mixer(h, w, p + "right.", m["right"], eps))


def stabilised_matrix_scan(q, k, v, log_in, log_keep) -> np.ndarray:
    """A matrix memory with a normaliser, both kept relative to exp(m), m a running maximum from 0: per head and token
    m' = max(log_keep + m, log_in); S and n decay by exp(log_keep + m - m') and take exp(log_in - m') times k v' and k; the
    read-out is S' q over max(|n . q|, exp(-m')) + 1e-6.  q, k [T, H, D], v [T, H, V], log_in, log_keep [T, H]."""
    T, H, D = q.shape
    V = v.shape[2]
    o = np.zeros((T, H, V), dtype=F64)
    for h in range(H):
        S, n, m = np.zeros((D, V), dtype=F64), np.zeros(D, dtype=F64), 0.0
        for t in range(T):
            above = max(log_keep[t, h] + m, log_in[t, h])
            keep, take = np.exp(log_keep[t, h] + m - above), np.exp(log_in[t, h] - above)
            S = keep * S + take * np.outer(k[t, h], v[t, h])
            n = keep * n + take * k[t, h]
            m = above
            o[t, h] = (S.T @ q[t, h]) / (max(abs(n @ q[t, h]), np.exp(-m)) + 1e-6)
    return o


def mlstm_mixer(h, w, p: str, m: dict, eps: float) -> np.ndarray:
    T, H, D, V = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    cap = float(m["gate_cap"])
    q = (h @ w[p + "q"].T).reshape(T, H, D) / np.sqrt(D)
    k = (h @ w[p + "k"].T).reshape(T, H, D)
    v = (h @ w[p + "v"].T).reshape(T, H, V)
    log_in = cap * np.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    log_keep = log_sigmoid(cap * np.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    o = rms_unit(stabilised_matrix_scan(q, k, v, log_in, log_keep), eps).reshape(T, H * V)
    return (o * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# --------------------------------------------------------------------------- feed-forwards
def squared_relu_ff(h, w, p: str) -> np.ndarray:
    return (np.maximum(h @ w[p + "up"].T, 0.0) ** 2) @ w[p + "down"].T


def softmax_rows(z):
    e = np.exp(z - z.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def route(h, router, top: int, scale: float):
    """Scores by a softmax over all outputs; the `top` largest (the lower index among equals) and, as weights, their scores over
    their sum, times `scale`.  -> (chosen [T, top], weights [T, top])."""
    s = softmax_rows(h @ router.T)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    best = np.take_along_axis(s, chosen, axis=-1)
    return chosen, best / (best.sum(-1, keepdims=True) + 1e-20) * scale


def route_margin(h, router, top: int) -> np.ndarray:
    """Per row, how far the last chosen expert's logit lies above the best one that was not chosen (inf where every expert
    is chosen): a choice closer than the rounding of h may fall the other way in another precision."""
    z = np.sort(h @ router.T, axis=-1)[:, ::-1]
    return z[:, top - 1] - z[:, top] if top < z.shape[1] else np.full(h.shape[0], np.inf)


def expert(h, gate, up, down) -> np.ndarray:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def moe_ff(h, w, p: str, mlp: dict, margins_out=None) -> np.ndarray:
    top = int(mlp["router"]["top"])
    chosen, weights = route(h, w[p + "router"], top, float(mlp["router"].get("scale", 1.0)))
    if margins_out is not None:
        margins_out.append(route_margin(h, w[p + "router"], top))
    out = np.zeros_like(h, dtype=F64)
    for e in range(int(mlp["router"]["experts"])):
        for c in range(top):
            at = np.nonzero(chosen[:, c] == e)[0]
            if at.size:
                q = f"{p}e{e}."
                out[at] += weights[at, c][:, None] * expert(h[at], w[q + "gate"], w[q + "up"], w[q + "down"])
    if mlp.get("shared") is not None:
        q = p + "shared."
        out = out + expert(h, w[q + "gate"], w[q + "up"], w[q + "down"])
    return out


# --------------------------------------------------------------------------- a second table's row
def token_side(x, rows, gate, proj) -> np.ndarray:
    """rows [T, d]: the tokens' entries of a second table, times gelu(gate x), projected to the width."""
    return (gelu_tanh(x @ gate.T) * rows) @ proj.T


# --------------------------------------------------------------------------- the model
def forward(cfg: dict, weights: dict, tokens, return_layers: bool = False, margins_out=None):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer, [layers, T, W]).  `margins_out`: a list
    that receives every expert layer's `route_margin` per token."""
    w = {k: np.asarray(v, dtype=F64) for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    ids = np.asarray(tokens)
    positions = np.arange(len(ids))
    x = w["embed"][ids]
    cached: dict = {}
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        if layer["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                cached[i] = own_keys_values(x, w, p + "mix.", m, positions, eps)
            k, v = cached[i if src is None else int(src)]
            d = sink_attention_mixer(x, k, v, w, p + "mix.", m, positions, eps)
        elif layer["type"] == "parallel":
            d = parallel_mixer(x, w, p + "mix.", m, positions, eps)
        elif layer["type"] == "mlstm":
            d = mlstm_mixer(x, w, p + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + norm_around_one(d, w[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            f = squared_relu_ff(x, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(x, w, p + "mlp.", mlp, margins_out)
            x = x + norm_around_one(f, w[p + "norm2"], eps)
        if cfg.get("token_side") is not None:
            n = int(cfg["token_side"]["dim"])
            y = token_side(x, w["side.embed"][ids, i * n:(i + 1) * n], w[p + "side.gate"], w[p + "side.proj"])
            x = x + rms_unit(y, eps) * w[p + "side.norm"]
        after.append(x.copy())
    logits = norm_around_one(x, w["final.norm"], eps) @ w["head"].T
    return (logits, np.stack(after)) if return_layers else logits
