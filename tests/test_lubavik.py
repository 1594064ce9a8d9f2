"""Lubavik without a GPU: the configuration reader, the model it describes, the tensors it declares, and the plain
implementation's mechanisms against hand-made cases."""
import copy

import numpy as np
import pytest

from tests import lubavik_helpers as LH
from tests.plain import lubavik_plain as Z


def test_registry_and_layers():
    from gibbs_amd.config import LubavikConfig, config_from_dict
    cfg = config_from_dict(LH.LUBAVIK_A)
    assert isinstance(cfg, LubavikConfig) and cfg.to_dict() == LH.LUBAVIK_A
    spec = cfg.model_spec()
    assert spec.order == (0, 1, 2, 3, 4) and spec.head == "head" and spec.embedding == "embed" and spec.embedding_norm is None
    assert spec.final_norm.offset == 1.0 and spec.final_norm.eps == 1e-5
    assert [ls.arrangement for ls in spec.layers] == ["post_norm"] * 5
    assert [r for r, _ in spec.layers[0].parts] == ["mixer", "norm1", "ffn", "norm2", "side", "side_norm"]
    assert [r for r, _ in spec.layers[1].parts] == ["left", "right", "norm1", "ffn", "norm2", "side", "side_norm"]
    assert [r for r, _ in spec.layers[2].parts] == ["mixer", "norm1", "side", "side_norm"]
    assert [ls.parts[0][1].kind for ls in spec.layers] == ["attention", "attention", "attention", "matrix_lstm", "attention"]
    assert spec.layers[1].part("right").kind == "gated_linear" and spec.layers[1].params == {"left_scale": 0.9, "right_scale": 1.6}
    assert spec.layers[0].part("norm1").offset == 1.0 and spec.layers[0].part("side_norm").offset == 0.0
    assert cfg.derived()["layers_by_type"] == {"attention": 3, "parallel": 1, "mlstm": 1} and cfg.derived()["reads_cache_of"] == {"2": 0, "4": 0}


def test_constants_come_from_the_configuration():
    spec = LH.ranked_config(LH.LUBAVIK_A, 3).model_spec()
    a = spec.layers[0].part("mixer")
    assert a.params == {"heads": 6, "kv_heads": 3, "head_dim": 10, "v_head_dim": 14, "scale": 0.7, "chunk": 0, "qk_norm": "whole", "qk_norm_eps": 1e-5, "sink": True}
    assert a.position.params == {"theta": 1000.0, "rotary_dim": 6, "variant": "half_split", "precision": "f64"}
    reads = spec.layers[2].part("mixer")
    assert reads.params["kv_source"] == 0 and reads.params["scale"] == 0.5 and "k_proj" not in reads.tensors and "v_proj" not in reads.tensors
    assert spec.layers[4].part("mixer").position is None
    left, right = spec.layers[1].part("left"), spec.layers[1].part("right")
    assert left.params["chunk"] == 13 and left.params["qk_norm"] == "before" and left.params["bias"] and left.params["out_bias"]
    assert left.position.params["variant"] == "interleaved" and left.position.params["rotary_dim"] == 4
    assert right.params == {"heads": 3, "dim": 9, "vdim": 15, "rank": 3, "tau": 4.0, "norm_eps": 1e-5}
    assert spec.layers[3].part("mixer").params == {"heads": 3, "dim": 11, "vdim": 14, "gate_cap": 3.0, "norm_eps": 1e-5}
    ff = spec.layers[0].part("ffn")
    assert ff.kind == "moe" and (ff.params["experts"], ff.params["top"], ff.params["inter"]) == (7, 3, 30)
    assert ff.params["scores"] == "softmax_all" and ff.params["weight_scale"] == 1.7 and ff.params["shared"] == {"inter": 22, "activation": "silu", "gate": False}
    assert spec.layers[3].part("ffn").params["shared"] is None
    assert spec.layers[1].part("ffn").params == {"inter": 45, "activation": "relu_squared"}
    side = spec.layers[3].part("side")
    assert (side.params["dim"], side.params["column"], side.params["columns"], side.params["vocab"]) == (5, 15, 25, 211) and side.params["activation"] == "gelu_tanh"
    assert [ls.part("side").params["declares_table"] for ls in spec.layers] == [True, False, False, False, False]


def test_declared_tensors_cache_and_state():
    from gibbs_amd.parts import DecoderModel
    model = DecoderModel(LH.ranked_config(LH.LUBAVIK_A, 3).model_spec())
    decls = model.tensor_decls()
    shapes = {d.name: d.shape for d in decls}
    assert len(decls) == len(shapes)
    assert shapes["embed"] == (211, 100) and shapes["side.embed"] == (211, 25) and shapes["head"] == (211, 100) and shapes["final.norm"] == (100,)
    assert shapes["l0.mix.q"] == (60, 100) and shapes["l0.mix.k"] == (30, 100) and shapes["l0.mix.v"] == (42, 100) and shapes["l0.mix.o"] == (100, 84)
    assert shapes["l0.mix.q.norm"] == (60,) and shapes["l0.mix.k.norm"] == (30,) and shapes["l0.mix.sink"] == (6,)
    assert "l2.mix.k" not in shapes and "l2.mix.k.norm" not in shapes and shapes["l2.mix.q.norm"] == (90,) and "l2.norm2" not in shapes
    assert shapes["l1.mix.left.q.b"] == (24,) and shapes["l1.mix.left.v.b"] == (18,) and shapes["l1.mix.left.o.b"] == (100,) and shapes["l1.mix.left.k.norm"] == (6,)
    assert shapes["l1.mix.right.a1"] == (3, 100) and shapes["l1.mix.right.a2"] == (27, 3) and shapes["l1.mix.right.a2.b"] == (27,) and shapes["l1.mix.right.norm"] == (15,)
    assert shapes["l3.mix.i"] == (3, 100) and shapes["l3.mix.f.b"] == (3,) and shapes["l3.mix.norm"] == (42,)
    assert shapes["l1.mlp.up"] == (45, 100) and "l1.mlp.gate" not in shapes and shapes["l0.mlp.shared.down"] == (100, 22) and "l3.mlp.shared.up" not in shapes
    assert shapes["l2.side.gate"] == (5, 100) and shapes["l2.side.proj"] == (100, 5) and shapes["l2.side.norm"] == (100,)
    owners = model.cache_owners()
    need = dict(zip(owners, model.cache_needs()))
    assert (need[(0, "mixer")].kv_heads, need[(0, "mixer")].head_dim, need[(0, "mixer")].value_dim, need[(0, "mixer")].window) == (3, 10, 14, None)
    assert (need[(1, "left")].kv_heads, need[(1, "left")].head_dim, need[(1, "left")].value_dim) == (2, 6, 9)
    assert need[(2, "mixer")] is None and need[(1, "right")] is None and need[(3, "mixer")] is None
    sources = dict(zip(owners, model.kv_sources()))
    assert owners[sources[(2, "mixer")]] == (0, "mixer") and owners[sources[(4, "mixer")]] == (0, "mixer")
    states = dict(zip(owners, model.state_needs()))
    assert [(s.name, s.shape) for s in states[(1, "right")]] == [("gated_linear_rule", (3, 9, 15))]
    assert [(s.name, s.shape) for s in states[(3, "mixer")]] == [("matrix_lstm_rule", (3, 11, 14)), ("matrix_lstm_norm", (36,))]


def test_tensors_of_a_missing_feed_forward_are_declared_and_read_by_nobody():
    from gibbs_amd.config import config_from_dict
    from gibbs_amd.parts import DecoderModel
    full = {d.name: d.shape for d in DecoderModel(LH.ranked_config(LH.LUBAVIK_A, 3).model_spec()).tensor_decls()}
    more = dict(full, **{"l2.norm2": (100,)})
    spec = config_from_dict(LH.LUBAVIK_A, tensors=more).model_spec()
    assert {d.name for d in DecoderModel(spec).tensor_decls()} == set(more) and "norm2" not in [r for r, _ in spec.layers[2].parts]


@pytest.mark.parametrize("change, words", [
    (lambda c: c["layers"][0].__setitem__("type", "mamba2"), "mixer type"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 4), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 12), "rotated"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].__setitem__("size", 0), "mask.size"),
    (lambda c: c["layers"][1]["mixer"]["left"].__setitem__("kv_from", 0), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("tau", 0.0), "tau"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 4), "kv_from"),
    (lambda c: c["layers"][4]["mixer"].__setitem__("kv_from", 2), "kv_from"),
    (lambda c: c["layers"][4]["mixer"].__setitem__("vdim", 12), "vdim"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("gate_cap", 0), "gate_cap"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("heads", 0), "heads"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 8), "experts a token"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "glu"), "feed-forward kind"),
    (lambda c: c["token_side"].__setitem__("dim", 0), "token_side"),
    (lambda c: c.pop("width"), "width"),
])
def test_refused_configurations(change, words):
    from gibbs_amd.config import ConfigError, config_from_dict
    cfg = copy.deepcopy(LH.LUBAVIK_A)
    change(cfg)
    with pytest.raises(ConfigError, match=words):
        config_from_dict(cfg)


def test_options_that_do_not_go_together():
    from gibbs_amd.config.spec import FeedForwardSpec, LayerSpec, MixerSpec, NormSpec
    from gibbs_amd.parts import build_block, build_feed_forward, build_mixer
    base = {"heads": 2, "kv_heads": 1, "head_dim": 8, "scale": 1.0}
    with pytest.raises(ValueError, match="whole projection"):
        build_mixer(MixerSpec("attention", dict(base, qk_norm="whole", bias=True), {}), 16, 0)
    with pytest.raises(ValueError, match="another layer"):
        build_mixer(MixerSpec("attention", dict(base, sink=True, kv_source=0), {}), 16, 1)
    build_mixer(MixerSpec("attention", dict(base, qk_norm="whole", sink=True, kv_source=0), {}), 16, 1)
    with pytest.raises(ValueError, match="not implemented"):
        build_feed_forward(FeedForwardSpec("mlp", {"inter": 8, "activation": "swish9"}, {}), 16)
    with pytest.raises(ValueError, match="softmax over all outputs"):
        build_feed_forward(FeedForwardSpec("moe", {"experts": 1, "top": 1, "inter": 8, "scores": "sigmoid", "weight_scale": 2.0}, {"router": "r", "gate": ("g",), "up": ("u",), "down": ("d",)}), 16)
    with pytest.raises(ValueError, match="table"):
        build_feed_forward(FeedForwardSpec("token_side", {"dim": 4, "column": 6, "columns": 8, "vocab": 5}, {}), 16)
    with pytest.raises(ValueError, match="lacks"):
        build_block(LayerSpec("l0", "post_norm", parts=[("left", MixerSpec("attention", base, {})), ("norm1", NormSpec("rms", 1e-5, "n"))]), 16, 0)


def test_segments_start_at_multiples_of_eight_rows():
    import torch
    from gibbs_amd.parts.segments import stacked_rows
    parts = [torch.full((n, 3), float(n)) for n in (5, 8, 1)]
    w, offsets = stacked_rows(parts)
    assert offsets == [0, 8, 16] and w.shape == (24, 3)
    for p, o in zip(parts, offsets):
        assert torch.equal(w[o:o + p.shape[0]], p)
    assert not w[5:8].any() and not w[17:].any()


# ----------------------------------------------------------------------------------------------- the plain mechanisms
def test_rotations_of_neighbours_and_of_halves():
    x = np.zeros((2, 1, 6))
    x[:, 0] = [1.0, 2.0, 3.0, 4.0, 5.0, 6.0]
    for neighbours, pairs in ((True, [(0, 1), (2, 3)]), (False, [(0, 2), (1, 3)])):
        y = Z.rotate(x, [0, 3], 100.0, 4, neighbours)
        assert np.array_equal(y[0], x[0]) and np.array_equal(y[1, 0, 4:], [5.0, 6.0])
        for i, (a, b) in enumerate(pairs):
            ang = 3 * 100.0 ** (-2 * i / 4)
            turned = np.exp(1j * ang) * (x[1, 0, a] + 1j * x[1, 0, b])
            assert np.allclose([y[1, 0, a], y[1, 0, b]], [turned.real, turned.imag], atol=1e-6)


def test_chunks_at_their_edges():
    c = Z.visible_chunk(10, 4)
    assert c[5].nonzero()[0].tolist() == [4, 5] and c[7].nonzero()[0].tolist() == [4, 5, 6, 7] and c[8].nonzero()[0].tolist() == [8]
    assert Z.visible_chunk(5, 1).sum() == 5 and Z.visible_chunk(4, None).sum() == 10


def test_a_sink_takes_weight_and_gives_nothing():
    q, k, v = np.ones((1, 1, 2)), np.ones((1, 1, 2)), np.full((1, 1, 3), 4.0)
    out = Z.softmax_attention(q, k, v, 0.5, np.ones((1, 1), dtype=bool), np.array([1.0]))
    assert np.allclose(out, 4.0 * np.e / (np.e + np.e))
    assert np.allclose(Z.softmax_attention(q, k, v, 0.5, np.ones((1, 1), dtype=bool), np.array([-800.0])), 4.0)


def test_the_linear_recurrence_against_its_closed_form():
    rng = np.random.default_rng(1)
    T, H, D, V = 6, 2, 3, 4
    q, k, v = rng.normal(size=(T, H, D)), rng.normal(size=(T, H, D)), rng.normal(size=(T, H, V))
    a = np.broadcast_to(rng.uniform(0.1, 0.95, size=(H, D)), (T, H, D))
    y = Z.decayed_outer_scan(q, k, v, a)
    for h in range(H):
        for t in range(T):
            want = sum((q[t, h] * a[0, h] ** (t - s) * k[s, h]).sum() * v[s, h] for s in range(t + 1))
            assert np.allclose(y[t, h], want)


def test_the_matrix_memory_against_unstabilised_sums():
    """With S~ = S exp(m) the running maximum drops out but for the constant under the quotient: o = S~' q / (max(|n~ . q|, 1) +
    1e-6 exp(m))."""
    rng = np.random.default_rng(2)
    T, H, D, V = 9, 2, 3, 4
    q, k, v = rng.normal(size=(T, H, D)), rng.normal(size=(T, H, D)), rng.normal(size=(T, H, V))
    li, lk = rng.normal(size=(T, H)) * 2.0, Z.log_sigmoid(rng.normal(size=(T, H)))
    o = Z.stabilised_matrix_scan(q, k, v, li, lk)
    for h in range(H):
        m = 0.0
        for t in range(T):
            m = max(lk[t, h] + m, li[t, h])
            w = [np.exp(li[s, h] + lk[s + 1:t + 1, h].sum()) * (k[s, h] @ q[t, h]) for s in range(t + 1)]
            den = max(abs(sum(w)), 1.0) + 1e-6 * np.exp(m)
            assert np.allclose(o[t, h], sum(x * v[s, h] for s, x in enumerate(w)) / den)


def test_gates_and_activations():
    z = np.array([-800.0, -2.0, 0.0, 3.0, 800.0])
    assert np.allclose(Z.log_sigmoid(z), [-800.0, np.log(Z.sigmoid(-2.0)), np.log(0.5), np.log(Z.sigmoid(3.0)), 0.0])
    assert np.allclose(Z.gelu_tanh(np.array([0.0, 10.0, -10.0])), [0.0, 10.0, 0.0])
    w = {"m.up": np.array([[1.0], [-1.0]]), "m.down": np.array([[2.0, 5.0]])}
    assert np.allclose(Z.squared_relu_ff(np.array([[3.0], [-2.0]]), w, "m."), [[18.0], [20.0]])
    assert np.allclose(Z.norm_around_one(np.array([[3.0, 4.0]]), np.array([0.0, -1.0]), 0.0), [[3.0 / np.sqrt(12.5), 0.0]])


def test_router_weights_sum_to_the_scale():
    h = np.abs(np.random.default_rng(3).normal(size=(4, 5)))
    router = np.random.default_rng(4).normal(size=(6, 5))
    chosen, weights = Z.route(h, router, 3, 2.5)
    assert np.allclose(weights.sum(-1), 2.5) and (np.diff(weights, axis=-1) <= 0).all()
    s = Z.softmax_rows(h @ router.T)
    assert np.allclose(weights[0, 0] / weights[0, 2], s[0, chosen[0, 0]] / s[0, chosen[0, 2]])
    assert Z.route(np.zeros((1, 5)), router, 2, 1.0)[0].tolist() == [[0, 1]]                   # equal scores: the lower index


def test_plain_forward_runs_every_configuration(tmp_path):
    for name, cfg in LH.MODELS.items():
        d = LH.make_model_dir(str(tmp_path), cfg, name, seed=3, rank=LH.RANKS[name])
        ids = LH.tokens(1, 30, cfg["vocab"])
        logits = LH.plain_logits(d, ids)
        assert logits.shape == (30, cfg["vocab"]) and np.isfinite(logits).all()
        # what a position's logits are does not depend on what follows it
        assert np.allclose(LH.plain_logits(d, ids[:17]), logits[:17], atol=1e-9)
        settled = LH.settle_choices(d, str(tmp_path))
        assert LH.plain_margins(settled, ids).min() > 0.05
