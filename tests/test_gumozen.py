"""Gumozen without a GPU: the configuration reader, the model it describes, the tensors it declares, and the plain
implementation's mechanisms against hand-made cases."""
import copy

import numpy as np
import pytest

from tests import gumozen_helpers as GH
from tests.plain import gumozen_plain as Z


def test_registry_and_layers():
    from gibbs_amd.config import GumozenConfig, config_from_dict
    cfg = config_from_dict(GH.GUMOZEN_A)
    assert isinstance(cfg, GumozenConfig) and cfg.to_dict() == GH.GUMOZEN_A
    spec = cfg.model_spec()
    assert spec.order == (0, 1, 2, 3, 4, 5) and spec.head == "head" and spec.embedding == "embed" and spec.streams == 1
    assert spec.embedding_norm.weight == "embed.norm" and spec.embedding_norm.eps == 1e-5 and spec.final_norm.scale is None
    assert [ls.arrangement for ls in spec.layers] == ["post_norm"] * 6
    assert [r for r, _ in spec.layers[0].parts] == ["mixer_input", "mixer", "norm1", "ffn", "norm2"]
    assert [r for r, _ in spec.layers[2].parts] == ["mixer_input", "mixer", "norm1"]
    assert [ls.part("mixer").kind for ls in spec.layers] == ["latent_attention", "differential_attention", "gated_outer", "latent_attention",
                                                             "differential_attention", "latent_attention"]
    assert spec.layers[1].part("norm1").scale == "l1.ls1" and spec.layers[1].part("norm2").scale == "l1.ls2"
    assert cfg.derived()["layers_by_type"] == {"attention": 2, "hgrn2": 1, "latent_attention": 3} and cfg.derived()["reads_latent_of"] == {"3": 0, "5": 0}


def test_constants_come_from_the_configuration():
    from gibbs_amd.config import config_from_dict
    spec = config_from_dict(GH.GUMOZEN_A).model_spec()
    a = spec.layers[1].part("mixer")
    assert a.params == {"heads": 6, "kv_heads": 3, "head_dim": 10, "v_head_dim": 14, "scale": 0.9, "chunk": 13, "diff": 0.35, "norm_eps": 1e-5}
    assert a.position.params == {"theta": 1000.0, "rotary_dim": 6, "variant": "half_split", "precision": "f64",
                                 "bands": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64.0}}
    b = spec.layers[4].part("mixer")
    assert b.position is None and b.params["chunk"] == 0
    own, reads = spec.layers[0].part("mixer"), spec.layers[3].part("mixer")
    assert own.params["kv_rank"] == 11 and own.params["q_rank"] == 13 and own.params["rot_dim"] == 0 and "kv_source" not in own.params
    assert reads.params["kv_source"] == 0 and reads.params["scale"] == 0.8 and "dkv" not in reads.tensors
    assert spec.layers[2].part("mixer").params == {"heads": 3, "dim": 7, "vdim": 10, "norm_eps": 1e-5}
    ff = spec.layers[0].part("ffn")
    assert ff.kind == "moe" and ff.params["experts"] == 7 and ff.params["top"] == 3 and ff.params["inter"] == 30
    assert ff.params["scores"] == "sigmoid" and ff.params["weigh"] == "input"
    assert config_from_dict(GH.GUMOZEN_B).model_spec().final_norm.eps == 1e-6


def test_declared_tensors_cache_and_state():
    from gibbs_amd.config import config_from_dict
    from gibbs_amd.parts import DecoderModel
    model = DecoderModel(config_from_dict(GH.GUMOZEN_A).model_spec())
    shapes = {d.name: d.shape for d in model.tensor_decls()}
    assert shapes["embed"] == (211, 100) and shapes["embed.norm"] == (100,) and shapes["head"] == (211, 100) and shapes["final.norm"] == (100,)
    assert shapes["l0.shift"] == (100,) and shapes["l2.ls1"] == (100,) and "l2.ls2" not in shapes and "l2.norm2" not in shapes
    assert shapes["l1.mix.q"] == (120, 100) and shapes["l1.mix.k"] == (60, 100) and shapes["l1.mix.v"] == (42, 100) and shapes["l1.mix.o"] == (100, 84)
    assert shapes["l1.mix.q.norm"] == (10,) and shapes["l1.mix.g"] == (6, 100)
    assert all(shapes[f"l1.mix.{n}"] == (10,) for n in ("lq1", "lk1", "lq2", "lk2"))
    assert shapes["l2.mix.f"] == (21, 100) and shapes["l2.mix.f.b"] == (21,) and shapes["l2.mix.lower"] == (21,) and shapes["l2.mix.norm"] == (10,)
    assert shapes["l0.mix.dkv"] == (11, 100) and shapes["l0.mix.dkv.norm"] == (11,) and shapes["l0.mix.uk"] == (30, 11) and shapes["l0.mix.uv"] == (45, 11)
    assert "l3.mix.dkv" not in shapes and shapes["l3.mix.dq"] == (17, 100) and shapes["l3.mix.uq"] == (30, 17) and shapes["l3.mix.uv"] == (21, 11)
    assert shapes["l0.mlp.router"] == (7, 100) and shapes["l0.mlp.e6.down"] == (100, 30) and "l0.mlp.e7.up" not in shapes
    owners = model.cache_owners()
    need = dict(zip(owners, model.cache_needs()))
    assert (need[(1, "mixer")].kv_heads, need[(1, "mixer")].head_dim, need[(1, "mixer")].value_dim, need[(1, "mixer")].window) == (3, 20, 14, None)
    assert (need[(0, "mixer")].kv_heads, need[(0, "mixer")].head_dim, need[(0, "mixer")].value_dim) == (1, 11, 0)
    assert need[(3, "mixer")] is None and need[(5, "mixer")] is None and need[(2, "mixer")] is None
    sources = dict(zip(owners, model.kv_sources()))
    assert owners[sources[(3, "mixer")]] == (0, "mixer") and owners[sources[(5, "mixer")]] == (0, "mixer") and sources[(0, "mixer")] is None
    states = dict(zip(owners, model.state_needs()))
    assert [(s.name, s.shape) for s in states[(4, "mixer_input")]] == [("token_shift", (100,))]
    assert [(s.name, s.shape) for s in states[(2, "mixer")]] == [("gated_outer_rule", (3, 7, 10))]


def test_tensors_of_a_missing_feed_forward_are_declared_and_read_by_nobody():
    from gibbs_amd.config import config_from_dict
    from gibbs_amd.parts import DecoderModel
    full = {d.name: d.shape for d in DecoderModel(config_from_dict(GH.GUMOZEN_A).model_spec()).tensor_decls()}
    more = dict(full, **{"l2.norm2": (100,), "l2.ls2": (100,)})
    spec = config_from_dict(GH.GUMOZEN_A, tensors=more).model_spec()
    assert {d.name for d in DecoderModel(spec).tensor_decls()} == set(more) and [r for r, _ in spec.layers[2].parts][-1] == "norm1"


@pytest.mark.parametrize("change, words", [
    (lambda c: c["layers"][0].__setitem__("type", "mamba2"), "mixer type"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 4), "multiple"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 12), "rotated"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].__setitem__("high", 0.5), "scaling"),
    (lambda c: c["layers"][1]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][1]["mixer"]["mask"].__setitem__("size", 0), "mask.size"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_from", 1), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_from", 5), "kv_from"),
    (lambda c: c["layers"][5]["mixer"].__setitem__("kv_from", 3), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].__setitem__("kv_rank", 12), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("heads", 0), "heads"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 8), "experts a token"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"), "feed-forward kind"),
    (lambda c: c.pop("width"), "width"),
])
def test_refused_configurations(change, words):
    from gibbs_amd.config import ConfigError, config_from_dict
    cfg = copy.deepcopy(GH.GUMOZEN_A)
    change(cfg)
    with pytest.raises(ConfigError, match=words):
        config_from_dict(cfg)


# ----------------------------------------------------------------------------------------------- the plain mechanisms
def test_shift_mixes_in_the_row_before_and_starts_from_zeros():
    h = np.array([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]])
    out = Z.token_shift(h, np.array([0.5, 1.0]))
    assert np.allclose(out, [[0.5, 0.0], [1.5, 10.0], [3.0, 20.0]])


def test_frequencies_by_band():
    from gibbs_amd.parts.rope import rope_inv_freq
    scaling = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 100.0}
    base, dims = 10000.0, 32
    plain, got = Z.frequencies(base, dims), Z.frequencies(base, dims, scaling)
    wave = 2 * np.pi / plain.astype(np.float64)
    kept, low = wave < 25.0, wave > 100.0
    assert kept.any() and low.any() and (~kept & ~low).any()
    assert np.array_equal(got[kept], plain[kept]) and np.allclose(got[low], plain[low] / 8.0)
    for f, g, l in zip(plain[~kept & ~low], got[~kept & ~low], wave[~kept & ~low]):
        s = (100.0 / l - 1.0) / 3.0
        assert np.isclose(g, (1 - s) * f / 8.0 + s * f, rtol=1e-6) and f / 8.0 <= g <= f
    assert np.array_equal(rope_inv_freq(dims, base, bands=scaling), got)
    assert np.array_equal(rope_inv_freq(dims, base), plain)


def test_chunks_at_their_edges():
    c = Z.visible_chunk(10, 4)
    assert c[5].nonzero()[0].tolist() == [4, 5] and c[7].nonzero()[0].tolist() == [4, 5, 6, 7] and c[8].nonzero()[0].tolist() == [8]
    assert Z.visible_chunk(5, 1).sum() == 5 and Z.visible_chunk(4, None).sum() == 10


def test_equal_maps_cancel_by_one_minus_lambda():
    """With both maps alike, a_1 - lambda a_2 = (1 - lambda) a, and the division by the root mean square leaves a's direction."""
    rng = np.random.default_rng(0)
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "scale": 0.5, "diff": 0.25}
    W, T = 5, 6
    one_q, one_k = rng.normal(size=(2, 1, 4, W)), rng.normal(size=(1, 1, 4, W))
    w = {"q": np.repeat(one_q, 2, 1).reshape(16, W), "k": np.repeat(one_k, 2, 1).reshape(8, W), "v": rng.normal(size=(3, W)), "o": np.eye(6),
         "q.norm": np.ones(4), "k.norm": np.ones(4), "g": np.zeros((2, W)), "lq1": np.zeros(4), "lk1": np.ones(4), "lq2": np.zeros(4), "lk2": np.ones(4)}
    h = rng.normal(size=(T, W))
    assert Z.combination_weight(w["lq1"], w["lk1"], w["lq2"], w["lk2"], 0.25) == 0.25
    out = Z.differential_attention_mixer(h, w, "", m, np.arange(T), 1e-12).reshape(T, 2, 3)
    first = out[0] / (0.5 * 0.75)                                     # one visible key: a = v_0, gate one half, times 1 - diff
    v0 = h[0] @ w["v"].T
    assert np.allclose(first, v0 / np.sqrt((v0 ** 2).mean()))
    assert np.allclose((out ** 2).mean(-1), (0.5 * 0.75) ** 2)


def test_the_recurrence_against_its_closed_form():
    """With a constant gate f per channel, y_t = sum_s sum_i q_i f_i^(t - s) (1 - f_i) v_s."""
    rng = np.random.default_rng(1)
    T, H, D, V = 6, 2, 3, 4
    q, v = rng.normal(size=(T, H, D)), rng.normal(size=(T, H, V))
    f = np.broadcast_to(rng.uniform(0.1, 0.95, size=(H, D)), (T, H, D))
    y = Z.gated_outer_scan(q, f, v)
    for h in range(H):
        for t in range(T):
            want = sum((q[t, h] * f[0, h] ** (t - s) * (1 - f[0, h])).sum() * v[s, h] for s in range(t + 1))
            assert np.allclose(y[t, h], want)


def test_the_gate_never_falls_below_its_bound():
    z = np.array([-80.0, 0.0, 80.0])
    assert np.allclose(Z.forget_gate(z, 0.0, 0.3), [0.3, 0.65, 1.0])


def test_scores_by_the_sigmoid_weigh_the_input():
    rng = np.random.default_rng(2)
    W, F = 6, 4
    router = np.zeros((3, W))
    router[0, 0], router[1, 0], router[2, 0] = 1.0, 3.0, -1.0
    h = np.abs(rng.normal(size=(2, W))) + 0.5
    chosen, weights = Z.route(h, router, 2)
    assert chosen.tolist() == [[1, 0], [1, 0]] and np.allclose(weights[:, 0], Z.sigmoid(3 * h[:, 0])) and np.allclose(weights[:, 1], Z.sigmoid(h[:, 0]))
    assert Z.route(np.zeros((1, W)), router, 2)[0].tolist() == [[0, 1]]                   # equal scores: the lower index
    w = {"m.router": router}
    for e in range(3):
        w[f"m.e{e}.gate"], w[f"m.e{e}.up"], w[f"m.e{e}.down"] = rng.normal(size=(F, W)), rng.normal(size=(F, W)), rng.normal(size=(W, F))
    out = Z.moe_ff(h, w, "m.", GH.moe(3, 2, F))
    want = sum(Z.expert(weights[:, c:c + 1] * h, w[f"m.e{e}.gate"], w[f"m.e{e}.up"], w[f"m.e{e}.down"]) for c, e in enumerate((1, 0)))
    assert np.allclose(out, want)
    outside = sum(weights[:, c:c + 1] * Z.expert(h, w[f"m.e{e}.gate"], w[f"m.e{e}.up"], w[f"m.e{e}.down"]) for c, e in enumerate((1, 0)))
    assert not np.allclose(out, outside)
    assert np.isinf(Z.route_margin(h, router, 3)).all()


def test_plain_forward_runs_every_configuration(tmp_path):
    for name, cfg in GH.MODELS.items():
        d = GH.make_model_dir(str(tmp_path), cfg, name, seed=3)
        ids = GH.tokens(1, 30, cfg["vocab"])
        logits = GH.plain_logits(d, ids)
        assert logits.shape == (30, cfg["vocab"]) and np.isfinite(logits).all()
        # what a position's logits are does not depend on what follows it
        assert np.allclose(GH.plain_logits(d, ids[:17]), logits[:17], atol=1e-9)
        settled = GH.settle_choices(d, str(tmp_path))
        assert GH.plain_margins(settled, ids).min() > 0.01
