"""Lubavik on the GPU against the plain implementation, in 32-bit and in bfloat16: each mechanism alone; whole prompts;
most of a prompt in one step and its last tokens one by one; portions of changing size down to two tokens; mixed
batches in a pool so small that pages and slots are used again; long decoding; the first tokens; kernels with inputs
made so that one key at a page's or chunk's edge, a state written long ago, a strong decay, a gate at its cap or a router's choice
stands out; generation through the scheduler, the replay program and the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import lubavik_helpers as LH
from tests.plain import lubavik_plain as Z
from tests.test_engine_gpu import mixed_schedule, portions, run_steps

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
NAMES = ["A", "B", "C", "D"]
LENGTHS = {"A": 150, "B": 230, "C": 120, "D": 140}
# bfloat16 against the plain implementation, per row: relative L2 error of the logits.  A router's choice between two
# experts whose logits differ by less than the rounding of its input may fall the other way than in float64, and with a
# norm behind the experts that changes the token's whole row, which every later token may read: a sequence is held to the
# bound up to its first token whose least clear choice (`route_margin`) is below CLEAR_CHOICE (sequences are picked so that
# this comes late, `clear_tokens`).  So that every row of every test is held to the bound in bfloat16 as well, each model
# also runs in a copy whose routers always choose clearly (`settle_choices`).  Rows that amplify rounding are held to a bound as
# much wider (`LH.amplification`); a row in a hundred may exceed it all the same, none by more than BF16_WORST.
BF16_REL_L2 = 0.06
BF16_ROWS_OVER = 0.02
BF16_WORST = 0.2
ORDINARY = 30.0
# Model A's small heads and sharp scores make bfloat16 operands cost about twice as much (the plain implementation with every operand
# of a product rounded to bfloat16 is as far off): twice the bounds.
SHARP = "lubavik_A"
CLEAR_CHOICE = 0.05


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("lubavik")
    out = {n: LH.make_model_dir(str(root), LH.MODELS[n], n, seed=61 + i, rank=LH.RANKS[n]) for i, n in enumerate(NAMES)}
    out.update({n + "_settled": LH.settle_choices(out[n], str(root)) for n in NAMES})
    one = LH.single_layer
    made = {"attention": one(LH.attention(6, 2, 10, 18, 0.9, rot=(1000.0, 8))), "attention_aligned": one(LH.attention(8, 4, 32, 48, 0.4, rot=(1e4, 32)), width=64, side=8),
            "shared_cache": LH.model(131, 60, [LH.with_mlp(LH.attention(4, 2, 10, 12, 0.6, rot=(100.0, 10)), None), LH.with_mlp(LH.attention(2, 2, 10, 12, 0.8, rot=(100.0, 10), kv_from=0), None)], 4),
            "pair": one(LH.parallel(LH.chunked(4, 2, 12, 18, 0.5, size=11, rot=(500.0, 6)), LH.linear(3, 9, 14, 5.0), 0.6, 1.5)),
            "pair_aligned": one(LH.parallel(LH.chunked(4, 2, 32, 64, 0.25, size=40, rot=(1e4, 16)), LH.linear(2, 64, 32, 16.0), 1.3, 0.4), width=64, side=16),
            "memory": one(LH.mlstm(5, 12, 9, 4.0)), "memory_aligned": one(LH.mlstm(2, 32, 64, 12.0), width=128, side=8),
            "squared_relu": one(LH.mlstm(2, 8, 10, 2.0), LH.dense(70)), "experts": one(LH.mlstm(2, 8, 10, 6.0), LH.moe(7, 3, 36, shared=20, scale=1.8))}
    for i, (name, cfg) in enumerate(made.items()):
        out[name] = LH.make_model_dir(str(root), cfg, name, seed=5 + i)
    out["experts_settled"] = LH.settle_choices(out["experts"], str(root))
    return out


def make_engine(model_dir, dtype, **kw):
    from gibbs_amd import Engine
    kw.setdefault("max_tokens", 2048)
    kw.setdefault("max_requests", 4)
    return Engine(model_dir, dtype=dtype, **kw)


def close(got, want, dtype, what, amplified=None, slack=1.0):
    """`amplified` (per row, `LH.amplification`): a row that amplifies rounding by more than ORDINARY is held to a bound as much wider."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    assert got.shape == want.shape, (what, got.shape, want.shape)
    wider = np.maximum(1.0, (np.ones(len(want)) if amplified is None else amplified / ORDINARY))
    if dtype == "float32":
        err = np.abs(got - want).max(-1)
        bound = 3e-5 * np.abs(want).max() * wider
        worst = int((err / bound).argmax())
        assert (err <= bound).all(), f"{what}: error {err[worst]:.3e} at row {worst} above {bound[worst]:.3e}; first bad row {int((err > bound).argmax())}"
        return
    rel = np.sqrt(((got - want) ** 2).sum(-1) / (want ** 2).sum(-1))
    assert np.isfinite(rel).all(), what
    wider = wider * slack
    over = rel > BF16_REL_L2 * wider
    worst = int((rel / wider).argmax())
    assert over.sum() <= max(2, int(BF16_ROWS_OVER * rel.size)) and (rel <= BF16_WORST * wider).all(), \
        f"{what}: relative L2 error {rel[worst]:.3e} (bound {wider[worst]:.1f} times wider); {int(over.sum())} of {rel.size} rows over; first bad row {int(over.argmax())}"


def check(model_dir, seqs, got, dtype, what):
    compared = total = 0
    for rid, ids in seqs.items():
        want = LH.plain_logits(model_dir, ids)
        places = sorted(p for r, p in got if r == rid)
        assert places, f"{what}: no logits for {rid}"
        total += len(places)
        if dtype != "float32":
            unclear = np.nonzero(LH.plain_margins(model_dir, ids) < CLEAR_CHOICE)[0]
            places = [p for p in places if not unclear.size or p < unclear[0]]
            if not places:
                continue
        compared += len(places)
        close(np.stack([got[(rid, p)] for p in places]), want[places], dtype, f"{what} request {rid}", LH.amplification(model_dir, ids)[places],
              slack=2.0 if SHARP in os.path.basename(model_dir) else 1.0)
    assert compared == total or not model_dir.endswith("_settled"), f"{what}: {total - compared} rows of a model with settled choices were not compared"


def variants(dirs, name, dtype):
    """The model's folder, and for bfloat16 also its copy with settled choices of experts."""
    return [dirs[name]] + ([dirs[name + "_settled"]] if dtype == "bfloat16" and name + "_settled" in dirs else [])


def pick(model_dir, seed, n):
    return LH.clear_tokens(model_dir, seed, n, vocab_of(model_dir), CLEAR_CHOICE)


def vocab_of(model_dir):
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)["vocab"]


# ----------------------------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "attention_aligned", "shared_cache", "pair", "pair_aligned", "memory", "memory_aligned", "squared_relu", "experts"])
def test_each_mechanism_alone(dirs, kind, dtype):
    for d in variants(dirs, kind, dtype):
        ids = pick(d, 1, 90)
        eng = make_engine(d, dtype)
        got = run_steps(eng, [([("r", ids[:61], list(range(61)))], []), ([("r", ids[61:], list(range(29)))], ["r"])])
        check(d, {"r": ids}, got, dtype, f"{kind} alone {dtype}")
        assert eng.cache.free_slots() == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole(dirs, name, dtype):
    for d in variants(dirs, name, dtype):
        ids = pick(d, 2, LENGTHS[name])
        eng = make_engine(d, dtype)
        got = run_steps(eng, [([("r", ids, list(range(len(ids))))], ["r"])])
        check(d, {"r": ids}, got, dtype, f"whole {name} {dtype}")
        eng.cache.check()
        assert all(eng.cache.free_pages(g) == eng.cache.pools[g].num_pages for g in range(eng.cache.n_groups))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_bulk_then_last_tokens_one_by_one(dirs, name, dtype):
    """The decoded tokens pass several chunks' and pages' edges."""
    for d in variants(dirs, name, dtype):
        ids = pick(d, 3, LENGTHS[name])
        cut = len(ids) - 70
        steps = [([("r", ids[:cut], list(range(cut)))], [])] + [([("r", [t], [0])], []) for t in ids[cut:]]
        got = run_steps(make_engine(d, dtype), steps)
        check(d, {"r": ids}, got, dtype, f"bulk+tail {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_changing_portions_down_to_two_tokens(dirs, name, dtype):
    """Cuts in the middle of pages and chunks; portions on both sides of what the recurrences take in chunks."""
    for d in variants(dirs, name, dtype):
        ids = pick(d, 4, LENGTHS[name])
        cuts = portions(len(ids) - 9, [7, 2, 13, 3, 2, 97, 5, 2, 17, 1, 2]) + [(len(ids) - 9 + i, len(ids) - 8 + i) for i in range(9)]
        steps = [([("r", ids[a:b], list(range(b - a)))], []) for a, b in cuts]
        got = run_steps(make_engine(d, dtype), steps)
        check(d, {"r": ids}, got, dtype, f"portions {name} {dtype}")


@pytest.mark.parametrize("name", NAMES)
def test_cutting_and_batching_change_nothing_in_32_bit(dirs, name):
    """Products add in ascending k, the attention takes keys in blocks aligned to absolute positions, the recurrences keep a
    request's tokens in order, and an expert's result for a row does not depend on which other rows the expert serves: 32-bit
    logits do not depend on how the prompt was cut or on what else was in the batch, beyond rounding."""
    d = dirs[name]
    ids = LH.tokens(5, 77, vocab_of(d))
    other = LH.tokens(6, 41, vocab_of(d))
    whole = run_steps(make_engine(d, "float32"), [([("r", ids, list(range(77)))], [])])
    eng = make_engine(d, "float32")
    steps = [([("o", other[:20], []), ("r", ids[:2], [0, 1])], []), ([("r", ids[2:50], list(range(48))), ("o", other[20:21], [])], []),
             ([("o", other[21:], []), ("r", ids[50:51], [0])], ["o"]), ([("r", ids[51:], list(range(26)))], [])]
    cut = run_steps(eng, steps)
    for p in range(77):
        assert np.abs(cut[("r", p)] - whole[("r", p)]).max() <= 6e-6 * np.abs(whole[("r", p)]).max(), p


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_with_pages_and_slots_used_again(dirs, name, dtype):
    for d in variants(dirs, name, dtype):
        rng = np.random.default_rng(7)
        seqs = {f"q{i}": pick(d, 100 + i, int(n)) for i, n in enumerate([70, 45, 90, 33, 64, 81, 50, 3, 2])}
        steps = mixed_schedule(seqs, rng)
        assert max(len(e) for e, _ in steps) >= 3
        assert any(len(t) > 1 for e, _ in steps for _, t, _ in e) and any(len(t) == 1 for e, _ in steps for _, t, _ in e)
        eng = make_engine(d, dtype, max_tokens=384, max_requests=4, page_size=16)
        assert sum(-(-len(s) // 16) for s in seqs.values()) > eng.cache.pools[0].num_pages, "the pool must be too small to avoid reuse"
        got = run_steps(eng, steps)
        check(d, seqs, got, dtype, f"mixed {name} {dtype}")
        eng.cache.check()
        assert eng.cache.free_slots() == 4 and all(eng.cache.free_pages(g) == eng.cache.pools[g].num_pages for g in range(eng.cache.n_groups))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B"])
def test_long_portions_beside_decoded_tokens(dirs, name, dtype):
    """Decoded tokens at the head of a batch beside a portion that the recurrences take in chunks and one that is shorter than a
    chunk: every request's state is its own."""
    for d in variants(dirs, name, dtype):
        a, b, c = pick(d, 61, 40), pick(d, 62, 250), pick(d, 63, 60)
        steps = [([("a", a[:30], [29]), ("c", c[:20], [])], [])]
        steps += [([("a", [a[30]], [0]), ("b", b[:130], [0, 63, 64, 129]), ("c", c[20:27], [6])], []),
                  ([("a", [a[31]], [0]), ("c", [c[27]], [0]), ("b", b[130:245], [0, 114])], []),
                  ([("a", [a[32]], [0]), ("b", [b[245]], [0]), ("c", c[28:59], [0, 30])], []),
                  ([("a", [a[33]], [0]), ("b", b[246:250], [3]), ("c", [c[59]], [0])], ["a", "b", "c"])]
        got = run_steps(make_engine(d, dtype), steps)
        check(d, {"a": a, "b": b, "c": c}, got, dtype, f"portions beside decoded tokens {name} {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dirs, dtype):
    for d in variants(dirs, "A", dtype):
        ids = pick(d, 9, 300)
        steps = [([("r", ids[:5], list(range(5)))], [])] + [([("r", [t], [0])], []) for t in ids[5:]]
        got = run_steps(make_engine(d, dtype), steps)
        check(d, {"r": ids}, got, dtype, f"long decoding {dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B"])
def test_first_tokens(dirs, name, dtype):
    """Sequences of one, two, three and five tokens, side by side and one token at a time: a single visible key beside the sink, an
    empty state, the running maximum at zero."""
    d = variants(dirs, name, dtype)[-1]
    seqs = {f"s{n}": pick(d, 20 + n, n) for n in (1, 2, 3, 5)}
    got = run_steps(make_engine(d, dtype), [([(r, ids, list(range(len(ids)))) for r, ids in seqs.items()], list(seqs))])
    check(d, seqs, got, dtype, f"first tokens together {dtype}")
    eng = make_engine(d, dtype)
    for r, ids in seqs.items():
        got = run_steps(eng, [([(r, ids[:1], [0])], [])] + [([(r, [t], [0])], []) for t in ids[1:]])
        check(d, {r: ids}, got, dtype, f"first tokens one by one {dtype}")
        eng.release(r)


# ----------------------------------------------------------------------------------------------- kernels with made-up inputs
_alive = []


def _dev(a, dtype=torch.float32):
    """A device tensor of `a` that lives until the module is done: kernels are handed raw addresses, and a tensor that is
    made inside a call's argument list would be given back before the kernel has run."""
    t = torch.tensor(np.asarray(a), dtype=dtype, device="cuda")
    _alive.append(t)
    if len(_alive) > 4000:
        torch.cuda.synchronize()
        del _alive[:2000]
    return t


def _f64(t):
    return t.float().cpu().numpy().astype(np.float64)


def _pad8(n):
    return -(-n // 8) * 8


def _cos_sin(freq, length):
    """The table of cosines and sines of the first `length` positions; positions behind it have theirs computed."""
    angle = (np.arange(length, dtype=np.float32)[:, None] * freq[None, :]).astype(np.float32).astype(np.float64)
    return np.stack([np.cos(angle), np.sin(angle)], axis=-1).astype(np.float32)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("variant", [0, 1])
@pytest.mark.parametrize("sizes", [(6, 3, 10, 14, 6, 10, 14), (4, 2, 24, 40, 16, 48, 48), (5, 1, 40, 128, 32, 128, 128), (8, 2, 64, 64, 64, 64, 64), (7, 7, 20, 12, 8, 32, 32)])
def test_rows_with_biases_and_normed_heads(sizes, variant, dtype):
    """Biases, q and k heads divided by their own root mean square, a gain that the heads share, the rotation of part of a head in both
    layouts, keys and values in their pages; heads stored wider than they are."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(5)
    H, G, D, V, rot, ks, vs = sizes
    ps, places = 16, [0, 15, 16, 250, 3000]
    n = len(places)
    ld = (H + G) * ks + G * vs + 8
    spans = [(0, H, ks, D), (H * ks, G, ks, D), ((H + G) * ks, G, vs, V)]
    r, bias = np.zeros((n, ld)), np.zeros((H + G) * ks + G * vs)
    for at, heads, stored, true in spans:
        for h in range(heads):
            r[:, at + h * stored:at + h * stored + true] = rng.normal(size=(n, true)) * (0.3 + h)
            bias[at + h * stored:at + h * stored + true] = rng.normal(size=true)
    rows = _dev(r, dtype)
    r64, b64 = _f64(rows), bias.astype(np.float32).astype(np.float64)
    gains = [(rng.normal(size=D) + 1.0).astype(np.float32) for _ in range(2)]
    base = 500.0
    freq = np.array([base ** (-2.0 * i / rot) for i in range(rot // 2)]).astype(np.float32)
    n_pages = 3000 // ps + 1
    kpages = torch.full((n_pages, G, ps, ks), 7.0, dtype=dtype, device="cuda")
    vpages = torch.full((n_pages, G, ps, vs), 7.0, dtype=dtype, device="cuda")
    table = torch.arange(n_pages - 1, -1, -1, dtype=torch.int32, device="cuda").view(1, n_pages).contiguous()
    turns, dev_gains = _dev(_cos_sin(freq, 100)), [_dev(np.pad(g, (0, ks - D))) for g in gains]
    call("gibbs_qkv_prepare_full", ptr(rows), ld, ptr(kpages), ptr(vpages), dtype_code(dtype), ptr(_dev(bias)), ptr(_dev(freq)), rot, variant, ptr(turns), 100,
         None, 0, V, None, ptr(_dev(places, torch.int32)), ptr(_dev([0] * n, torch.int32)), ptr(table), n_pages, ps, n_pages, n, H, G, ks, vs,
         ptr(dev_gains[0]), ptr(dev_gains[1]), 1e-5, D, 0, None, 0, stream())
    got = _f64(rows)
    tol = 1e-4 if dtype == torch.float32 else 0.1
    want = []
    for which, (at, heads, stored, true) in enumerate(spans):
        x = (r64[:, at:at + heads * stored] + b64[at:at + heads * stored]).reshape(n, heads, stored)[:, :, :true]
        if which < 2:
            x = Z.rotate(Z.rms_unit(x, 1e-5) * gains[which].astype(np.float64), places, base, rot, neighbours=variant == 1)
        want.append(x)
        have = got[:, at:at + heads * stored].reshape(n, heads, stored)
        assert (np.abs(have[:, :, :true] - x) <= tol * np.maximum(1.0, np.abs(x) / 4)).all()
        assert not have[:, :, true:].any()
    assert np.array_equal(got[:, (H + G) * ks + G * vs:], r64[:, (H + G) * ks + G * vs:])
    for pages, x, true in ((kpages, want[1], D), (vpages, want[2], V)):
        for row, p in enumerate(places):
            have = _f64(pages[n_pages - 1 - p // ps, :, p % ps])
            assert (np.abs(have[:, :true] - x[row]) <= tol * np.maximum(1.0, np.abs(x[row]) / 4)).all() and not have[:, true:].any()
        assert int((pages == 7.0).all(-1).sum()) == (n_pages * ps - n) * G


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("variant", [0, 1])
@pytest.mark.parametrize("sizes", [(6, 3, 10, 14, 6, 10, 14), (4, 2, 24, 40, 24, 48, 48), (8, 2, 64, 128, 32, 128, 128), (3, 0, 16, 16, 16, 16, 16), (2, 1, 5, 3, 0, 5, 3),
                                   (40, 8, 64, 64, 64, 64, 64), (72, 16, 64, 32, 48, 64, 64), (160, 8, 64, 64, 64, 64, 64)])
def test_rows_normed_over_the_whole_projection(sizes, variant, dtype):
    """q and k divided by the root mean square of all their heads at once, a gain per channel, the rotation of both layouts, keys and
    values in their pages on both sides of page borders and far out; heads stored wider than they are; queries alone (no kv heads)."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(2)
    H, G, D, V, rot, ks, vs = sizes
    ps, places = 16, [0, 15, 16, 17, 31, 250, 70000]
    n = len(places)
    ld = (H + G) * ks + G * vs + 3 * (ks % 8 == 0) * 8
    r = np.zeros((n, ld))
    q, k, v = rng.normal(size=(n, H, D)) * np.linspace(0.2, 3.0, H)[None, :, None], rng.normal(size=(n, G, D)), rng.normal(size=(n, G, V))
    for x, heads, stored, true, at in ((q, H, ks, D, 0), (k, G, ks, D, H * ks), (v, G, vs, V, (H + G) * ks)):
        block = np.zeros((n, heads, stored))
        block[:, :, :true] = x
        r[:, at:at + heads * stored] = block.reshape(n, -1)
    rows = _dev(r, dtype)
    r64 = _f64(rows)
    gains = []
    for heads in (H, G):
        g = np.zeros((heads, ks), dtype=np.float32)
        g[:, :D] = rng.normal(size=(heads, D)) + 1.0
        gains.append(g)
    base = 1000.0
    freq = np.array([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=np.float64).astype(np.float32)
    n_pages = 70000 // ps + 1
    kpages = torch.full((n_pages, max(G, 1), ps, ks), 7.0, dtype=dtype, device="cuda")
    vpages = torch.full((n_pages, max(G, 1), ps, vs), 7.0, dtype=dtype, device="cuda")
    table = torch.arange(n_pages - 1, -1, -1, dtype=torch.int32, device="cuda").view(1, n_pages).contiguous()
    turns = _dev(_cos_sin(freq, 100)) if rot else None
    call("gibbs_qkv_prepare_whole", ptr(rows), ld, ptr(kpages) if G else None, ptr(vpages) if G else None, dtype_code(dtype), ptr(_dev(gains[0])), ptr(_dev(gains[1])) if G else None,
         1e-5, D, ptr(_dev(freq)) if rot else None, rot, variant, ptr(turns) if rot else None, 100,
         ptr(_dev(places, torch.int32)), ptr(_dev([0] * n, torch.int32)), ptr(table), n_pages, ps, n_pages, n, H, G, ks, vs, stream())

    def want_of(at, heads, g):
        x = r64[:, at:at + heads * ks].reshape(n, heads, ks)[:, :, :D]
        x = (Z.rms_unit(x.reshape(n, heads * D), 1e-5).reshape(n, heads, D)) * g[:, :D].astype(np.float64)
        return Z.rotate(x, places, base, rot, neighbours=variant == 1) if rot else x

    tol = 4e-5 if dtype == torch.float32 else 0.2
    got = _f64(rows)
    assert np.abs(got[:, :H * ks].reshape(n, H, ks)[:, :, :D] - want_of(0, H, gains[0])).max() <= tol
    assert not got[:, :H * ks].reshape(n, H, ks)[:, :, D:].any()
    assert np.array_equal(got[:, (H + G) * ks + G * vs:], r64[:, (H + G) * ks + G * vs:])
    if not G:
        assert (kpages == 7.0).all()
        return
    want_k = want_of(H * ks, G, gains[1])
    for i, p in enumerate(places):
        page = n_pages - 1 - p // ps
        assert np.abs(_f64(kpages[page, :, p % ps])[:, :D] - want_k[i]).max() <= tol, p
        assert np.array_equal(_f64(vpages[page, :, p % ps])[:, :V], r64[i, (H + G) * ks:(H + G) * ks + G * vs].reshape(G, vs)[:, :V]), p
    assert int((kpages != 7.0).any(-1).sum()) == n * G and int((vpages != 7.0).any(-1).sum()) == n * G      # nothing else was written


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [100, 2048, 5120])
def test_a_sum_of_two_results_with_a_bias_at_the_border(dtype, W):
    """x += norm(s1 (a + bias) + s2 b) in one pass, with and without the second term, the bias and the rows that the next sublayer
    reads; each term whole or as partial sums; and the same terms written out as partial sums."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(1)
    n = 5
    gain, bias = (rng.normal(size=W) + 1.0).astype(np.float32), rng.normal(size=W).astype(np.float32)
    for parts1, parts2, with_bias, two in ((1, 1, True, True), (3, 1, True, True), (1, 2, False, True), (2, 2, True, True), (1, 1, True, False), (4, 1, False, False)):
        a = _dev(rng.normal(size=(parts1, n, W)), torch.float32 if parts1 > 1 else dtype)
        b = _dev(rng.normal(size=(parts2, n, W)), torch.float32 if parts2 > 1 else dtype)
        s1, s2 = 1.7, -0.4
        first = s1 * (_f64(a).sum(0) + (bias.astype(np.float64) if with_bias else 0.0))
        second = s2 * _f64(b).sum(0) if two else np.zeros((n, W))
        x0 = rng.normal(size=(n, W)).astype(np.float32)
        want = x0 + Z.rms_unit(first + second, 1e-5) * gain
        for read in (0, 1):
            x, out = _dev(x0), torch.full((n, W), 9.0, dtype=dtype, device="cuda")
            call("gibbs_rmsnorm_rows_sum_add_read", ptr(x), ptr(a), parts1, n * W, ptr(_dev(bias)) if with_bias else None, s1, ptr(b) if two else None, parts2, s2,
                 ptr(_dev(gain)), 1e-5, read, ptr(out), dtype_code(dtype), n, W, stream())
            assert np.abs(_f64(x) - want).max() <= 2e-5 * np.abs(want).max()
            assert (out == 9.0).all() if read == 0 else np.abs(_f64(out) - want).max() <= (2e-5 if dtype == torch.float32 else 1e-2) * np.abs(want).max()
        terms = torch.empty((2, n, W), dtype=torch.float32, device="cuda")
        call("gibbs_rows_terms", ptr(a), parts1, ptr(_dev(bias)) if with_bias else None, s1, ptr(b) if two else None, parts2, s2, ptr(terms), dtype_code(dtype), n, W, stream())
        t = _f64(terms)
        assert np.abs(t[0] - first).max() <= 1e-5 * np.abs(first).max() and np.abs(t[1] - second).max() <= 1e-5 * (1.0 + np.abs(second).max())


@pytest.mark.parametrize("n", [1, 7, 16, 40, 64])
@pytest.mark.parametrize("case", [(64, 128, 5, False), (24, 256, 1, True), (200, 72, 1, True), (513, 96, 5, False), (1024, 1024, 3, True)])
def test_activations_and_a_tables_rows_behind_a_product(n, case):
    """act(W x), times the entries of the row's token from a column of a wider table on: in the few-row product's epilogue (row-major and
    in tile order) and as a pass of its own in both precisions, with padded rows."""
    from gibbs_amd import ops
    from gibbs_amd.ops.lib import call, ptr, stream
    F, W, act, with_table = case
    rng = np.random.default_rng(6)
    fn = {1: Z.gelu_tanh, 3: lambda z: np.maximum(z, 0.0), 5: lambda z: np.maximum(z, 0.0) ** 2}[act]
    x, w = _dev(rng.normal(size=(n, W)), torch.bfloat16), _dev(rng.normal(size=(F, W)) * W ** -0.5, torch.bfloat16)
    vocab, column, columns = 23, 8, F + 24
    table = _dev(rng.normal(size=(vocab, columns)), torch.bfloat16)
    ids = _dev(rng.integers(0, vocab, size=n), torch.int32)
    mult = table.data_ptr() + 2 * column if with_table else None
    entries = _f64(table)[ids.cpu().numpy().astype(np.int64), column:column + F] if with_table else 1.0
    z64 = _f64(x) @ _f64(w).T
    want = fn(z64) * entries
    scale = np.abs(want).max()
    for weight, ldw in ((w, W), (ops.PackedWeight(w), 0)):
        _alive.append(weight)
        out = torch.full((n, F), 9.0, dtype=torch.bfloat16, device="cuda")
        call("gibbs_skinny_act", ptr(x), weight.data_ptr(), ptr(out), n, F, W, W, ldw, F, act, mult, columns, ptr(ids), vocab, stream())
        assert np.abs(_f64(out) - want).max() <= 1e-2 * scale
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1.2e-2)):
        z, tab = _dev(z64, dtype), table.to(dtype)
        _alive.append(tab)
        wide = _pad8(F)
        out = torch.full((n, wide), 9.0, dtype=dtype, device="cuda")
        m = tab.data_ptr() + tab.element_size() * column if with_table else None
        call("gibbs_act_rows", ptr(z), ptr(out), wide, int(dtype == torch.bfloat16), act, m, columns, ptr(ids), vocab, n, F, stream())
        assert np.abs(_f64(out)[:, :F] - fn(_f64(z)) * entries).max() <= tol * scale and not out[:, F:].any()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", [(52, 5, 3, 100, 2.5), (600, 8, 4, 256, 0.7), (9, 16, 1, 64, 1.0), (3, 1, 1, 40, 3.0)])
def test_router_weights_over_their_sum_times_a_constant(case, dtype):
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    n, E, top, W, scale = case
    rng = np.random.default_rng(3)
    h, router = _dev(rng.normal(size=(n, W)), dtype), _dev(rng.normal(size=(E, W)) * 0.3)
    chosen, weight = torch.empty((n, top), dtype=torch.int32, device="cuda"), torch.empty((n, top), dtype=torch.float32, device="cuda")
    call("gibbs_moe_route_scaled", ptr(h), W, dtype_code(dtype), ptr(router), None, None, ptr(chosen), ptr(weight), None, n, W, E, top, 1, scale, stream())
    hh, r64 = _f64(h), _f64(router)
    want_c, want_w = Z.route(hh, r64, top, scale)
    order = np.sort(hh @ r64.T, -1)[:, ::-1]
    sure = (order[:, :-1] - order[:, 1:]).min(-1) > 1e-4 if E > 1 else np.ones(n, dtype=bool)
    assert sure.mean() > 0.5 and np.array_equal(chosen.cpu().numpy()[sure], want_c[sure])
    assert np.abs(weight.cpu().numpy() - want_w)[sure].max() <= 3e-5 * scale and np.abs(weight.cpu().numpy().sum(-1) - scale).max() <= 1e-5 * scale


# ---- gated linear attention
class LinearCase:
    def __init__(self, sizes, T, dtype, seed=5, tau=4.0, z_shift=1.0):
        self.H, self.D, self.V, self.rank = H, D, V, R = sizes
        self.dtype, self.tau, self.eps = dtype, tau, 1e-5
        rng = np.random.default_rng(seed)
        at, self.off = 0, []
        for size in (H * D, H * D, H * V, H * V, R):
            self.off.append(at)
            at = _pad8(at + size)
        self.ld = at
        r = np.zeros((T, self.ld))
        for o, size in zip(self.off, (H * D, H * D, H * V, H * V, R)):
            r[:, o:o + size] = rng.normal(size=(T, size))
        self.bias, self.gain = (rng.normal(size=H * D) + z_shift).astype(np.float32), (rng.normal(size=V) + 1.0).astype(np.float32)
        self.set(r, _dev(rng.normal(size=(H * D, R)) * R ** -0.5, dtype))

    def set(self, rows, w_z):
        self.raw, self.w_z = _dev(rows, self.dtype), w_z
        _alive.append(w_z)

    def columns(self, r, i, width):
        return r[:, self.off[i]:self.off[i] + width]

    def plain(self, rows):
        H, D, V = self.H, self.D, self.V
        r = _f64(self.raw)[rows]
        T = len(rows)
        z = self.columns(r, 4, self.rank) @ _f64(self.w_z).T + self.bias.astype(np.float64)
        alpha = np.exp(Z.log_sigmoid(z) / self.tau).reshape(T, H, D)
        q, k, v = self.columns(r, 0, H * D).reshape(T, H, D) * D ** -0.5, self.columns(r, 1, H * D).reshape(T, H, D), self.columns(r, 2, H * V).reshape(T, H, V)
        y = Z.rms_unit(Z.decayed_outer_scan(q, k, v, alpha), self.eps) * self.gain
        return y.reshape(T, H * V) * Z.silu(self.columns(r, 3, H * V))

    def takes_chunks(self):
        from gibbs_amd.ops.lib import library
        return library().gibbs_gated_linear_chunks_take(self.D, self.V)

    def run(self, steps, state, how):
        """The kernels of one kind over `steps`, lists of (slot, rows) -> one output row per row of raw."""
        from gibbs_amd.ops.lib import call, dtype_code, library, ptr, stream
        H, D, V = self.H, self.D, self.V
        out = torch.zeros((self.raw.shape[0], H * V), dtype=self.dtype, device="cuda")
        bias, gain, code = _dev(self.bias), _dev(self.gain), dtype_code(self.dtype)
        for step in steps:
            index = np.concatenate([np.asarray(rows) for _, rows in step])
            x = self.raw[_dev(index, torch.int64)].contiguous()
            _alive.append(x)
            n, R = x.shape[0], len(step)
            cu, slots = _dev(np.concatenate([[0], np.cumsum([len(rows) for _, rows in step])]), torch.int32), _dev([s for s, _ in step], torch.int32)
            y = torch.empty((n, H * V), dtype=self.dtype, device="cuda")
            o = self.off
            if how == "chunks":
                z = (x[:, o[4]:o[4] + self.rank].float() @ self.w_z.float().T).contiguous()
                work = torch.full((library().gibbs_gated_linear_chunks_workspace(n, R, H, D, V),), float("nan"), dtype=torch.float32, device="cuda")
                _alive.extend([z, work])
                call("gibbs_gated_linear_chunks", ptr(x), self.ld, o[0], o[1], o[2], o[3], ptr(z), ptr(bias), 1.0 / self.tau, D ** -0.5, ptr(gain), self.eps, ptr(state),
                     state.stride(0), ptr(cu), ptr(slots), ptr(y), ptr(work), code, n, R, H, D, V, stream())
            else:
                call("gibbs_gated_linear_rows", ptr(x), self.ld, o[0], o[1], o[2], o[3], o[4], ptr(self.w_z), self.rank, ptr(bias), 1.0 / self.tau, D ** -0.5, ptr(gain), self.eps,
                     ptr(state), state.stride(0), None if how == "single" else ptr(cu), ptr(slots), ptr(y), code, R, H, D, V, stream())
            out[_dev(index, torch.int64)] = y
        torch.cuda.synchronize()
        return _f64(out)


# ---- matrix memory
class MemoryCase:
    def __init__(self, sizes, T, dtype, seed=5, cap=6.0, W=40, gate_std=2.0):
        self.H, self.D, self.V = H, D, V = sizes
        self.dtype, self.cap, self.eps, self.W = dtype, cap, 1e-5, W
        rng = np.random.default_rng(seed)
        at, self.off = 0, []
        self.widths = (H * D, H * D, H * V, H * V)
        for size in self.widths:
            self.off.append(at)
            at = _pad8(at + size)
        self.ld = at
        r = np.zeros((T, self.ld))
        for o, size in zip(self.off, self.widths):
            r[:, o:o + size] = rng.normal(size=(T, size))
        self.b = np.concatenate([rng.normal(size=H), rng.normal(size=H) + 2.0]).astype(np.float32)
        self.gain = (rng.normal(size=H * V) + 1.0).astype(np.float32)
        self.set(r, rng.normal(size=(T, W)), rng.normal(size=(2 * H, W)) * gate_std * W ** -0.5)

    def set(self, rows, h, w_gates):
        self.raw, self.h, self.w_gates = _dev(rows, self.dtype), _dev(h, self.dtype), _dev(w_gates, self.dtype)

    def plain(self, rows):
        H, D, V = self.H, self.D, self.V
        r, T = _f64(self.raw)[rows], len(rows)
        q, k, v, g = (r[:, o:o + w] for o, w in zip(self.off, self.widths))
        pre = _f64(self.h)[rows] @ _f64(self.w_gates).T + self.b.astype(np.float64)
        log_in = self.cap * np.tanh(pre[:, :H] / self.cap)
        log_keep = Z.log_sigmoid(self.cap * np.tanh(pre[:, H:] / self.cap))
        o = Z.stabilised_matrix_scan(q.reshape(T, H, D) * D ** -0.5, k.reshape(T, H, D), v.reshape(T, H, V), log_in, log_keep)
        return Z.rms_unit(o, self.eps).reshape(T, H * V) * self.gain * Z.sigmoid(g)

    def takes_chunks(self):
        from gibbs_amd.ops.lib import library
        return library().gibbs_matrix_lstm_chunks_take(self.D, self.V)

    def run(self, steps, state, how):
        """state: [slots, stride]: S of every head, then n of every head, then m of every head, from the offsets `self.places(state)`."""
        from gibbs_amd.ops.lib import call, dtype_code, library, ptr, stream
        H, D, V = self.H, self.D, self.V
        out = torch.zeros((self.raw.shape[0], H * V), dtype=self.dtype, device="cuda")
        b, gain, code = _dev(self.b), _dev(self.gain), dtype_code(self.dtype)
        norm_state = state.data_ptr() + 4 * _pad8(H * D * V)
        for step in steps:
            index = np.concatenate([np.asarray(rows) for _, rows in step])
            at = _dev(index, torch.int64)
            x, h = self.raw[at].contiguous(), self.h[at].contiguous()
            _alive.extend([x, h])
            n, R = x.shape[0], len(step)
            cu, slots = _dev(np.concatenate([[0], np.cumsum([len(rows) for _, rows in step])]), torch.int32), _dev([s for s, _ in step], torch.int32)
            y = torch.empty((n, H * V), dtype=self.dtype, device="cuda")
            operands = (ptr(x), self.ld, *self.off, ptr(h), self.W, ptr(self.w_gates), ptr(b), ptr(gain), self.cap, self.eps, D ** -0.5, ptr(state), norm_state, state.stride(0),
                        None if how == "single" else ptr(cu), ptr(slots), ptr(y))
            if how == "chunks":
                gates = (self.w_gates.float() @ h.float().T).contiguous()
                work = torch.full((library().gibbs_matrix_lstm_chunks_workspace(n, R, H, D, V),), float("nan"), dtype=torch.float32, device="cuda")
                _alive.extend([gates, work])
                call("gibbs_matrix_lstm_chunks", *operands, ptr(gates), ptr(work), code, n, R, H, D, V, stream())
            else:
                call("gibbs_matrix_lstm_rows", *operands, code, R, H, D, V, stream())
            out[at] = y
        torch.cuda.synchronize()
        return _f64(out)

    def stride(self):
        return _pad8(self.H * self.D * self.V) + _pad8(self.H * (self.D + 1))


def _three_ways(case, stride, tol):
    """Two requests (300 and 131 rows) in scattered slots: token by token, in ragged portions walked row by row, and in chunks (last
    chunks that are not full, both requests in one call), each from the state the one before it left; all against the plain
    recurrence, the states against each other."""
    rows = [np.arange(300), 300 + np.arange(131)]
    slots = [2, 0]
    want = np.concatenate([case.plain(r) for r in rows])
    tol = tol * np.abs(want).max()
    states = {}
    for how in ("walk", "single", "chunks"):
        if how == "chunks" and not case.takes_chunks():
            continue
        state = torch.zeros((4, stride), dtype=torch.float32, device="cuda")
        if how == "single":
            steps = [[(slots[0], [t])] + ([(slots[1], [300 + t])] if t < 131 else []) for t in range(300)]
        elif how == "walk":
            steps = [[(slots[0], rows[0][:33]), (slots[1], rows[1][:2])], [(slots[1], rows[1][2:131]), (slots[0], rows[0][33:34])], [(slots[0], rows[0][34:])]]
        else:
            steps = [[(slots[0], rows[0][:130]), (slots[1], rows[1][:65])], [(slots[1], rows[1][65:]), (slots[0], rows[0][130:293])], [(slots[0], rows[0][293:])]]
        got = case.run(steps, state, how)
        err = np.abs(got - want).max(-1)
        assert err.max() <= tol, f"{how}: error {err.max():.2e} above {tol:.2e} at row {int(err.argmax())}; first bad row {int((err > tol).argmax())}"
        assert not state[1].any() and not state[3].any()
        states[how] = state
    for how in states:
        scale = states["walk"].abs().max()
        assert (states[how] - states["walk"]).abs().max() <= 5e-5 * scale, how
    return states


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(3, 7, 10, 3), (2, 64, 32, 8), (1, 128, 128, 16), (2, 24, 136, 11), (2, 40, 256, 8), (5, 20, 33, 5), (1, 300, 12, 8), (1, 16, 640, 4)])
def test_gated_linear_attention_by_its_three_ways(sizes, dtype):
    H, D, V, _ = sizes
    case = LinearCase(sizes, 431, dtype)
    stride = (H * D * V + 7) // 4 * 4 + (1 if D == 20 else 0)      # (one case with slots that are not aligned to 16 bytes)
    states = _three_ways(case, stride, 1e-4 if dtype == torch.float32 else 1.2e-2)
    assert ("chunks" in states) == (V <= 256 and D <= 128), "sizes on both sides of what the chunks take"
    assert not states["walk"][:, H * D * V:].any()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(3, 7, 10), (2, 64, 32), (1, 128, 128), (2, 24, 136), (2, 40, 300), (5, 20, 33), (1, 200, 12), (1, 150, 260), (35, 4, 8), (1, 8, 600)])
def test_the_matrix_memory_by_its_three_ways(sizes, dtype):
    case = MemoryCase(sizes, 431, dtype)
    states = _three_ways(case, case.stride() + (1 if sizes[1] == 20 else 0), 1.5e-4 if dtype == torch.float32 else 1.2e-2)
    assert ("chunks" in states) == (sizes[2] <= 512)


@pytest.mark.parametrize("how", ["walk", "single", "chunks"])
def test_linear_state_written_long_ago_read_back_and_strong_decays(how):
    """Channels whose decay stays at nearly one carry what one token wrote 400 tokens on; channels whose decay nearly closes at single
    tokens lose it there and then hold what comes next: sums of logarithms far beyond what an exponential can hold, and
    products that must not become infinite or lose what follows."""
    H, D, V, T = 2, 32, 16, 450
    case = LinearCase((H, D, V, D), T, torch.float32, tau=1.0)
    rng = np.random.default_rng(7)
    r = np.zeros((T, case.ld))
    r[:, :H * D] = rng.normal(size=(T, H * D))
    k = np.full((T, H, D), 0.01) * rng.normal(size=(T, H, D))
    k[10] = 1.0                                              # token 10 is written into every channel
    r[:, case.off[1]:case.off[1] + H * D] = k.reshape(T, -1)
    r[:, case.off[2]:case.off[2] + H * V] = rng.normal(size=(T, H * V))
    r[:, case.off[3]:case.off[3] + H * V] = 2.0
    z = np.full((T, D), 9.0)                                 # decay 1 - 1.2e-4: holds
    z[:, 8:16] = rng.normal(size=(T, 8)) * 3.0
    z[np.ix_(range(0, T, 37), range(16, 24))] = -60.0        # closes
    z[200:216, 24:28] = -15.0                                # a whole segment nearly closed
    z[:, 28:] = 15.0                                         # decay 1 - 3e-7
    r[:, case.off[4]:case.off[4] + D] = z
    case.bias = np.zeros(H * D, dtype=np.float32)
    case.gain = np.ones(V, dtype=np.float32)
    case.set(r, _dev(np.concatenate([np.eye(D)] * H), torch.float32))
    want = case.plain(np.arange(T))
    state = torch.zeros((2, H * D * V), dtype=torch.float32, device="cuda")
    got = case.run([[(1, [t])] for t in range(T)] if how == "single" else [[(1, np.arange(T))]], state, how)
    assert np.isfinite(got).all()
    err = np.abs(got - want).max(-1)
    assert err.max() <= 3e-4, f"row {int(err.argmax())}: {err.max():.2e}"
    S = state[1].view(H, D, V).cpu().numpy()
    wrote = r[10, case.off[2]:case.off[2] + H * V].reshape(H, V)
    assert all(np.corrcoef(S[h, i], wrote[h])[0, 1] > 0.9 for h in range(H) for i in list(range(8)) + list(range(28, 32)))


@pytest.mark.parametrize("how", ["walk", "single", "chunks"])
def test_memory_gates_at_their_caps(how):
    """Head 0 keeps everything (forget gate at the cap) and takes one token strongly at position 10: it is what the state holds 400 tokens
    on, and what came after counts for little beside it.  Head 1 forgets everything at single tokens.  Head 2's input gate stays at
    its lowest: |n . q| stays below exp(-m), and the read-out is the undivided state's.  Head 3 changes its maximum at almost every token."""
    H, D, V, T = 4, 24, 20, 450
    case = MemoryCase((H, D, V), T, torch.float32, cap=8.0, W=2 * H)
    rng = np.random.default_rng(9)
    r = rng.normal(size=(T, case.ld))
    # (keys resemble queries, and head 0's queries the key at position 10 as well: no read-out cancels, which would show rounding alone)
    queries, keys = slice(case.off[0], case.off[0] + H * D), slice(case.off[1], case.off[1] + H * D)
    r[:, keys] = 0.5 * r[:, keys] + r[:, queries]
    r[:, case.off[0]:case.off[0] + D] += 2.0 * r[10, case.off[1]:case.off[1] + D]
    pre = np.zeros((T, 2 * H))
    pre[:, 0], pre[10, 0], pre[:, H] = -3.0, 60.0, 90.0
    pre[:, 1], pre[:, H + 1] = 0.0, 3.0
    pre[::37, H + 1] = -90.0
    pre[:, 2], pre[:, H + 2] = -90.0, -1.0
    pre[:, 3], pre[:, H + 3] = np.linspace(-6.0, 6.0, T) + rng.normal(size=T), 1.0
    case.b = np.zeros(2 * H, dtype=np.float32)
    case.gain = np.ones(H * V, dtype=np.float32)
    case.set(r, pre, np.eye(2 * H))
    want = case.plain(np.arange(T))
    state = torch.zeros((2, case.stride()), dtype=torch.float32, device="cuda")
    got = case.run([[(1, [t])] for t in range(T)] if how == "single" else [[(1, np.arange(T))]], state, how)
    assert np.isfinite(got).all()
    err = np.abs(got - want).max(-1)
    assert err.max() <= 4e-4, f"row {int(err.argmax())}: {err.max():.2e}"
    S = state[1, :D * V].view(D, V).cpu().numpy()
    v10, k10 = r[10, case.off[2]:case.off[2] + V], r[10, case.off[1]:case.off[1] + D]
    assert np.corrcoef(S.ravel(), np.outer(k10, v10).ravel())[0, 1] > 0.9
    m = state[1, _pad8(H * D * V) + H * D:][:H].cpu().numpy()
    assert np.all(m <= 8.0 + 1e-5) and m[0] > 7.0 and m[2] < -3.0


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_whole_in_portions_and_decoded(dtype, tmp_path):
    """A prompt over many chunks of the recurrences and several of the attention (600 tokens in one step), the same prompt in
    portions, and its last tokens one by one: all against the plain logits."""
    cfg = LH.model(150, 64, [LH.with_mlp(LH.mlstm(4, 16, 24, 8.0), None), LH.with_mlp(LH.attention(4, 2, 16, 32, 0.25, rot=(1e4, 16)), LH.moe(2, 2, 32, shared=16)),
                             LH.with_mlp(LH.parallel(LH.chunked(4, 2, 8, 16, 0.35, size=150, rot=(1e4, 8)), LH.linear(2, 96, 48, 8.0), 0.8, 1.2), LH.dense(48)),
                             LH.with_mlp(LH.attention(2, 2, 16, 32, 0.3, kv_from=1, rot=(1e4, 16)), LH.moe(1, 1, 48)), LH.with_mlp(LH.mlstm(2, 96, 40, 15.0), None)], 8)
    d = LH.make_model_dir(str(tmp_path), cfg, "long", seed=12)
    ids = LH.tokens(8, 600, 150)
    want = [0, 63, 64, 149, 150, 255, 256, 300, 511, 512, 598, 599]
    whole = run_steps(make_engine(d, dtype), [([("r", ids, want)], ["r"])])
    check(d, {"r": ids}, whole, dtype, f"long prompt whole {dtype}")
    cuts = portions(560, [200, 90, 255, 15]) + [(560 + i, 561 + i) for i in range(40)]
    cut = run_steps(make_engine(d, dtype), [([("r", ids[a:b], [p - a for p in want if a <= p < b])], []) for a, b in cuts])
    check(d, {"r": ids}, cut, dtype, f"long prompt in portions {dtype}")
    assert sorted(cut) == sorted(whole)


def test_keys_far_back_through_another_layers_cache(tmp_path):
    """Two attention layers over one cache; the second's scores are made sharp (a scale far above 1 / sqrt(dim)), so that its rows are
    dominated by single keys anywhere in the sequence: 32-bit, a prompt of 300 in one step, in portions and decoded."""
    cfg = LH.model(131, 40, [LH.with_mlp(LH.attention(2, 2, 8, 8, 0.3, rot=(1e5, 4)), None), LH.with_mlp(LH.attention(6, 2, 8, 8, 4.0, kv_from=0, rot=(1e5, 4)), None)], 4)
    d = LH.make_model_dir(str(tmp_path), cfg, "far", seed=3)
    c, w = LH.load_model_dir(d)
    ids = np.asarray(LH.tokens(3, 300, 131))
    at = np.arange(300)
    m0, m1 = (l["mixer"] for l in c["layers"])
    x = w["embed"][ids]
    k, v = Z.own_keys_values(x, w, "l0.mix.", m0, at, 1e-5)
    x = x + Z.norm_around_one(Z.sink_attention_mixer(x, k, v, w, "l0.mix.", m0, at, 1e-5), w["l0.norm1"], 1e-5)
    x = x + Z.rms_unit(Z.token_side(x, w["side.embed"][ids, :4], w["l0.side.gate"], w["l0.side.proj"]), 1e-5) * w["l0.side.norm"]
    q = Z.rotate((Z.rms_unit(x @ w["l1.mix.q"].T, 1e-5) * w["l1.mix.q.norm"]).reshape(300, 6, 8), at, 1e5, 4, neighbours=False)
    s = np.einsum("thd,shd->ths", q, np.repeat(k, 3, axis=1))[-30:] * 4.0
    far = s.argmax(-1)
    assert (np.sort(s, -1)[..., -1] - np.sort(s, -1)[..., -20] > 3.0).mean() > 0.5 and (far < 200).mean() > 0.4, "keys far back must stand out"
    for cuts in ([(0, 300)], portions(280, [33, 2, 64, 90, 17, 74]) + [(280 + i, 281 + i) for i in range(20)]):
        got = run_steps(make_engine(d, "float32"), [([("r", ids[a:b].tolist(), list(range(b - a)))], []) for a, b in cuts])
        check(d, {"r": ids.tolist()}, got, "float32", "keys far back")


@pytest.mark.parametrize("dtype", DTYPES)
def test_chunk_edges_show_in_the_logits(dirs, dtype):
    """Just before, at and just behind every chunk's edge, with scores so sharp that one key more or less changes the row: in a prompt and
    decoded; a model with chunks one position longer gives other rows there."""
    import copy
    d = dirs["pair"] if dtype == "float32" else dirs["pair_aligned"]
    with open(os.path.join(d, "config.json")) as f:
        size = json.load(f)["layers"][0]["mixer"]["left"]["mask"]["size"]
    cfg, w = LH.load_model_dir(d)
    longer = copy.deepcopy(cfg)
    longer["layers"][0]["mixer"]["left"]["mask"]["size"] = size + 1
    n = 3 * size + 2
    ids = LH.tokens(31, n, vocab_of(d))
    edges = sorted({p for e in range(size, n, size) for p in (e - 1, e, e + 1) if p < n})
    plain, other = LH.plain_logits(d, ids), Z.forward(longer, w, ids)
    rel = np.sqrt(((plain - other) ** 2).sum(-1) / (plain ** 2).sum(-1))
    assert rel[size] > 0.15 and rel[2 * size] > 0.15, "one key more or less must show"
    whole = run_steps(make_engine(d, dtype), [([("r", ids, edges)], ["r"])])
    check(d, {"r": ids}, whole, dtype, "chunk edges in a prompt")
    one = run_steps(make_engine(d, dtype), [([("r", ids[:size - 2], [])], [])] + [([("r", [t], [0])], []) for t in ids[size - 2:]])
    check(d, {"r": ids}, {k: v for k, v in one.items() if k[1] in edges}, dtype, "chunk edges decoded")


def test_captured_steps_repeat_and_agree_with_eager_ones(dirs):
    """A captured decode step (graphs of one and of several steps, replayed over and over with eager work between) gives what
    the same steps give without a graph, for requests of different lengths."""
    from gibbs_amd.engine.decode import DecodeLoop
    d = dirs["B"]
    prompts = [LH.tokens(80 + i, n, vocab_of(d)) for i, n in enumerate([9, 38, 25])]
    logs = []
    for use_graph in (True, False):
        eng = make_engine(d, "bfloat16")
        last = []
        for i, p in enumerate(prompts):
            last.append(int(eng.step([(f"r{i}", p, [len(p) - 1])]).argmax(-1)[0]))
        loop = DecodeLoop(eng, [f"r{i}" for i in range(3)], last, use_graph=use_graph)
        tokens = []
        for n in (3, 9, 1, 20):
            loop.run(n)
            tokens.append(np.asarray(loop.tokens(n)).reshape(-1))
            eng.step([("other", [1, 2, 3], [2])])
            eng.release("other")
        logs.append(np.concatenate(tokens))
    assert np.array_equal(logs[0], logs[1])


# ----------------------------------------------------------------------------------------------- entry points
def plain_greedy(model_dir, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(np.argmax(LH.plain_logits(model_dir, ids)[-1])))
    return ids[len(prompt):]


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_scheduler(dirs, dtype):
    """`generate` (scheduler, prompt steps, bursts of captured decode steps) gives the plain implementation's greedy
    tokens; in bfloat16 wherever the plain logits' lead exceeds the precision's error."""
    from gibbs_amd import Engine, generate
    held = 0
    for name, lens in (("A", [7, 13, 2]), ("D", [5])):
        d = variants(dirs, name, dtype)[-1]
        eng = Engine(d, dtype=dtype, max_tokens=512, max_requests=4)
        prompts = [LH.tokens(40 + i, n, vocab_of(d)) for i, n in enumerate(lens)]
        outs = generate(eng, prompts, max_tokens=20, temperature=0.0, ignore_eos=True)
        for p, o in zip(prompts, outs):
            assert o.finish_reason == "length" and len(o.tokens) == 20
            if dtype == "float32":
                assert o.tokens == plain_greedy(d, p, 20)
                held += 20
                continue
            logits = LH.plain_logits(d, list(p) + list(o.tokens))
            for i, t in enumerate(o.tokens):
                row = logits[len(p) - 1 + i]
                best, second = np.sort(row)[[-1, -2]]
                margin = 2 * 0.05 * np.abs(row).max()
                if best - second > margin:
                    held += 1
                    assert t == int(np.argmax(row)), f"token {i}"
                else:
                    assert row[t] >= best - margin, f"token {i}"
        eng.cache.check()
        assert eng.cache.free_slots() == 4
    assert held >= 20


def test_decode_bursts_change_nothing(dirs):
    from gibbs_amd import Engine, Generator, SamplingParams
    d = dirs["B"]
    prompts = [LH.tokens(70 + i, n, vocab_of(d)) for i, n in enumerate([9, 21, 5])]
    runs = []
    for burst in (0, 16):
        eng = Engine(d, dtype="float32", max_tokens=1024, max_requests=4)
        gen = Generator(eng, decode_burst=burst, eos_token_ids=())
        rids = [gen.submit(p, SamplingParams(temperature=0.0, max_new_tokens=n), rid=f"r{i}") for i, (p, n) in enumerate(zip(prompts, [60, 20, 9]))]
        res = gen.run()
        runs.append([res[r].tokens for r in rids])
    assert runs[0] == runs[1]
    assert runs[0][0] == plain_greedy(d, prompts[0], 60)


@pytest.mark.parametrize("dtype", DTYPES)
def test_replay_program(dirs, dtype, tmp_path):
    d = dirs["C"]                  # (every router output is chosen there: no choice can fall the other way)
    ids = pick(d, 50, 40)
    other = pick(d, 51, 9)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:17], "want": [0, 16]}, {"id": "b", "tokens": other[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": other[2:], "want": [6]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": ids[17:39], "want": [21]}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": ids[39:], "want": [0]}], "end": ["a"]}]
    out = tmp_path / "out"
    proc = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", dtype, "--out", str(out), "--max-tokens", "128"],
                          input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    want_a, want_b = LH.plain_logits(d, ids), LH.plain_logits(d, other)
    read = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab_of(d))
    close(read(0), want_a[[0, 16]], dtype, "step 0")
    close(read(1), want_b[[8]], dtype, "step 1")
    close(read(2), want_a[[38]], dtype, "step 2")
    close(read(3), want_a[[39]], dtype, "step 3")


def test_command_line(dirs):
    d = dirs["A"]
    prompt = LH.tokens(60, 6, vocab_of(d))
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "gibbs"), "--model", d, "--dtype", "float32", "--prompt-ids",
                           ",".join(map(str, prompt)), "--max-tokens", "8", "--temperature", "0", "--ignore-eos"],
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    line = proc.stdout.split("✨ Output:\n")[1].splitlines()[0]
    assert [int(t) for t in line.split()] == plain_greedy(d, prompt, 8)
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "gibbs"), "--model", d, "--arch-dump"], capture_output=True, text=True, timeout=600)
    dump = json.loads(proc.stdout)
    assert dump["architecture"] == "Lubavik" and dump["unconsumed"] == [] and dump["missing"] == []
    assert dump["derived"]["layers_by_type"] == {"attention": 3, "parallel": 1, "mlstm": 1}
