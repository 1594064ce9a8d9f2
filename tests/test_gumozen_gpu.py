"""Gumozen on the GPU against the plain implementation, in 32-bit and in bfloat16: each mechanism alone; whole prompts;
most of a prompt in one step and its last tokens one by one; portions of changing size down to two tokens; mixed
batches in a pool so small that pages and slots are used again; long decoding; the first tokens; kernels with inputs
made so that one key at a chunk's edge, a state written long ago, a strong decay, a map or a router's choice stands
out; generation through the scheduler, the replay program and the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import gumozen_helpers as GH
from tests.plain import gumozen_plain as Z
from tests.test_engine_gpu import mixed_schedule, portions, run_steps

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]
NAMES = ["A", "B", "C", "D"]
LENGTHS = {"A": 150, "B": 230, "C": 120, "D": 140}
# bfloat16 against the plain implementation, per row: relative L2 error of the logits.  A router's choice between two
# experts whose scores differ by less than the rounding of its input may fall the other way than in float64, and with a
# norm behind the experts that changes the token's whole row, which every later token may read: a sequence is held to the
# bound up to its first token whose least clear choice (`route_margin`) is below CLEAR_CHOICE (sequences are picked so that
# this comes late, `clear_tokens`).  So that every row of every test is held to the bound in bfloat16 as well, each model
# also runs in a copy whose routers always choose clearly (`settle_choices`).  A sublayer's result is normed before it is
# added, and a differential head's before it is projected: where it nearly cancels for a token, the division by its root mean
# square amplifies the rounding of its operands: a few rows in a hundred may exceed the bound, none by more than BF16_WORST.
BF16_REL_L2 = 0.06
BF16_ROWS_OVER = 0.03
BF16_WORST = 0.5
CLEAR_CHOICE = 0.01


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("gumozen")
    out = {n: GH.make_model_dir(str(root), GH.MODELS[n], n, seed=41 + i) for i, n in enumerate(NAMES)}
    out.update({n + "_settled": GH.settle_choices(out[n], str(root)) for n in NAMES})
    one = GH.single_layer
    out["differential"] = GH.make_model_dir(str(root), one(GH.differential(6, 2, 10, 18, 0.4, 0.3, size=11, rot=(1000.0, 8), scaling=(4.0, 1.0, 4.0, 40))), "differential", seed=5)
    out["differential_aligned"] = GH.make_model_dir(str(root), one(GH.differential(4, 2, 24, 48, 0.25, 0.7, size=40, rot=(1e4, 24)), width=64), "differential_aligned", seed=6)
    out["recurrence"] = GH.make_model_dir(str(root), one(GH.recurrence(5, 12, 9)), "recurrence", seed=7)
    out["latent"] = GH.make_model_dir(str(root), one(GH.latent(3, 14, 10, 20, 18, 0.5)), "latent", seed=8)
    out["shared_latent"] = GH.make_model_dir(str(root), GH.model(131, 60, [GH.with_mlp(GH.latent(4, 10, 12, 24, 16, 0.6), None), GH.with_mlp(GH.latent(2, 6, 20, 24, 8, 0.8, kv_from=0), None)]),
                                             "shared_latent", seed=10)
    out["experts"] = GH.make_model_dir(str(root), one(GH.recurrence(2, 8, 10), GH.moe(7, 3, 36)), "experts", seed=9)
    out["experts_settled"] = GH.settle_choices(out["experts"], str(root))
    return out


def make_engine(model_dir, dtype, **kw):
    from gibbs_amd import Engine
    kw.setdefault("max_tokens", 2048)
    kw.setdefault("max_requests", 4)
    return Engine(model_dir, dtype=dtype, **kw)


def close(got, want, dtype, what):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    assert got.shape == want.shape, (what, got.shape, want.shape)
    if dtype == "float32":
        err = np.abs(got - want).max(-1)
        bound = 3e-5 * np.abs(want).max()
        assert err.max() <= bound, f"{what}: max error {err.max():.3e} at row {int(err.argmax())} above {bound:.3e}; first bad row {int((err > bound).argmax())}"
        return
    rel = np.sqrt(((got - want) ** 2).sum(-1) / (want ** 2).sum(-1))
    assert np.isfinite(rel).all(), what
    over = rel > BF16_REL_L2
    assert over.sum() <= max(2, int(BF16_ROWS_OVER * rel.size)) and rel.max() <= BF16_WORST, \
        f"{what}: relative L2 error {rel.max():.3e}; {int(over.sum())} of {rel.size} rows over; first bad row {int(over.argmax())}"


def check(model_dir, seqs, got, dtype, what):
    compared = total = 0
    for rid, ids in seqs.items():
        want = GH.plain_logits(model_dir, ids)
        places = sorted(p for r, p in got if r == rid)
        assert places, f"{what}: no logits for {rid}"
        total += len(places)
        if dtype != "float32":
            unclear = np.nonzero(GH.plain_margins(model_dir, ids) < CLEAR_CHOICE)[0]
            places = [p for p in places if not unclear.size or p < unclear[0]]
            if not places:
                continue
        compared += len(places)
        close(np.stack([got[(rid, p)] for p in places]), want[places], dtype, f"{what} request {rid}")
    assert compared == total or not model_dir.endswith("_settled"), f"{what}: {total - compared} rows of a model with settled choices were not compared"


def variants(dirs, name, dtype):
    """The model's folder, and for bfloat16 also its copy with settled choices of experts."""
    return [dirs[name]] + ([dirs[name + "_settled"]] if dtype == "bfloat16" and name + "_settled" in dirs else [])


def pick(model_dir, seed, n):
    return GH.clear_tokens(model_dir, seed, n, vocab_of(model_dir), CLEAR_CHOICE)


def vocab_of(model_dir):
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)["vocab"]


# ----------------------------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["differential", "differential_aligned", "recurrence", "latent", "shared_latent", "experts"])
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
    """Cuts in the middle of pages and chunks; portions on both sides of what the recurrence takes in chunks."""
    for d in variants(dirs, name, dtype):
        ids = pick(d, 4, LENGTHS[name])
        cuts = portions(len(ids) - 9, [7, 2, 13, 3, 2, 97, 5, 2, 17, 1, 2]) + [(len(ids) - 9 + i, len(ids) - 8 + i) for i in range(9)]
        steps = [([("r", ids[a:b], list(range(b - a)))], []) for a, b in cuts]
        got = run_steps(make_engine(d, dtype), steps)
        check(d, {"r": ids}, got, dtype, f"portions {name} {dtype}")


@pytest.mark.parametrize("name", NAMES)
def test_cutting_and_batching_change_nothing_in_32_bit(dirs, name):
    """Products add in ascending k, the attention takes keys in blocks aligned to absolute positions, the recurrence keeps a
    request's tokens in order, and an expert's result for a row does not depend on which other rows the expert serves: 32-bit
    logits do not depend on how the prompt was cut or on what else was in the batch, beyond rounding."""
    d = dirs[name]
    ids = GH.tokens(5, 77, vocab_of(d))
    other = GH.tokens(6, 41, vocab_of(d))
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
    """Decoded tokens at the head of a batch beside a portion that the recurrence takes in chunks and one that is shorter than a
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
    """Sequences of one, two, three and five tokens, side by side and one token at a time: a single visible key, no row before
    the first, an empty state."""
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


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [48, 51, 1024, 4096])
def test_rows_of_the_stream_shifted_through_short_portions_and_a_reused_slot(dtype, W):
    """Three requests in portions of 1, 2, 5, 1, ... rows, states in scattered slots; a slot that is cleared starts from zeros."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(3)
    mu = rng.normal(size=W)
    seqs = [rng.normal(size=(n, W)) for n in (23, 17, 9)]
    state = torch.zeros((5, W + 3), dtype=torch.float32, device="cuda")
    slots, at, got, step = [2, 0, 4], [0, 0, 0], [[], [], []], 0
    sizes = [1, 2, 5, 1, 1, 3, 7, 2, 30]
    while any(at[r] < len(seqs[r]) for r in range(3)):
        rows, cu, req, live = [], [0], [], []
        for r in range(3):
            n = min(sizes[(step + r) % len(sizes)], len(seqs[r]) - at[r])
            if n > 0:
                live.append((r, n))
                rows.append(seqs[r][at[r]:at[r] + n])
                req += [len(live) - 1] * n
                cu.append(cu[-1] + n)
        x = _dev(np.concatenate(rows))
        out = torch.empty_like(x, dtype=dtype)
        call("gibbs_stream_shift", ptr(x), ptr(_dev(mu)), ptr(state), state.stride(0), ptr(_dev(req, torch.int32)), ptr(_dev(cu, torch.int32)),
             ptr(_dev([slots[r] for r, _ in live], torch.int32)), ptr(out), dtype_code(dtype), x.shape[0], W, stream())
        o = _f64(out)
        for i, (r, n) in enumerate(live):
            got[r].append(o[cu[i]:cu[i + 1]])
            at[r] += n
        step += 1
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    for r in range(3):
        want = Z.token_shift(seqs[r].astype(np.float32).astype(np.float64), mu.astype(np.float32).astype(np.float64))
        assert np.abs(np.concatenate(got[r]) - want).max() <= tol * np.abs(want).max(), r
        assert np.array_equal(state[slots[r], :W].cpu().numpy(), seqs[r][-1].astype(np.float32))
    assert not state[1].any() and not state[3].any() and not state[:, W:].any()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("mixed", [0, 1, 3])
@pytest.mark.parametrize("W", [100, 2048, 5120])
def test_a_sublayers_result_added_and_the_rows_that_the_next_one_reads(dtype, mixed, W):
    """x += norm(result) in one pass with nothing, the rows as they are, or the rows shifted; the result whole, or a mixture of
    experts' rows still to be summed (with weights and without)."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(1)
    n = 6
    x0, gain, mu = rng.normal(size=(n, W)), rng.normal(size=W) + 1.0, rng.normal(size=W)
    rows = _dev(rng.normal(size=(n * max(mixed, 1), W)), dtype)
    place = rng.permutation(n * mixed).reshape(n, mixed) if mixed else None
    weight = rng.uniform(0.2, 1.0, size=(n, mixed)).astype(np.float32) if mixed == 3 else None
    r64 = _f64(rows)
    delta = r64 if not mixed else (r64[place] * (1.0 if weight is None else weight.astype(np.float64)[:, :, None])).sum(1)
    want_x = x0.astype(np.float32) + Z.rms_unit(delta, 1e-5) * gain.astype(np.float32)
    state0 = rng.normal(size=(n + 2, W)).astype(np.float32)
    slots = [3, 0, 7, 1, 5, 2]
    for read in (0, 1, 2):
        x, state = _dev(x0), _dev(state0)
        out = torch.full((n, W), 9.0, dtype=dtype, device="cuda")
        call("gibbs_rmsnorm_rows_add_read", ptr(x), ptr(rows), 1, n * W, ptr(_dev(place, torch.int32)) if mixed else None,
             ptr(_dev(weight)) if weight is not None else None, mixed, None, None, ptr(_dev(gain)), 1e-5, read, ptr(_dev(mu)), ptr(state), W,
             ptr(_dev(slots, torch.int32)), ptr(out), dtype_code(dtype), n, W, stream())
        assert np.abs(_f64(x) - want_x).max() <= 2e-5 * np.abs(want_x).max()
        if read == 0:
            assert (out == 9.0).all()
            continue
        before = state0[slots].astype(np.float64)
        want = want_x if read == 1 else want_x + (before - want_x) * mu.astype(np.float32)
        assert np.abs(_f64(out) - want).max() <= (3e-5 if dtype == torch.float32 else 1e-2) * np.abs(want).max()
        if read == 2:
            assert torch.equal(state[slots], x) and torch.equal(state[[4, 6]].cpu(), torch.tensor(state0[[4, 6]]))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_normed_embedding(dtype):
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(4)
    for W in (52, 51, 3000):
        table, gain = _dev(rng.normal(size=(20, W)) * 0.01, dtype), rng.normal(size=W)
        ids = [3, 19, 0, 3]
        x = torch.empty((4, W), dtype=torch.float32, device="cuda")
        call("gibbs_embed_norm", ptr(table), dtype_code(dtype), ptr(_dev(ids, torch.int32)), ptr(x), ptr(_dev(gain)), 1e-4, 4, W, 20, stream())
        want = Z.rms_unit(_f64(table)[ids], 1e-4) * gain.astype(np.float32)
        assert np.abs(_f64(x) - want).max() <= 1e-5 * np.abs(want).max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(6, 3, 10, 14, 6, 20, 14), (3, 1, 24, 40, 24, 48, 48), (2, 2, 64, 128, 32, 128, 128), (2, 1, 150, 300, 20, 300, 300), (4, 2, 5, 3, 0, 16, 16)])
def test_projected_rows_become_two_maps_and_the_heads_are_combined(dtype, sizes):
    """q and k normed per map and turned, a map's query zero elsewhere, keys of both maps side by side, keys and values in their
    pages on both sides of page borders and far out; then a_1 - lambda a_2, normed, scaled and gated."""
    from gibbs_amd.ops.lib import call, dtype_code, ptr, stream
    rng = np.random.default_rng(2)
    H, G, D, V, rot, ks, vs = sizes
    ps, places = 16, [0, 15, 16, 17, 31, 250, 70000]
    n = len(places)
    ld = 2 * (H + G) * D + G * V + H + 5
    rows = _dev(rng.normal(size=(n, ld)), dtype)
    r64 = _f64(rows)
    qg, kg = (rng.normal(size=D) + 1.0).astype(np.float32), (rng.normal(size=D) + 1.0).astype(np.float32)
    freq = Z.frequencies(1000.0, rot, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}) if rot else None
    n_pages = 70000 // ps + 1
    kpages = torch.full((n_pages, G, ps, ks), 7.0, dtype=dtype, device="cuda")
    vpages = torch.full((n_pages, G, ps, vs), 7.0, dtype=dtype, device="cuda")
    table = torch.arange(n_pages - 1, -1, -1, dtype=torch.int32, device="cuda").view(1, n_pages).contiguous()
    q_out = torch.full((n, 2 * H, ks), 7.0, dtype=dtype, device="cuda")
    call("gibbs_diff_prepare", ptr(rows), ld, ptr(q_out), ptr(kpages), ptr(vpages), dtype_code(dtype), ptr(_dev(qg)), ptr(_dev(kg)), 1e-5,
         ptr(_dev(freq)) if rot else None, rot, 0, None, 0, ptr(_dev(places, torch.int32)), ptr(_dev([0] * n, torch.int32)), ptr(table), n_pages, ps, n_pages, n, H, G, D, V,
         ks, vs, stream())

    def maps(flat, heads, gain):
        x = Z.rms_unit(flat.reshape(n, heads * 2, D), 1e-5) * gain.astype(np.float64)
        return Z.rotate(x, places, freq, rot) if rot else x

    q, k = maps(r64[:, :2 * H * D], H, qg), maps(r64[:, 2 * H * D:2 * (H + G) * D], G, kg)
    v = r64[:, 2 * (H + G) * D:2 * (H + G) * D + G * V].reshape(n, G, V)
    want_q = np.zeros((n, 2 * H, ks))
    for c in range(2):
        want_q[:, c::2, c * D:(c + 1) * D] = q[:, c::2]
    tol = 4e-5 if dtype == torch.float32 else 0.15
    assert np.abs(_f64(q_out) - want_q).max() <= tol
    assert np.array_equal(_f64(q_out) == 0.0, want_q == 0.0)
    want_k, want_v = np.zeros((n, G, ks)), np.zeros((n, G, vs))
    want_k[:, :, :2 * D] = k.reshape(n, G, 2 * D)
    want_v[:, :, :V] = v
    for i, p in enumerate(places):
        page = n_pages - 1 - p // ps
        assert np.abs(_f64(kpages[page, :, p % ps]) - want_k[i]).max() <= tol, p
        assert np.abs(_f64(vpages[page, :, p % ps]) - want_v[i]).max() <= 1e-6, p
    assert int((kpages != 7.0).any(-1).sum()) == n * G and int((vpages != 7.0).any(-1).sum()) == n * G      # nothing else was written
    att = rng.normal(size=(n, 2 * H, vs))
    att[:, 1::2] = att[:, ::2] * 1.1 + 0.05 * att[:, 1::2]                # (maps that nearly cancel)
    att = _dev(att, dtype)
    o = torch.empty((n, H * V), dtype=dtype, device="cuda")
    gate_off = 2 * (H + G) * D + G * V
    call("gibbs_diff_finish", ptr(att), vs, rows.data_ptr() + gate_off * rows.element_size(), ld, ptr(_dev([0.8])), 1e-5, 0.3, ptr(o), dtype_code(dtype), n, H, V, stream())
    a64 = _f64(att)[:, :, :V]
    lam = float(np.float32(0.8))
    want = Z.rms_unit(a64[:, ::2] - lam * a64[:, 1::2], 1e-5) * 0.3 * Z.sigmoid(r64[:, gate_off:gate_off + H])[:, :, None]
    assert np.abs(_f64(o).reshape(n, H, V) - want).max() <= (2e-5 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("kernel", ["plain32", "plain16", "decode", "prefill"])
def test_each_map_at_a_chunks_edges(kernel):
    """Two maps over the same values, pages of 16 scattered over the pool, 700 keys, chunks of 180.  In map 1 one key is made to
    dominate, in map 2 another: each map's output is its own key's value where the chunk lets the last row see it (the chunk's
    first key, a page's border, the row itself), and not one key earlier."""
    from gibbs_amd import ops
    rng = np.random.default_rng(0)
    dtype = torch.float32 if kernel == "plain32" else torch.bfloat16
    T, H, G, D, V, ps, n_pages, size = 700, 4, 2, 16, 32, 16, 64, 180
    p = T - 1
    first = p - p % size
    order = rng.permutation(n_pages)[:-(-T // ps)].tolist()
    table = _dev([order], torch.int32)
    keys, vals = _dev(rng.normal(size=(T, G, 2 * D)) * 0.1, dtype), _dev(rng.normal(size=(T, G, V)), dtype)
    maps = rng.normal(size=(2 * H, D)) * 0.3
    q0 = np.zeros((2 * H, 2 * D))
    for c in range(2):
        q0[c::2, c * D:(c + 1) * D] = maps[c::2]
    q = _dev(q0.reshape(1, -1), dtype)
    qd = q.float().view(2 * H, 2 * D)

    def pages_of(rows):
        pages = torch.full((n_pages, G, ps, rows.shape[-1]), 7.0, dtype=dtype, device="cuda")
        for t in range(T):
            pages[order[t // ps], :, t % ps] = rows[t]
        return pages

    vp = pages_of(vals)
    h, g = 2, 1                                                     # head 2 reads kv head 1
    for one, two in ((first, first + 5), (first - 1, p), (p, first - 1), ((first // ps + 1) * ps, (first // ps + 1) * ps - 1)):
        k_rows = keys.clone()
        for c, at in ((0, one), (1, two)):
            m = qd[2 * h + c, c * D:(c + 1) * D]
            k_rows[at, g, c * D:(c + 1) * D] = (m / m.norm() ** 2 * 14.0).to(dtype)
        kp = pages_of(k_rows)
        pos, req = _dev([p], torch.int32), torch.zeros(1, dtype=torch.int32, device="cuda")
        if kernel.startswith("plain"):
            out = ops.attention_plain(q, 1, 2 * H, G, 2 * D, kp, vp, table, 1, pos, req, 1.0, chunk=size)
        elif kernel == "decode":
            out = ops.attention_decode(q, 1, 2 * H, G, 2 * D, kp, vp, table, 1, pos, req, 1.0, max_seq=T, n_splits=3, chunk=size)
        else:
            n = 40
            qs = torch.zeros((n, 2 * H * 2 * D), dtype=dtype, device="cuda")
            qs[-1] = q[0]
            out = ops.attention_prefill(qs, n, 2 * H, G, 2 * D, kp, vp, table, 1, _dev([0, n], torch.int32), _dev([T - n], torch.int32), 1.0, max_seq=T, chunk=size)[-1:]
        got = _f64(out).reshape(2 * H, V)
        kk, vv = _f64(k_rows), _f64(vals)
        for c, at in ((0, one), (1, two)):
            want = Z.softmax_attention(np.repeat(_f64(qd)[None, 2 * h + c:2 * h + c + 1], T, 0), kk[:, g:g + 1], vv[:, g:g + 1], 1.0, Z.visible_chunk(T, size))[-1, 0]
            assert np.abs(got[2 * h + c] - want).max() <= (3e-5 if kernel == "plain32" else 0.1), (one, two, c)
            assert (np.abs(got[2 * h + c] - vv[at, g]).max() < 0.2) == (at >= first), (one, two, c)


def _gated_raw(rng, T, H, D, V, dtype):
    return _dev(rng.normal(size=(T, H * (2 * D + V))), dtype)


def _gated_plain(raw, bias, lower, gain, eps, H, D, V):
    r = _f64(raw)
    T, C = r.shape[0], H * D
    q = Z.silu(r[:, :C]).reshape(T, H, D)
    f = Z.forget_gate(r[:, C:2 * C], bias.astype(np.float64), lower.astype(np.float64)).reshape(T, H, D)
    y = Z.gated_outer_scan(q, f, r[:, 2 * C:].reshape(T, H, V))
    return (Z.rms_unit(y, eps) * gain).reshape(T, H * V), y


def _run_gated(raw, pieces, bias, lower, gain, eps, H, D, V, state, how, dtype):
    """The kernels of one kind over `pieces`, a list of steps of [(slot, rows of `raw`), ..] -> one output row per row of raw."""
    from gibbs_amd.ops.lib import call, dtype_code, library, ptr, stream
    b, l, g = _dev(bias), _dev(lower), _dev(gain)
    out = torch.zeros((raw.shape[0], H * V), dtype=dtype, device="cuda")
    code = dtype_code(dtype)
    for step in pieces:
        index = np.concatenate([np.asarray(rows) for _, rows in step])
        x = raw[_dev(index, torch.int64)].contiguous()
        _alive.append(x)
        n, R = x.shape[0], len(step)
        cu = _dev(np.concatenate([[0], np.cumsum([len(rows) for _, rows in step])]), torch.int32)
        slots = _dev([s for s, _ in step], torch.int32)
        y = torch.empty((n, H * V), dtype=dtype, device="cuda")
        if how == "step":
            call("gibbs_gated_outer_step", ptr(x), x.shape[1], code, ptr(b), ptr(l), ptr(g), eps, ptr(state), state.stride(0), ptr(slots), ptr(y), R, H, D, V, stream())
        elif how == "chunks":
            floats = library().gibbs_gated_outer_chunks_workspace(n, R, H, D, V)
            work = torch.full((floats,), float("nan"), dtype=torch.float32, device="cuda")
            call("gibbs_gated_outer_chunks", ptr(x), x.shape[1], code, ptr(b), ptr(l), ptr(g), eps, ptr(state), state.stride(0), ptr(cu), ptr(slots), ptr(y), ptr(work),
                 n, R, H, D, V, stream())
            _alive.append(work)
        else:
            q, f, k = (torch.empty((n, H * D), dtype=torch.float32, device="cuda") for _ in range(3))
            v, o = (torch.empty((n, H * V), dtype=torch.float32, device="cuda") for _ in range(2))
            call("gibbs_gated_outer_prep", ptr(x), x.shape[1], code, ptr(b), ptr(l), ptr(q), ptr(f), ptr(k), ptr(v), n, H, D, V, stream())
            call("gibbs_gated_outer_rule", ptr(q), ptr(k), ptr(v), ptr(f), ptr(state), state.stride(0), ptr(cu), ptr(slots), ptr(o), R, H, D, V, stream())
            call("gibbs_head_norm_gate", ptr(o), ptr(g), V, None, 0, ptr(y), code, n, H, V, eps, 0, stream())
            torch.cuda.synchronize()
        out[_dev(index, torch.int64)] = y
    torch.cuda.synchronize()
    return _f64(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(3, 7, 10), (2, 64, 32), (1, 128, 128), (2, 24, 136), (2, 40, 256), (5, 20, 33)])
def test_the_recurrence_by_its_three_ways(sizes, dtype):
    """Two requests (300 and 131 rows) in scattered slots: token by token through the step kernel, in ragged portions through the
    walk, and in chunks (sizes that are no multiples of the tiles, last chunks that are not full, both requests in one call),
    each from the state the one before it left; all against the plain recurrence, the states against each other."""
    from gibbs_amd.ops.lib import library
    H, D, V = sizes
    rng = np.random.default_rng(5)
    eps = 1e-5
    lens, slots = [300, 131], [2, 0]
    raw = _gated_raw(rng, sum(lens), H, D, V, dtype)
    bias = (rng.normal(size=H * D) + 2.0).astype(np.float32)
    lower, gain = rng.uniform(0.0, 0.95, size=H * D).astype(np.float32), (rng.normal(size=V) + 1.0).astype(np.float32)
    rows = [np.arange(300), 300 + np.arange(131)]
    want = np.concatenate([_gated_plain(raw[r[0]:r[-1] + 1], bias, lower, gain, eps, H, D, V)[0] for r in rows])
    tol = (1e-4 if dtype == torch.float32 else 1.2e-2) * np.abs(want).max()
    stride = (H * D * V + 7) // 4 * 4 + (1 if D == 20 else 0)      # (one case with slots that are not aligned to 16 bytes)
    states = {}
    for how in ("walk", "step", "chunks"):
        assert library().gibbs_gated_outer_chunks_take(D, V) and library().gibbs_gated_outer_step_takes(D, V)
        state = torch.zeros((4, stride), dtype=torch.float32, device="cuda")
        if how == "step":
            steps = [[(slots[0], [t])] + ([(slots[1], [300 + t])] if t < 131 else []) for t in range(300)]
        elif how == "walk":
            steps = [[(slots[0], rows[0][:33]), (slots[1], rows[1][:2])], [(slots[1], rows[1][2:131]), (slots[0], rows[0][33:34])], [(slots[0], rows[0][34:])]]
        else:
            steps = [[(slots[0], rows[0][:130]), (slots[1], rows[1][:65])], [(slots[1], rows[1][65:]), (slots[0], rows[0][130:293])], [(slots[0], rows[0][293:])]]
        got = _run_gated(raw, steps, bias, lower, gain, eps, H, D, V, state, how, dtype)
        err = np.abs(got - want).max(-1)
        assert err.max() <= tol, f"{how}: error {err.max():.2e} above {tol:.2e} at row {int(err.argmax())}; first bad row {int((err > tol).argmax())}"
        assert not state[1].any() and not state[3].any() and not state[:, H * D * V:].any()
        states[how] = state
    for how in states:
        scale = states["walk"].abs().max()
        assert (states[how] - states["walk"]).abs().max() <= 3e-5 * scale, how


@pytest.mark.parametrize("how", ["walk", "step", "chunks"])
def test_a_state_written_long_ago_read_back_and_strong_decays(how):
    """Channels whose gate stays at nearly one carry what one token wrote 400 tokens on; channels whose gate nearly closes
    at single tokens, and whose lower bound is zero, lose it there and then hold what comes next: sums of logarithms far beyond
    what an exponential can hold, and products that must not become infinite or lose what follows."""
    H, D, V, T = 2, 32, 16, 450
    rng = np.random.default_rng(7)
    dtype = torch.float32
    r = np.zeros((T, H * (2 * D + V)))
    C = H * D
    r[:, :C] = rng.normal(size=(T, C))
    z = np.full((T, H, D), 9.0)                       # f = 1 - 1.2e-4: holds
    z[10] = -3.0                                      # token 10 is written into every channel
    z[:, :, 8:16] = rng.normal(size=(T, H, 8)) * 3.0
    z[np.ix_(range(0, T, 37), range(H), range(16, 24))] = -60.0     # closes: f = 8.8e-27 with a bound of zero
    z[200:216, :, 24:28] = -25.0                      # a whole segment nearly closed
    z[:, :, 28:] = -2.0
    r[:, C:2 * C] = z.reshape(T, C)
    r[:, 2 * C:] = rng.normal(size=(T, H * V)) * 0.1
    r[10, 2 * C:] = rng.normal(size=H * V)
    raw = _dev(r, dtype)
    bias, lower, gain = np.zeros(C, dtype=np.float32), np.zeros(C, dtype=np.float32), np.ones(V, dtype=np.float32)
    want, y = _gated_plain(raw, bias, lower, gain, 1e-6, H, D, V)
    state = torch.zeros((2, H * D * V), dtype=torch.float32, device="cuda")
    steps = {"walk": [[(1, np.arange(T))]], "step": [[(1, [t])] for t in range(T)], "chunks": [[(1, np.arange(T))]]}[how]
    got = _run_gated(raw, steps, bias, lower, gain, 1e-6, H, D, V, state, how, dtype)
    assert np.isfinite(got).all()
    err = np.abs(got - want).max(-1)
    assert err.max() <= 3e-4, f"row {int(err.argmax())}: {err.max():.2e}"
    # the token at 10 is what the channels 0 .. 7 still hold at the end
    S = state[1].view(H, D, V).cpu().numpy()
    wrote = r[10, 2 * C:].reshape(H, V)
    assert all(np.corrcoef(S[h, i], wrote[h])[0, 1] > 0.9 for h in range(H) for i in range(8))


@pytest.mark.parametrize("case", [(torch.float32, 52, 5, 3, 100, 30), (torch.bfloat16, 52, 5, 3, 100, 30), (torch.bfloat16, 300, 8, 3, 128, 64),
                                  (torch.float32, 40, 2, 1, 24, 8), (torch.bfloat16, 9, 16, 4, 64, 32), (torch.bfloat16, 1200, 4, 2, 64, 32),
                                  (torch.bfloat16, 1200, 2, 2, 2048, 512)])
def test_sigmoid_scores_with_and_without_a_correction_and_weighted_inputs(case):
    """Scores by the sigmoid of every output alone, the choice by the score (or by score + correction, made so that it differs),
    weights the scores as they are; the experts' products with the weight on the input, against the plain functions."""
    from gibbs_amd.ops.lib import call, dtype_code, library, ptr, stream
    dtype, n, E, top, W, F = case
    rng = np.random.default_rng(3)
    h = _dev(rng.normal(size=(n, W)), dtype)
    router = _dev(rng.normal(size=(E, W)) * 0.3)
    corr = rng.normal(size=E) * 0.7
    corr[-1] += 1.0                                               # (the last output is chosen often by its correction alone)
    corr = _dev(corr)
    hh, r64, c64 = _f64(h), _f64(router), _f64(corr)
    s = Z.sigmoid(hh @ r64.T)
    chosen, weight = torch.empty((n, top), dtype=torch.int32, device="cuda"), torch.empty((n, top), dtype=torch.float32, device="cuda")
    for c in (corr, None):
        call("gibbs_moe_route_mode", ptr(h), W, dtype_code(dtype), ptr(router), ptr(c), None, ptr(chosen), ptr(weight), None, n, W, E, top, 2, stream())
        rank = s + (c64[None] if c is not None else 0.0)
        want_c = np.argsort(-rank, axis=-1, kind="stable")[:, :top]
        ordered = np.sort(rank, -1)[:, ::-1]
        gaps = (ordered[:, :-1] - ordered[:, 1:]).min(-1) if E > 1 else np.ones(n)
        sure = gaps > 1e-5
        got_c, got_w = chosen.cpu().numpy(), weight.cpu().numpy()
        assert sure.sum() >= 0.5 * n and np.array_equal(got_c[sure], want_c[sure])
        assert np.abs(got_w - np.take_along_axis(s, got_c.astype(np.int64), -1)).max() <= 2e-5
        if c is None and top < E:
            assert (want_c != np.argsort(-(s + c64[None]), axis=-1, kind="stable")[:, :top]).any()
    gate, up, down = _dev(rng.normal(size=(E, F, W)) * 0.1, dtype), _dev(rng.normal(size=(E, F, W)) * 0.1, dtype), _dev(rng.normal(size=(E, W, F)) * 0.1, dtype)
    lib = library()
    pairs = n * top
    bm = lib.gibbs_moe_tile(pairs, E)
    cap = lib.gibbs_moe_capacity(pairs, E, bm)
    sorted_pair, tile_expert = torch.empty(cap, dtype=torch.int32, device="cuda"), torch.empty(cap // bm, dtype=torch.int32, device="cuda")
    place = torch.empty(pairs, dtype=torch.int32, device="cuda")
    call("gibbs_moe_group", ptr(chosen), pairs, E, bm, ptr(sorted_pair), ptr(place), ptr(tile_expert), cap, stream())
    mid, y = torch.zeros((cap, F), dtype=dtype, device="cuda"), torch.zeros((cap, W), dtype=dtype, device="cuda")
    call("gibbs_moe_gemm_weighted", ptr(h), W, top, ptr(sorted_pair), ptr(tile_expert), cap, bm, ptr(gate), ptr(up), ptr(weight), ptr(mid), F, dtype_code(dtype), F, W, 0, stream())
    call("gibbs_moe_gemm", ptr(mid), F, 0, ptr(sorted_pair), ptr(tile_expert), cap, bm, ptr(down), None, ptr(y), W, dtype_code(dtype), W, F, 0, stream())
    out = torch.empty((n, W), dtype=dtype, device="cuda")
    call("gibbs_moe_combine", ptr(y), ptr(place), None, None, None, ptr(out), dtype_code(dtype), n, top, W, stream())
    g64, u64, d64 = _f64(gate), _f64(up), _f64(down)
    want = np.zeros((n, W))
    for e in range(E):
        for c in range(top):
            at = np.nonzero(got_c[:, c] == e)[0]
            if at.size:
                want[at] += Z.expert(got_w[at, c:c + 1].astype(np.float64) * hh[at], g64[e], u64[e], d64[e])
    tol = 3e-5 if dtype == torch.float32 else 3e-2
    assert np.abs(_f64(out) - want).max() <= tol * np.abs(want).max()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_whole_in_portions_and_decoded(dtype, tmp_path):
    """A prompt over many chunks of the recurrence and several of the attention (600 tokens in one step), the same prompt in
    portions, and its last tokens one by one: all against the plain logits."""
    cfg = GH.model(150, 64, [GH.with_mlp(GH.recurrence(4, 16, 24), None), GH.with_mlp(GH.differential(4, 2, 8, 16, 0.35, 0.4, size=150, rot=(1e4, 8)), GH.moe(2, 2, 32)),
                             GH.with_mlp(GH.latent(3, 16, 16, 32, 24, 0.3), None), GH.with_mlp(GH.recurrence(2, 96, 48), GH.moe(1, 1, 48)),
                             GH.with_mlp(GH.latent(2, 8, 24, 32, 16, 0.4, kv_from=2), None)])
    d = GH.make_model_dir(str(tmp_path), cfg, "long", seed=12)
    ids = GH.tokens(8, 600, 150)
    want = [0, 63, 64, 149, 150, 255, 256, 300, 511, 512, 598, 599]
    whole = run_steps(make_engine(d, dtype), [([("r", ids, want)], ["r"])])
    check(d, {"r": ids}, whole, dtype, f"long prompt whole {dtype}")
    cuts = portions(560, [200, 90, 255, 15]) + [(560 + i, 561 + i) for i in range(40)]
    cut = run_steps(make_engine(d, dtype), [([("r", ids[a:b], [p - a for p in want if a <= p < b])], []) for a, b in cuts])
    check(d, {"r": ids}, cut, dtype, f"long prompt in portions {dtype}")
    assert sorted(cut) == sorted(whole)


def test_a_key_far_back_through_a_shared_latent(tmp_path):
    """Two latent layers over one cache; the second's scores are made sharp (a scale far above 1 / sqrt(dim)), so that its rows are
    dominated by single keys anywhere in the sequence: 32-bit, a prompt of 300 in one step, in portions and decoded."""
    cfg = GH.model(131, 40, [GH.with_mlp(GH.latent(2, 8, 8, 12, 10, 0.3), None), GH.with_mlp(GH.latent(3, 8, 10, 12, 14, 9.0, kv_from=0), None)])
    d = GH.make_model_dir(str(tmp_path), cfg, "far", seed=3)
    c, w = GH.load_model_dir(d)
    ids = GH.tokens(3, 300, 131)
    x = Z.rms_unit(w["embed"][ids], 1e-5) * w["embed.norm"]
    lat = Z.latent(Z.token_shift(x, w["l0.shift"]), w, "l0.mix.", 1e-5)
    x = x + Z.rms_unit(Z.latent_attention_mixer(Z.token_shift(x, w["l0.shift"]), lat, w, "l0.mix.", c["layers"][0]["mixer"], 1e-5), 1e-5) * w["l0.norm1"] * w["l0.ls1"]
    h = Z.token_shift(x, w["l1.shift"])
    q = ((Z.rms_unit(h @ w["l1.mix.dq"].T, 1e-5) * w["l1.mix.dq.norm"]) @ w["l1.mix.uq"].T).reshape(300, 3, 8)
    s = np.einsum("thd,shd->ths", q, (lat @ w["l1.mix.uk"].T).reshape(300, 3, 8))[-30:] * 9.0
    far = s.argmax(-1)
    assert (np.sort(s, -1)[..., -1] - np.sort(s, -1)[..., -20] > 3.0).mean() > 0.5 and (far < 200).mean() > 0.4, "keys far back must stand out"
    for cuts in ([(0, 300)], portions(280, [33, 2, 64, 90, 17, 74]) + [(280 + i, 281 + i) for i in range(20)]):
        got = run_steps(make_engine(d, "float32"), [([("r", ids[a:b], list(range(b - a)))], []) for a, b in cuts])
        check(d, {"r": ids}, got, "float32", "keys far back")


def test_captured_steps_repeat_and_agree_with_eager_ones(dirs):
    """A captured decode step (graphs of one and of several steps, replayed over and over with eager work between) gives what
    the same steps give without a graph, for requests of different lengths."""
    from gibbs_amd.engine.decode import DecodeLoop
    d = dirs["B"]
    prompts = [GH.tokens(80 + i, n, vocab_of(d)) for i, n in enumerate([9, 38, 25])]
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
        ids.append(int(np.argmax(GH.plain_logits(model_dir, ids)[-1])))
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
        prompts = [GH.tokens(40 + i, n, vocab_of(d)) for i, n in enumerate(lens)]
        outs = generate(eng, prompts, max_tokens=20, temperature=0.0, ignore_eos=True)
        for p, o in zip(prompts, outs):
            assert o.finish_reason == "length" and len(o.tokens) == 20
            if dtype == "float32":
                assert o.tokens == plain_greedy(d, p, 20)
                held += 20
                continue
            logits = GH.plain_logits(d, list(p) + list(o.tokens))
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
    prompts = [GH.tokens(70 + i, n, vocab_of(d)) for i, n in enumerate([9, 21, 5])]
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
    want_a, want_b = GH.plain_logits(d, ids), GH.plain_logits(d, other)
    read = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, vocab_of(d))
    close(read(0), want_a[[0, 16]], dtype, "step 0")
    close(read(1), want_b[[8]], dtype, "step 1")
    close(read(2), want_a[[38]], dtype, "step 2")
    close(read(3), want_a[[39]], dtype, "step 3")


def test_command_line(dirs):
    d = dirs["A"]
    prompt = GH.tokens(60, 6, vocab_of(d))
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "gibbs"), "--model", d, "--dtype", "float32", "--prompt-ids",
                           ",".join(map(str, prompt)), "--max-tokens", "8", "--temperature", "0", "--ignore-eos"],
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    line = proc.stdout.split("✨ Output:\n")[1].splitlines()[0]
    assert [int(t) for t in line.split()] == plain_greedy(d, prompt, 8)
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "gibbs"), "--model", d, "--arch-dump"], capture_output=True, text=True, timeout=600)
    dump = json.loads(proc.stdout)
    assert dump["architecture"] == "Gumozen" and dump["unconsumed"] == [] and dump["missing"] == []
    assert dump["derived"]["layers_by_type"] == {"attention": 2, "hgrn2": 1, "latent_attention": 3}
