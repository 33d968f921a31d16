"""The Sagopel parts on the GPU against the plain implementation (tests/plain/sagopel_plain.py): every kernel alone, then
small random models in every way of cutting requests into steps, in 32-bit and in bfloat16, then generation through the
scheduler, the command line and the trace tool.  The configurations differ from each other in every size, and hold
values that a model may happen to make equal or 1 (one head, kv heads = heads, value size = key size, a rotation of the
whole head, a decay of 1, a window of one key, nothing kept, no identities, one expert, every choice taken, a loop of one
pass, no loop, no feed-forward)."""
import json
import os

import numpy as np
import pytest
import torch

from helpers import last_one_by_one, make_requests, max_difference, mixed, plain_logits, portions, run_steps, whole
from plain import sagopel_plain as P

pytestmark = pytest.mark.gpu

DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def lightning(heads, dim, vdim, decay):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=[decay[i % len(decay)] for i in range(heads)]))


def window(heads, kv, dim, vdim, rot, size, keep, cap=20.0, scale=None, base=10000.0):
    return dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, rot=dict(dims=rot, base=base), scale=scale or 2.0 * dim ** -0.5, softcap=cap,
                mask=dict(size=size, keep_first=keep))


def retention(heads, dim, vdim, rot, decay, base=10000.0):
    return dict(lightning(heads, dim, vdim, decay)["mixer"], rot=dict(dims=rot, base=base))


def parallel(left, right):
    return dict(type="parallel", mixer=dict(left=left, right=right))


def dense(layer, ff):
    return dict(layer, mlp=None if ff is None else dict(kind="dense", ff=ff))


def moe(layer, ff, experts, identity, top, shared):
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, identity=identity, top=top),
                                **({} if shared is None else dict(shared=dict(ff=shared)))))


def model(vocab, width, layers, eps=1e-5, mult=0.4, loop=None):
    return dict(architecture="Sagopel", vocab=vocab, width=width, norm=dict(eps=eps), residual_mult=mult, layers=layers,
                **({} if loop is None else dict(loop=dict(start=loop[0], stop=loop[1], times=loop[2]))))


CONFIGS = {
    # both mixers, every feed-forward, a loop over the middle
    "loop": model(203, 96, [dense(lightning(3, 16, 48, [0.6, 0.98]), 80),
                            moe(parallel(window(6, 2, 32, 16, 16, 29, 5), retention(2, 24, 40, 16, [0.9, 0.995])), 48, 6, 2, 3, 40),
                            moe(lightning(5, 24, 16, [0.8, 1.0, 0.97]), 32, 4, 3, 2, 64), dense(lightning(2, 64, 64, [0.99]), None)],
                  loop=(1, 3, 2)),
    # sizes the matrix cores do not take, a window of one key, nothing kept, no identities, one expert, all chosen
    "odd": model(97, 72, [moe(parallel(window(3, 3, 20, 36, 10, 1, 0, cap=7.0), retention(1, 12, 12, 12, [0.7], base=50.0)), 20, 3, 2, 5, 12),
                          dense(lightning(1, 10, 6, [1.0]), 50), moe(lightning(4, 6, 30, [0.5, 0.95]), 24, 1, 0, 1, 30),
                          dense(parallel(window(5, 1, 6, 10, 2, 12, 17, base=30.0), retention(6, 2, 4, 2, [0.85, 0.999])), None)],
                 eps=3e-6, mult=1.0, loop=(0, 4, 1)),
    # no loop; heads = kv heads, value size = key size, a window longer than most requests, more kept than a page
    "plain_order": model(160, 128, [dense(parallel(window(4, 4, 64, 64, 64, 61, 33, cap=50.0), retention(4, 64, 64, 64, [0.97, 0.9921875])), 96),
                                    moe(lightning(2, 128, 128, [0.9, 0.999]), 64, 8, 8, 4, 64),
                                    moe(parallel(window(8, 2, 128, 80, 32, 40, 1), retention(3, 128, 96, 64, [0.95, 0.99])), 16, 12, 1, 2, None)],
                         mult=0.25),
    # the first layer loops alone, each pass of a mixture
    "first": model(64, 64, [moe(parallel(window(8, 1, 16, 32, 8, 18, 9), retention(3, 16, 16, 8, [0.9, 0.99])), 32, 5, 1, 2, 16),
                            dense(lightning(4, 32, 16, [0.96]), 32)], mult=0.7, loop=(0, 1, 3)),
}
LENGTHS = [70, 33, 150, 17, 64, 129, 2, 45]
LEAST = 6.0                   # of a token's margins (see `route_margin`, `retention_margin`)
_cache = {}


def write_model(folder, cfg, seed, matrix_std=0.12):
    """A random model whose routers' corrections are a few times as large as usual: fewer tokens' choices are close calls."""
    from safetensors.torch import load_file, save_file

    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.weights import write_random_model
    write_random_model(folder, config_from_dict(cfg), seed=seed, matrix_std=matrix_std, norm_std=0.2)
    path = os.path.join(folder, "model.safetensors")
    save_file({n: (t * 4.0).contiguous() if n.endswith(".correction") else t for n, t in load_file(path).items()}, path)
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    out = {}
    for i, (name, cfg) in enumerate(CONFIGS.items()):
        out[name] = write_model(str(tmp_path_factory.mktemp(f"sagopel_{name}")), cfg, seed=370 + i)
    return out


def decisive_requests(oracle, vocab, lengths, seed):
    """Random requests in which no token is a close call (its choice of experts, a head of retention that cancels): an
    engine that rounds takes what the plain model takes, and rows can be compared."""
    rng = np.random.default_rng(3000 + seed)
    return {rid: oracle.decisive(toks, rng, LEAST) for rid, toks in make_requests(vocab, lengths, seed).items()}


def plain(folders, name):
    if ("plain", name) not in _cache:
        oracle = P.PlainSagopel(folders[name])
        reqs = decisive_requests(oracle, CONFIGS[name]["vocab"], LENGTHS, seed=9)
        _cache[("plain", name)] = (oracle, reqs, plain_logits(oracle, reqs))
    return _cache[("plain", name)]


def load(folders, name, dtype_name):
    from mini_llm_runtime_amd.parts import DecoderModel
    if (name, dtype_name) not in _cache:
        _cache[(name, dtype_name)] = DecoderModel.load(folders[name], DTYPES[dtype_name])
    return _cache[(name, dtype_name)]


def runner_for(loaded, max_tokens, **kwargs):
    from mini_llm_runtime_amd.engine import Runner
    kwargs.setdefault("max_length", 512)
    kwargs.setdefault("page_size", 8)
    return Runner(loaded, max_tokens=max_tokens, max_slots=4, **kwargs)


def close(got, want, dtype_name, scale, outliers=None, band=3.0):
    """Rows against float64: the float engine to rounding at every row; the bfloat16 engine to 4 % of the largest logit
    at the worst place and 1.2 % in the root mean square, where one row in fifty may reach `band` times that."""
    assert set(got) == set(want)
    over = []
    for key in sorted(want):
        err = np.abs(got[key] - want[key])
        assert np.isfinite(got[key]).all(), key
        if dtype_name == "float32":
            assert err.max() <= 3e-4 * scale, (key, err.max(), scale)
        elif not (err.max() <= 0.04 * scale and np.sqrt((err ** 2).mean()) <= 0.012 * scale):
            assert err.max() <= band * 0.04 * scale and np.sqrt((err ** 2).mean()) <= band * 0.012 * scale, (key, err.max(), scale)
            over.append(key)
    assert len(over) <= (max(1, len(want) // 50) if outliers is None else outliers), over


def idle(r):
    r.cache.check()
    assert r.free_slots() == 4
    for g in range(len(r.cache.group_pages)):
        assert r.cache.free_pages(g) == r.cache.group_pages[g]


def rounded(x, dtype):
    return torch.from_numpy(np.ascontiguousarray(x)).to(dtype).cuda()


def back(t):
    return t.double().cpu().numpy()


def ints(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def tolerance(dtype_name):
    # (a score near a cap of 30 carries 32-bit rounding of a few 1e-6, and so does its exponential)
    return dict(rtol=6e-5, atol=6e-5) if dtype_name == "float32" else dict(rtol=3e-2, atol=2e-2)


def rope_table(dims, base, positions):
    from mini_llm_runtime_amd.config.specs import PositionSpec
    from mini_llm_runtime_amd.parts.rope import Rope
    return Rope(PositionSpec("rope", dims, base)).rotation(positions, "cuda").table


# ---- the kernels alone --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("rows,width", [(5, 24), (3, 37), (70, 128), (2, 1), (9, 4100), (2, 9000), (130, 2050)])
def test_a_delta_with_a_factor_and_a_vector_ride_in_the_norms_pass(dtype_name, rows, width):
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(width)
    h64 = back(rounded(rng.normal(size=(rows, width)), torch.float32))
    delta = rounded(rng.normal(size=(rows, width)), dtype)
    vec, w = (rounded(rng.normal(size=width), torch.float32) for _ in range(2))
    tol = dict(rtol=1e-4, atol=1e-4) if dtype_name == "float32" else dict(rtol=1e-2, atol=1e-2)
    for d, v, factor in ((delta, vec, 0.3), (delta, None, -1.7), (None, vec, 0.3), (delta, vec, 1.0)):
        total = h64 + (factor * back(d) if d is not None else 0.0) + (back(v) if v is not None else 0.0)
        h = rounded(h64, torch.float32)
        out = torch.full((rows, width), float("nan"), dtype=dtype, device="cuda")
        k.add_rmsnorm(h, d, w, out, 1e-3, factor=factor, vector=v)
        np.testing.assert_allclose(back(h), total, rtol=1e-5, atol=1e-5)
        np.testing.assert_allclose(back(out), P.rms_norm(total, back(w), 1e-3), **tol)
        h = rounded(h64, torch.float32)
        pick = ints([rows - 1, 0])
        out = torch.full((2, width), float("nan"), dtype=dtype, device="cuda")
        k.add_rmsnorm(h, d, w, out, 1e-3, rows=pick, write_h=False, factor=factor, vector=v)
        assert np.array_equal(back(h), h64)
        np.testing.assert_allclose(back(out), P.rms_norm(total, back(w), 1e-3)[[rows - 1, 0]], **tol)
        k.residual_add(h, d, factor, v)
        np.testing.assert_allclose(back(h), total, rtol=1e-5, atol=1e-5)
    big = rounded(np.full((rows, width), 1e30), torch.float32)         # (squares beyond 32 bits: the row is rescaled)
    out = torch.empty((rows, width), dtype=dtype, device="cuda")
    k.add_rmsnorm(big, delta, w, out, 1e-3, factor=0.5, vector=vec)
    np.testing.assert_allclose(back(out), np.tile(back(w), (rows, 1)), **tol)


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("rows,width", [(5, 24), (3, 37), (70, 128), (2, 1), (9, 4104), (3, 9000), (2, 8195)])
def test_two_rows_are_normed_apart_and_added(dtype_name, rows, width):
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(width)
    a, b = rounded(rng.normal(size=(rows, width)) * 30.0, dtype), rounded(rng.normal(size=(rows, width)) * 0.01, dtype)
    wa, wb = (rounded(1.0 + rng.normal(size=width), torch.float32) for _ in range(2))
    na, nb = P.rms_norm(back(a), back(wa), 1e-4), P.rms_norm(back(b), back(wb), 1e-4)
    tol = dict(rtol=1e-4, atol=1e-4) if dtype_name == "float32" else dict(rtol=1e-2, atol=1e-2)
    out = torch.full((rows, width), float("nan"), dtype=dtype, device="cuda")
    k.normed_sum(a, b, wa, wb, out, 0.5, 0.25, 1e-4)
    np.testing.assert_allclose(back(out), 0.5 * na + 0.25 * nb, **tol)
    fresh = rounded(rng.normal(size=(rows, width)), dtype)             # (a third mixer joins a sum, in place)
    want = back(fresh) + 3.0 * nb
    k.normed_sum(fresh, b, None, wb, fresh, 1.0, 3.0, 1e-4)
    np.testing.assert_allclose(back(fresh), want, **tol)


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("rows,hidden,inter", [(1, 64, 48), (7, 128, 6200), (20, 40, 100), (64, 64, 20), (90, 2048, 24)])
def test_the_relu_gate(dtype_name, rows, hidden, inter):
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(hidden)
    x, w = rounded(rng.normal(size=(rows, hidden)), dtype), rounded(rng.normal(size=(2 * inter, hidden)) * 1.5 * hidden ** -0.5, dtype)
    both = rounded(back(x) @ back(w).T, dtype)
    out = torch.full((rows, inter), float("nan"), dtype=dtype, device="cuda")
    k.gated_act_mul(both, out, "relu")
    want = P.relu(back(both)[:, :inter]) * back(both)[:, inter:]
    np.testing.assert_allclose(back(out), want, **(dict(rtol=1e-6, atol=1e-6) if dtype_name == "float32" else dict(rtol=1e-2, atol=1e-3)))
    assert (back(out)[want == 0.0] == 0.0).all() and (want == 0.0).any()
    if dtype_name == "bfloat16" and rows <= 64:
        exact = back(x) @ back(w).T
        out.fill_(float("nan"))
        k.gemm_gated_act(x, w, out, "relu")
        np.testing.assert_allclose(back(out), P.relu(exact[:, :inter]) * exact[:, inter:], rtol=2e-2, atol=5e-3)


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("heads,values", [(3, 20), (2, 64), (1, 8), (6, 32), (5, 24), (3, 136), (2, 1024), (1, 1032), (1, 4096), (1, 9000), (2, 512)])
def test_heads_over_their_own_root_mean_square_without_a_weight(dtype_name, heads, values):
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(values)
    o = rounded(rng.normal(size=(9, heads * values)) * np.exp(rng.normal(size=(9, heads * values)) * 3), torch.float32)
    wide = rounded(rng.normal(size=(9, heads * values + 16)), dtype)
    out = torch.full((9, heads * values), float("nan"), dtype=dtype, device="cuda")
    k.gated_part_norm(o, wide[:, 16:], None, out, values, 1e-3, gate_first=False, gate_kind="silu")
    want = P.over_rms(back(o).reshape(9, heads, values), 1e-3).reshape(9, -1) * P.silu(back(wide)[:, 16:])
    np.testing.assert_allclose(back(out), want, **(dict(rtol=1e-4, atol=1e-5) if dtype_name == "float32" else dict(rtol=1e-2, atol=1e-2)))


def continued(q, kk, v, decay, S):
    """One head from the state S [D, V]: (outputs [T, V], the state after)."""
    S, out = S.copy(), np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        S = decay * S + np.outer(kk[t], v[t])
        out[t] = S.T @ q[t]
    return out, S


RECURRENCES = [(3, 24, 40, 16), (1, 2, 1, 2), (2, 128, 128, 128), (4, 64, 32, 0), (2, 33, 70, 32), (1, 256, 24, 64), (5, 8, 8, 0), (3, 96, 136, 64)]


def recurrence_case(k, dtype, heads, keys, values, rot, silu, lengths, seed, far=900):
    """Random rows of several requests at positions that start far from 0, from states that are not zero: the device
    arguments and, per request, the plain outputs and end states."""
    rng = np.random.default_rng(seed)
    n = sum(lengths)
    slot_of = [int(s) for s in rng.permutation(len(lengths) + 1)[:len(lengths)]]
    starts = [int(p) for p in rng.integers(0, far, len(lengths))]
    proj = rounded(rng.normal(size=(n, heads * (2 * keys + values) + 5)), dtype)
    decay = [[0.5, 0.9, 1.0, 0.9995, 0.03][h % 5] for h in range(heads)]
    a, b, c = heads * keys, 2 * heads * keys, 2 * heads * keys + heads * values
    base = 300.0
    state = heads * keys * values
    live = rounded(rng.normal(size=(len(lengths) + 1, state)), torch.float32)
    positions = np.concatenate([np.arange(s, s + m) for s, m in zip(starts, lengths)])
    slots = np.concatenate([[s] * m for s, m in zip(slot_of, lengths)])
    x = back(proj)
    act = P.silu if silu else (lambda z: z)
    q, kk, v = act(x[:, :a]).reshape(n, heads, keys), act(x[:, a:b]).reshape(n, heads, keys), act(x[:, b:c]).reshape(n, heads, values)
    if rot:
        q, kk = P.rotate(q, positions, rot, base), P.rotate(kk, positions, rot, base)
    want, ends, at = np.zeros((n, heads, values)), back(live).copy(), 0
    for s, m in zip(slot_of, lengths):
        for h in range(heads):
            S = ends[s, h * keys * values:(h + 1) * keys * values].reshape(keys, values)
            want[at:at + m, h], end = continued(q[at:at + m, h] * 0.3, kk[at:at + m, h], v[at:at + m, h], decay[h], S)
            ends[s, h * keys * values:(h + 1) * keys * values] = end.reshape(-1)
        at += m
    log_decay = torch.tensor([float(np.log(d)) for d in decay], dtype=torch.float32, device="cuda")
    more = dict(q_scale=0.3, activation="silu" if silu else None)
    if rot:
        more.update(rope=rope_table(rot, base, far + max(lengths) + 1), positions=ints(positions.tolist()))
    first = [sum(lengths[:i]) for i in range(len(lengths))]
    return dict(args=(proj[:, :a], proj[:, a:b], proj[:, b:c], log_decay), live=live, slots=ints(slots.tolist()), first=first, count=list(lengths),
                more=more, want=want.reshape(n, -1), ends=ends, slot_of=slot_of, n=n)


def check_recurrence(case, out, stage, tol):
    np.testing.assert_allclose(back(out), case["want"], atol=tol * np.abs(case["want"]).max(), rtol=tol)
    for s in range(case["ends"].shape[0]):
        if s in case["slot_of"]:
            np.testing.assert_allclose(back(stage[s]), case["ends"][s], atol=tol * np.abs(case["ends"][s]).max(), rtol=tol)
        else:
            assert torch.isnan(stage[s]).all()                         # (no other slot is touched)


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("silu", [False, True])
@pytest.mark.parametrize("heads,keys,values,rot", RECURRENCES)
def test_the_recurrence_turns_its_queries_and_keys(dtype_name, silu, heads, keys, values, rot):
    """Token by token and in pieces side by side."""
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    case = recurrence_case(k, dtype, heads, keys, values, rot, silu, [37, 1, 150, 2], seed=keys + values)
    for piece in (None, 64):
        out = torch.full((case["n"], heads * values), float("nan"), device="cuda")
        stage = torch.full_like(case["live"], float("nan"))
        first, count, more = case["first"], case["count"], dict(case["more"])
        if piece is not None:
            cut = [(f + i, min(piece, c - i)) for f, c in zip(first, count) for i in range(0, c, piece)]
            first, count = [f for f, _ in cut], [c for _, c in cut]
            nan = lambda m: torch.full((m,), float("nan"), device="cuda")
            more.update(piece_state=nan(len(cut) * heads * keys * values), piece_decay=nan(len(cut) * heads * keys))
        k.linear_recurrence(*case["args"], out, case["live"], stage, 0, ints(first), ints(count), len(first), case["slots"], heads, keys,
                            values, **more)
        check_recurrence(case, out, stage, 6e-5)


@pytest.mark.parametrize("silu", [False, True])
@pytest.mark.parametrize("heads,keys,values,rot", [(3, 24, 48, 16), (2, 128, 128, 128), (4, 64, 32, 0), (1, 8, 16, 0), (5, 96, 144, 64), (2, 40, 272, 32),
                                                   (6, 48, 80, 48), (1, 112, 64, 112), (2, 16, 16, 16)])
def test_the_recurrence_in_chunks_on_the_matrix_cores(silu, heads, keys, values, rot):
    """Requests shorter and longer than a chunk, ends around blocks of 64 rows, single tokens between them, from states that
    are not zero; decays from none at all to 0.03 a token.  What differs from 32-bit arithmetic is rounding, not bfloat16."""
    from mini_llm_runtime_amd.kernels import Kernels
    k = Kernels(torch.bfloat16)
    for chunk, lengths in ((128, [37, 1, 128, 300, 64, 2, 129, 65]), (64, [200, 63, 1]), (192, [1, 500, 192])):
        case = recurrence_case(k, torch.bfloat16, heads, keys, values, rot, silu, lengths, seed=keys + values + chunk)
        args = case["args"]
        if args[0].stride(0) % 8:                                      # (rows that start at multiples of 16 bytes)
            wide = torch.zeros((case["n"], -(-args[0].stride(0) // 8) * 8), dtype=torch.bfloat16, device="cuda")
            a, b, c = heads * keys, 2 * heads * keys, 2 * heads * keys + heads * values
            for lo, hi, t in ((0, a, args[0]), (a, b, args[1]), (b, c, args[2])):
                wide[:, lo:hi] = t
            args = (wide[:, :a], wide[:, a:b], wide[:, b:c], args[3])
        cut = [(f + i, min(chunk, n - i)) for f, n in zip(case["first"], case["count"]) for i in range(0, n, chunk)]
        out = torch.full((case["n"], heads * values), float("nan"), device="cuda")
        stage = torch.full_like(case["live"], float("nan"))
        scratch = torch.full((len(cut) * heads * keys * values,), float("nan"), device="cuda")
        k.decayed_recurrence_chunks(*args, out, case["live"], stage, 0, ints(case["first"]), ints(case["count"]), len(lengths), case["slots"],
                                    ints([f for f, _ in cut]), ints([n for _, n in cut]), len(cut), chunk, scratch, heads, keys, values,
                                    **case["more"])
        check_recurrence(case, out, stage, 6e-5 if rot else 1e-5)      # (an angle near 1000 carries 32-bit rounding of 6e-5)


def paged(x, page, dtype, seed=0):
    """[T, G, D] of ONE request in row-major pages that lie in a shuffled order, NaN where nothing was written; (pages, block
    table [1, blocks])."""
    T, G, D = x.shape
    blocks = -(-T // page)
    order = np.random.default_rng(seed).permutation(blocks + 3)[:blocks]
    pages = np.full((blocks + 3, G, page, D), np.nan)
    for t in range(T):
        pages[order[t // page], :, t % page] = x[t]
    return rounded(pages, dtype), ints(order[None].tolist())


WINDOW_SHAPES = [(4, 2, 32, 16, 8), (6, 2, 64, 128, 16), (3, 1, 20, 70, 4), (8, 8, 128, 64, 24), (5, 1, 40, 48, 8), (1, 1, 256, 256, 32)]


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("size,keep", [(37, 5), (1, 1), (64, 64), (150, 33), (20, 100), (3, 0), (90, 31)])
@pytest.mark.parametrize("heads,kv,dim,vdim,page", WINDOW_SHAPES)
def test_a_window_that_keeps_the_first_tokens_finds_one_key_wherever_it_lies(dtype_name, size, keep, heads, kv, dim, vdim, page):
    """For one query one key among 300 is made to stand out (scores near the cap): at the first tokens, at the border of
    what is kept, at page and tile borders, just inside and outside the window.  The scalar kernel, and where it takes the
    sizes the matrix-core kernel, for queries that are groups of their own (whole and in key ranges); pages that lie wholly
    between the kept tokens and every query's window hold NaN."""
    from mini_llm_runtime_amd.kernels import Kernels
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(5)
    T, cap = 300, 30.0
    keys, values = back(rounded(rng.normal(size=(T, kv, dim)) * 0.3, dtype)), back(rounded(rng.normal(size=(T, kv, vdim)), dtype))
    pairs = sorted({(qp, kp) for qp in (0, 1, 5, page - 1, page, 31, 32, 63, 64, 65, 127, 128, 200, 299)
                    for kp in (0, 1, keep - 1, keep, keep + 1, qp, qp - size + 1, qp - size, qp - size - 1, qp - page, qp - 64, page, 31, 32)
                    if 0 <= kp <= qp})
    q = np.zeros((len(pairs), heads, dim))
    for i, (qp, kp) in enumerate(pairs):
        for h in range(heads):
            key = keys[kp, h // (heads // kv)]
            q[i, h] = key * (60.0 / max(1e-6, float(np.sum(key ** 2))))
    q = back(rounded(q, dtype))
    positions = [p for p, _ in pairs]
    seen = P.seen_in_window(positions, np.arange(T), size, keep)
    want = P.attend(q, keys, values, 0.8, cap, seen)
    asked = [bool(seen[i, kp]) for i, (_, kp) in enumerate(pairs)]
    assert any(asked) and not all(asked)
    m = len(pairs)
    k_pages, table = paged(keys, page, dtype, seed=1)
    v_pages, _ = paged(values, page, dtype, seed=1)
    zeros, pos = ints([0] * m), ints(positions)
    out = torch.full((m, heads * vdim), float("nan"), dtype=dtype, device="cuda")
    k.sink_attention(rounded(q.reshape(m, -1), dtype), k_pages, v_pages, table, zeros, pos, None, out, heads, kv, dim, vdim, page, 0.8,
                     "window", size, keep_first=keep, softcap=cap)
    np.testing.assert_allclose(back(out), want, **tolerance(dtype_name))
    taken = k.sink_tiles_supported(dim, vdim, dim, vdim, page, "window", size, T, keep)
    assert taken == (dtype_name == "bfloat16" and dim % 8 == 0 and vdim % 16 == 0)
    if taken:
        first, count = ints(list(range(m))), ints([1] * m)
        big_heads, _, small_heads, small_tokens = k.sink_tiles_layout(heads, kv)
        for head_block, split, ranges in ((small_heads, True, 0), (big_heads, False, 0), (small_heads, True, 64), (small_heads, True, 32)):
            more = {}
            if ranges:
                splits = -(-(T + 31) // ranges)
                more = dict(partial=torch.full((k.sink_partial_numel(m, small_tokens, heads, vdim, splits),), float("nan"), device="cuda"),
                            split_keys=ranges, splits=splits)
            out.fill_(float("nan"))
            k.sink_attention_tiles(rounded(q.reshape(m, -1), dtype), k_pages, v_pages, table, zeros, pos, None, out, first, count, m,
                                   head_block, split, heads, kv, dim, vdim, page, 0.8, "window", size, T, keep_first=keep, softcap=cap, **more)
            np.testing.assert_allclose(back(out), want, err_msg=str((head_block, split, ranges)), **tolerance(dtype_name))
    # ONE query at the end: what lies between the kept tokens and its window is given back (no page, NaN in the memory)
    table_gone, first_needed = table.clone(), max(0, T - size)
    for blk in range(-(-keep // page), first_needed // page):
        k_pages[table[0, blk]] = float("nan")
        v_pages[table[0, blk]] = float("nan")
        table_gone[0, blk] = -1
    lone = rounded(q[-1:].reshape(1, -1), dtype)
    out = torch.full((1, heads * vdim), float("nan"), dtype=dtype, device="cuda")
    k.sink_attention(lone, k_pages, v_pages, table_gone, ints([0]), ints([T - 1]), None, out, heads, kv, dim, vdim, page, 0.8, "window", size,
                     keep_first=keep, softcap=cap)
    np.testing.assert_allclose(back(out), want[-1:], **tolerance(dtype_name))
    if taken:
        for ranges in (0, 32):
            splits = -(-(T + 31) // 32)
            more = dict(partial=torch.full((k.sink_partial_numel(1, small_tokens, heads, vdim, splits),), float("nan"), device="cuda"),
                        split_keys=32, splits=splits) if ranges else {}
            out.fill_(float("nan"))
            k.sink_attention_tiles(lone, k_pages, v_pages, table_gone, ints([0]), ints([T - 1]), None, out, ints([0]), ints([1]), 1, small_heads,
                                   True, heads, kv, dim, vdim, page, 0.8, "window", size, T, keep_first=keep, softcap=cap, **more)
            np.testing.assert_allclose(back(out), want[-1:], err_msg=str(ranges), **tolerance(dtype_name))


@pytest.mark.parametrize("size,keep,cap", [(37, 5, 3.0), (1, 1, None), (64, 64, 50.0), (150, 33, None), (20, 100, 8.0)])
@pytest.mark.parametrize("heads,kv,dim,vdim,page", [s for s in WINDOW_SHAPES if s[4] != 4])
def test_groups_of_tokens_under_such_a_window(size, keep, cap, heads, kv, dim, vdim, page):
    """Every position of a request of 210 tokens at once, in groups as the engine makes them for portions and for short
    pieces; bfloat16 on the matrix cores, and the scalar kernel in both engines."""
    from mini_llm_runtime_amd.kernels import Kernels
    rng = np.random.default_rng(12)
    T, scale = 210, 0.3
    for dtype_name, dtype in DTYPES.items():
        k = Kernels(dtype)
        keys, values, q = (rounded(rng.normal(size=(T, n, d)), dtype) for n, d in ((kv, dim), (kv, vdim), (heads, dim)))
        seen = P.seen_in_window(np.arange(T), np.arange(T), size, keep)
        want = P.attend(back(q), back(keys), back(values), scale, cap if cap is not None else 1e12, seen)
        k_pages, table = paged(back(keys), page, dtype, seed=3)
        v_pages, _ = paged(back(values), page, dtype, seed=3)
        zeros, pos = ints([0] * T), ints(list(range(T)))
        out = torch.full((T, heads * vdim), float("nan"), dtype=dtype, device="cuda")
        k.sink_attention(q.view(T, -1), k_pages, v_pages, table, zeros, pos, None, out, heads, kv, dim, vdim, page, scale, "window", size,
                         keep_first=keep, softcap=cap)
        np.testing.assert_allclose(back(out), want, **tolerance(dtype_name))
        if dtype_name == "float32":
            continue
        big_heads, big_tokens, small_heads, small_tokens = k.sink_tiles_layout(heads, kv)
        for head_block, tokens, split, ranges in ((big_heads, big_tokens, False, 0), (small_heads, small_tokens, True, 0), (small_heads, small_tokens, True, 96)):
            first = list(range(0, T, tokens))
            count = [min(tokens, T - f) for f in first]
            splits = -(-(T + 31) // ranges) if ranges else 1
            more = dict(partial=torch.full((k.sink_partial_numel(len(first), tokens, heads, vdim, splits),), float("nan"), device="cuda"),
                        split_keys=ranges, splits=splits) if ranges else {}
            out.fill_(float("nan"))
            k.sink_attention_tiles(q.view(T, -1), k_pages, v_pages, table, zeros, pos, None, out, ints(first), ints(count), len(first), head_block,
                                   split, heads, kv, dim, vdim, page, scale, "window", size, T, keep_first=keep, softcap=cap, **more)
            np.testing.assert_allclose(back(out), want, err_msg=str((head_block, split, ranges)), **tolerance(dtype_name))


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("rows,experts,identity,top,hidden,inter,shared", [(5, 3, 1, 2, 40, 16, 24), (300, 4, 4, 3, 64, 48, None), (2100, 2, 1, 2, 128, 160, 33),
                                                                           (33, 5, 0, 5, 24, 20, 8), (40, 1, 6, 3, 32, 32, 16), (64, 60, 40, 8, 48, 32, 32)])
def test_experts_that_give_their_input_back(dtype_name, rows, experts, identity, top, hidden, inter, shared):
    """The part itself against the plain mixture.  Some tokens choose identities only, and none of the experts has to be
    chosen by anyone."""
    from mini_llm_runtime_amd.config.specs import MlpSpec, RoutedMlpSpec
    from mini_llm_runtime_amd.engine.context import StepContext, Workspace
    from mini_llm_runtime_amd.kernels import Kernels
    from mini_llm_runtime_amd.parts import build_part
    dtype = DTYPES[dtype_name]
    k = Kernels(dtype)
    rng = np.random.default_rng(rows)
    cfg = dict(kind="moe", expert=dict(ff=inter), router=dict(experts=experts, identity=identity, top=top),
               **({} if shared is None else dict(shared=dict(ff=shared))))
    spec = RoutedMlpSpec("routed_mlp", hidden, inter, experts, top, 1, 1, "silu", "softmax", False, gated=True, correction=True, identity=identity,
                         shared=None if shared is None else MlpSpec("swiglu", hidden, shared, "silu"))
    part = build_part("ffn", spec)
    weights = {n: rounded(rng.normal(size=ws.shape) * 1.5 * ws.shape[-1] ** -0.5, torch.float32 if ws.keep_float32 else dtype)
               for n, ws in part.weight_specs().items()}
    weights["correction"] = rounded(rng.normal(size=experts + identity) * 0.1, torch.float32)
    x = rng.normal(size=(rows, hidden))
    if identity >= top:
        x[:3] = 4.0 * back(weights["router"])[experts:].mean(axis=0)          # (drawn towards the identities)
        x[:3] -= 4.0 * back(weights["router"])[:experts].mean(axis=0)
    x = rounded(x, dtype)
    w64 = {}
    for n, t in weights.items():
        head, dot, last = n.rpartition(".")
        w64[f"{head}{dot}" + {"gate_proj": "gate", "up_proj": "up", "down_proj": "down"}.get(last, last)] = back(t)
    near = np.nonzero(P.route_margin(back(x), w64, cfg) < 4.0)[0]
    part.bind(weights)
    k.prepare(part.libraries())
    ctx = StepContext(k, None, Workspace("cuda"), dtype, 64, 0, 0)
    got, want = back(part.forward(ctx, x)), P.moe_ffn(back(x), w64, cfg)
    keep = np.setdiff1d(np.arange(rows), near) if dtype_name == "bfloat16" else np.arange(rows)
    assert len(keep) > rows // 2
    err = np.abs(got - want)[keep]
    assert err.max() <= (2e-5 if dtype_name == "float32" else 3e-2) * np.abs(want).max(), err.max()
    ids, _ = P.route(back(x), w64, cfg["router"])
    assert identity == 0 or (ids >= experts).any()


@pytest.mark.parametrize("K,N", [(64, 128), (128, 352), (192, 136), (704, 256), (320, 1408), (64, 130)])
@pytest.mark.parametrize("counts", [[700, 0, 1, 333, 128, 129], [900], [0, 640, 300, 0], [257] * 9 + [0] * 60 + [6000]])
def test_products_of_experts_with_many_rows(counts, K, N):
    """Uneven experts, empty ones among them, rows that belong to none behind the others'; every activation, rows gathered
    and in place, against products in 32-bit."""
    from mini_llm_runtime_amd.kernels import Kernels
    k = Kernels(torch.bfloat16)
    g = torch.Generator(device="cuda").manual_seed(K + N)
    draw = lambda *shape: torch.randn(shape, generator=g, device="cuda").to(torch.bfloat16)
    experts, rows, tail = len(counts), sum(counts), 37
    tokens = rows // 2 + 5
    x, w = draw(tokens, K), draw(experts, N, K) * K ** -0.5
    gather = torch.randint(0, tokens, (rows + tail,), generator=g, device="cuda", dtype=torch.int32)
    offsets = ints(np.concatenate([[0], np.cumsum(counts)]).tolist())
    gathered = x[gather.long()]
    want = torch.zeros((rows + tail, N), device="cuda")
    for e, (lo, n) in enumerate(zip(np.cumsum([0] + counts), counts)):
        want[lo:lo + n] = gathered[lo:lo + n].float() @ w[e].float().t()
    for act, apply in ((None, lambda z: z), ("relu_squared", lambda z: torch.relu(z) ** 2), ("gelu_erf", torch.nn.functional.gelu)):
        for source, rows_of in ((x, gather), (gathered.contiguous(), None)):
            out = torch.full((rows + tail, N), float("nan"), dtype=torch.bfloat16, device="cuda")
            k.experts_gemm(source, w, out, offsets, gather=rows_of, act=act)
            torch.testing.assert_close(out[:rows].float(), apply(want[:rows]), rtol=2e-2, atol=1e-2)
            assert torch.isnan(out[rows:].float()).all()               # (rows of no expert are not touched)
    if N % 32 == 0:
        both = want.view(rows + tail, N // 32, 2, 16)
        gate, up = both[:, :, 0].reshape(-1, N // 2), both[:, :, 1].reshape(-1, N // 2)
        clamped = lambda z, u: torch.clamp(z, max=0.8) * torch.sigmoid(1.5 * torch.clamp(z, max=0.8)) * (torch.clamp(u, -0.8, 0.8) + 1.0)
        for act, y in (("gated_silu", torch.nn.functional.silu(gate) * up), ("gated_clamped", clamped(gate, up)),
                       ("gated_gelu_tanh", torch.nn.functional.gelu(gate, approximate="tanh") * up)):
            out = torch.full((rows + tail, N // 2), float("nan"), dtype=torch.bfloat16, device="cuda")
            k.experts_gemm(x, w, out, offsets, gather=gather, act=act, limit=0.8, slope=1.5)
            torch.testing.assert_close(out[:rows].float(), y[:rows], rtol=2e-2, atol=1e-2)
            assert torch.isnan(out[rows:].float()).all()


@pytest.mark.parametrize("shapes", [[(5,)], [(3, 8), (4096,), (7,), (4100,)], [(1,), (9000,)]])
def test_staged_states_become_live_in_one_launch(shapes):
    from mini_llm_runtime_amd.cache import CacheManager, StateSpec
    from mini_llm_runtime_amd.kernels import Kernels
    k = Kernels(torch.float32)
    specs = [StateSpec(shape, torch.int32 if i == 2 else torch.float32) for i, shape in enumerate(shapes)]
    cache = CacheManager(specs, torch.float32, "cuda", 8, 64, 5, 64)
    g = torch.Generator().manual_seed(3)
    for slots in ([3], [0, 4, 2], [1, 5, 0]):                          # (the last holds the scratch request)
        want = {}
        for cid in cache._states:
            for t in (cache._states[cid], cache._staged[cid]):
                t.copy_(torch.randint(-1000, 1000, t.shape, generator=g).to(t.dtype))
            want[cid] = cache._states[cid].clone()
            want[cid][slots] = cache._staged[cid][slots]
            if 5 in slots:
                want[cid][5] = 0
        cache.commit_state(ints(slots), k)
        for cid in want:
            assert torch.equal(cache._states[cid], want[cid])


# ---- one mechanism a model ----------------------------------------------------------------------------------------
ALONE = dict(heads=1, dim=2, vdim=2, decay=[0.5], rot=dict(dims=2, base=10.0))
ONE_LAYER = {
    "lightning": dense(lightning(3, 10, 20, [0.7, 1.0, 0.97]), None),
    "window": dense(parallel(window(2, 1, 16, 48, 8, 11, 3), ALONE), None),
    "window_of_one_key": dense(parallel(window(2, 2, 16, 16, 16, 1, 2), ALONE), None),
    "retention": dense(parallel(window(1, 1, 4, 4, 2, 3, 1), retention(5, 16, 32, 8, [0.9, 0.99])), None),
    "dense": dense(lightning(2, 8, 8, [0.9]), 40),
    "experts": moe(lightning(2, 8, 16, [0.9]), 20, 7, 3, 3, 9),
    "identities_only_beside_one": moe(lightning(2, 16, 16, [0.8]), 32, 1, 5, 4, None),
}


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("name", ONE_LAYER)
def test_one_layer_models(tmp_path, dtype_name, name):
    from mini_llm_runtime_amd.parts import DecoderModel
    cfg = model(50, 48, [ONE_LAYER[name]], mult=0.8)
    folder = write_model(str(tmp_path), cfg, seed=1, matrix_std=0.2)
    loaded = DecoderModel.load(folder, DTYPES[dtype_name])
    oracle = P.PlainSagopel(folder)
    reqs = decisive_requests(oracle, 50, [90, 3], seed=4)
    want = plain_logits(oracle, reqs)
    scale = max(float(np.abs(v).max()) for v in want.values())
    r = runner_for(loaded, 128)
    close(run_steps(r, whole(reqs)), want, dtype_name, scale)
    close(run_steps(r, portions(reqs)), want, dtype_name, scale)
    close(run_steps(r, last_one_by_one(reqs, tail=40)), want, dtype_name, scale)
    idle(r)


# ---- whole models -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_every_way_of_cutting_gives_the_plain_logits(folders, name, dtype_name):
    _, reqs, want = plain(folders, name)
    scale = max(float(np.abs(v).max()) for v in want.values())
    loaded = load(folders, name, dtype_name)
    results = {}
    r = runner_for(loaded, max_tokens=192)          # one request at a time: 150 tokens -> 192
    for mode, steps in [("whole", whole(reqs)), ("last50", last_one_by_one(reqs, tail=50)), ("portions", portions(reqs))]:
        results[mode] = run_steps(r, steps)
        close(results[mode], want, dtype_name, scale)
        idle(r)
    steps, peak = mixed(reqs, seed=5)
    assert max(len(s["entries"]) for s in steps) == 4
    assert any(min(len(e["tokens"]) for e in s["entries"]) == 1 and max(len(e["tokens"]) for e in s["entries"]) > 1 for s in steps)
    assert peak < sum(-(-n // 64) * 64 for n in LENGTHS)        # pages and slots are freed and used again
    r = runner_for(loaded, max_tokens=peak)
    results["mixed"] = run_steps(r, steps)
    close(results["mixed"], want, dtype_name, scale)
    idle(r)
    # however a request was cut and whatever ran beside it: the float engine takes every sum in an order that follows
    # from the token alone, so the logits are the same to the bit
    limit = 0.0 if dtype_name == "float32" else 0.04 * scale
    for mode in ("last50", "portions", "mixed"):
        assert max_difference(results["whole"], results[mode]) <= limit, mode


@pytest.mark.parametrize("dtype_name", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_long_decoding_and_the_first_tokens(folders, name, dtype_name):
    """Five tokens, then 225 one by one, through captured graphs and without, with pages of 4: the windows pass over
    decoded tokens, pages between the kept ones and the window are given back; requests of one, two and three tokens."""
    oracle, _, _ = plain(folders, name)
    loaded = load(folders, name, dtype_name)
    reqs = decisive_requests(oracle, CONFIGS[name]["vocab"], [230, 1, 2, 3], seed=17)
    want = plain_logits(oracle, reqs)
    scale = max(float(np.abs(v).max()) for v in want.values())
    r = runner_for(loaded, max_tokens=256)
    close(run_steps(r, last_one_by_one(reqs, tail=225)), want, dtype_name, scale)
    idle(r)
    r = runner_for(loaded, max_tokens=256, use_graphs=False, page_size=4)
    close(run_steps(r, last_one_by_one(reqs, tail=225)), want, dtype_name, scale)
    close(run_steps(r, portions(reqs, sizes=(1, 1, 2, 1, 3, 2))), want, dtype_name, scale)
    idle(r)


@pytest.mark.parametrize("dtype_name", DTYPES)
def test_a_windows_pages_are_given_back_and_its_first_tokens_stay(folders, dtype_name):
    """A pool of the window's size serves a request many times as long; another request takes the pages between."""
    from mini_llm_runtime_amd.engine import Entry
    oracle, reqs, want = plain(folders, "loop")
    toks, other = reqs["r2"], reqs["r0"]
    r = runner_for(load(folders, "loop", dtype_name), max_tokens=192, page_size=8)
    scale = max(float(np.abs(v).max()) for v in want.values())
    slot = r.open_request()
    got = {}
    for t in range(0, len(toks), 6):
        rows = r.step([Entry(slot, toks[t:t + 6], list(range(len(toks[t:t + 6]))))])
        got.update({("r2", t + i): row for i, row in enumerate(back(rows))})
        windowed = [g for g, spec in enumerate(r.cache.group_specs) if spec.window is not None]
        assert windowed
        for g in windowed:
            held = int((r.cache.book.table(g)[slot] >= 0).sum())
            assert held <= -(-29 // 8) + 1 + -(-5 // 8)               # the window's pages and the kept ones
            assert r.cache.book.table(g)[slot][0] >= 0
        r.cache.check()
        if t == 96:
            beside = r.open_request()
            rows = back(r.step([Entry(beside, other, list(range(len(other))))]))
            close({("r0", i): row for i, row in enumerate(rows)}, {k: v for k, v in want.items() if k[0] == "r0"}, dtype_name, scale)
            r.close_request(beside)
    r.close_request(slot)
    close(got, {k: v for k, v in want.items() if k[0] == "r2"}, dtype_name, scale)
    idle(r)


@pytest.mark.parametrize("dtype_name", DTYPES)
def test_a_long_prompt_whole_in_portions_and_beside_single_tokens(folders, dtype_name):
    """700 tokens: long enough for the forms that many rows take."""
    oracle, _, _ = plain(folders, "plain_order")
    loaded = load(folders, "plain_order", dtype_name)
    if "long" not in _cache:
        reqs = decisive_requests(oracle, CONFIGS["plain_order"]["vocab"], [700, 40], seed=31)
        _cache["long"] = (reqs, plain_logits(oracle, reqs))
    reqs, want = _cache["long"]
    scale = max(float(np.abs(v).max()) for v in want.values())
    a, b = reqs["r0"], reqs["r1"]
    r = runner_for(loaded, max_tokens=896, max_length=768)
    close(run_steps(r, whole(reqs)), want, dtype_name, scale)
    close(run_steps(r, portions(reqs, sizes=(300, 2, 17, 129))), want, dtype_name, scale)
    steps = [dict(step=0, entries=[dict(id="r1", tokens=b[:20], want=list(range(20)))], end=[]),
             dict(step=1, entries=[dict(id="r1", tokens=b[20:21], want=[0]), dict(id="r0", tokens=a[:600], want=list(range(600)))], end=[]),
             dict(step=2, entries=[dict(id="r1", tokens=b[21:], want=list(range(19))), dict(id="r0", tokens=a[600:], want=list(range(100)))],
                  end=["r0", "r1"])]
    close(run_steps(r, steps), want, dtype_name, scale)
    idle(r)


@pytest.mark.parametrize("dtype_name", DTYPES)
def test_a_slot_used_again_starts_from_nothing(folders, dtype_name):
    from mini_llm_runtime_amd.engine import Entry
    oracle, _, _ = plain(folders, "loop")
    loaded = load(folders, "loop", dtype_name)
    reqs = decisive_requests(oracle, CONFIGS["loop"]["vocab"], [60, 44], seed=77)
    r = runner_for(loaded, max_tokens=64)
    for _ in range(2):
        for toks in reqs.values():
            slot = r.open_request()
            assert slot == 0
            got = back(r.step([Entry(slot, toks, list(range(len(toks))))]))
            want = oracle.logits(toks)
            close(dict(enumerate(got)), dict(enumerate(want)), dtype_name, np.abs(want).max())
            r.close_request(slot)
    idle(r)


@pytest.mark.parametrize("dtype_name", DTYPES)
def test_a_failed_step_leaves_the_state_as_it_was(folders, dtype_name):
    from mini_llm_runtime_amd.engine import Entry
    oracle, reqs, _ = plain(folders, "loop")
    toks = reqs["r0"]
    want = oracle.logits(toks)
    r = runner_for(load(folders, "loop", dtype_name), max_tokens=96, use_graphs=False)
    slot = r.open_request()
    first = back(r.step([Entry(slot, toks[:30], [29])]))
    original = r.kernels.normed_sum

    def failing(*args, **kwargs):
        raise RuntimeError("not this time")
    r.kernels.normed_sum = failing
    before = {cid: t.clone() for cid, t in r.cache._states.items()}
    with pytest.raises(RuntimeError, match="not this time"):
        r.step([Entry(slot, toks[30:33], [2])])
    r.kernels.normed_sum = original
    for cid, t in r.cache._states.items():
        assert torch.equal(t[slot], before[cid][slot])
    scale = np.abs(want).max()
    close({0: first[0]}, {0: want[29]}, dtype_name, scale, outliers=1)


def test_the_stream_after_every_run(folders):
    """The 32-bit engine's residual stream behind every layer run against the plain model's."""
    from mini_llm_runtime_amd.engine import Entry
    for name in ("loop", "odd"):
        oracle, _, _ = plain(folders, name)
        toks = make_requests(CONFIGS[name]["vocab"], [21], seed=2)["r0"]
        want = oracle.streams(toks)
        r = runner_for(load(folders, name, "float32"), max_tokens=64, check_finite=True, use_graphs=False)
        seen = []
        original = r.kernels.finite_check

        def recording(h, delta, layer, status, factor=1.0):
            seen.append(back(h) if delta is None else back(h) + factor * back(delta))
            original(h, delta, layer, status, factor)
        r.kernels.finite_check = recording
        r.step([Entry(r.open_request(), toks, [len(toks) - 1])])
        assert len(seen) == want.shape[0] == {"loop": 6, "odd": 4}[name]
        for i, (got, w) in enumerate(zip(seen, want)):
            np.testing.assert_allclose(got, w, atol=3e-5 * np.abs(w).max(), rtol=0, err_msg=f"run {i}")


@pytest.mark.parametrize("dtype_name,name", [("float32", "loop"), ("float32", "odd"), ("bfloat16", "plain_order"), ("bfloat16", "loop")])
def test_greedy_generation_through_the_scheduler(folders, dtype_name, name):
    from mini_llm_runtime_amd.api import LLM
    oracle, _, _ = plain(folders, name)
    prompts = list(make_requests(CONFIGS[name]["vocab"], [9, 2, 31, 1, 14, 40], seed=23).values())
    llm = LLM(folders[name], dtype=dtype_name, context_tokens=256, max_model_len=64, max_active=3, batch_tokens=24,
              prefill_chunk=8, block_size=8)
    got = llm.generate(prompts, max_tokens=7)
    for p, g in zip(prompts, got):
        w = oracle.greedy(p, 7)
        if g == w:
            continue
        assert dtype_name == "bfloat16", (g, w)
        i = next(j for j in range(7) if g[j] != w[j])                 # bfloat16 may part at a near tie only
        row = oracle.logits(p + w[:i], [len(p) + i - 1])[0]
        top = np.sort(row)[-2:]
        margins = oracle.margins(p + w[:i])
        assert top[1] - top[0] < 0.05 * np.abs(row).max() or (margins is not None and margins.min() < LEAST), (g, w)
    assert llm.runner.free_slots() == 3


def test_the_command_line_runs_a_random_model(tmp_path):
    import subprocess
    import sys
    from conftest import ROOT
    from mini_llm_runtime_amd.config import config_from_dict
    from mini_llm_runtime_amd.weights import write_random_model
    cfg = os.path.join(str(tmp_path), "config.json")
    with open(cfg, "w") as f:
        json.dump(CONFIGS["odd"], f)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "mini-llm"), "--random-weights", cfg, "--seed", "3",
                          "--prompt-ids", "1,2,3,4,5", "--tokens", "5", "--context", "256", "--dtype", "float32"], capture_output=True,
                         text=True, timeout=600)
    assert out.returncode == 0, out.stderr[-2000:]
    report = json.loads(out.stdout[out.stdout.index("{"):])
    folder = write_random_model(os.path.join(str(tmp_path), "again"), config_from_dict(CONFIGS["odd"]), 3)
    assert report["input_token_ids"] == [1, 2, 3, 4, 5] and len(report["token_ids"]) == 5
    if report["dtype"] == "float32":
        assert report["token_ids"] == P.PlainSagopel(folder).greedy([1, 2, 3, 4, 5], 5)


def test_the_trace_tool_replays_steps(folders, tmp_path):
    """bin/trace_run on a folder: portions of two requests beside each other, a request that ends and one that takes
    its slot, logits written per step."""
    import subprocess
    import sys
    from conftest import ROOT
    oracle, _, _ = plain(folders, "loop")
    reqs = make_requests(CONFIGS["loop"]["vocab"], [40, 23, 9], seed=41)
    a, b, c = reqs["r0"], reqs["r1"], reqs["r2"]
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:30], want=[0, 29])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=a[30:31], want=[0]), dict(id="b", tokens=b[:20], want=[])], end=[]),
             dict(step=2, entries=[dict(id="b", tokens=b[20:], want=[0, 2]), dict(id="a", tokens=a[31:], want=[8])], end=["a"]),
             dict(step=3, entries=[dict(id="c", tokens=c, want=[8])], end=["b", "c"])]
    out_dir = os.path.join(str(tmp_path), "out")
    os.makedirs(out_dir)
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders["loop"], "--dtype", "float32",
                          "--out", out_dir, "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps),
                         capture_output=True, text=True, timeout=900)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [line for line in run.stdout.splitlines() if line.startswith("done ")] == [f"done {i}" for i in range(4)]
    vocab = CONFIGS["loop"]["vocab"]
    rows = {i: np.fromfile(os.path.join(out_dir, f"{i}.f32"), dtype="<f4").reshape(-1, vocab) for i in range(4)}
    wa, wb, wc = oracle.logits(a), oracle.logits(b), oracle.logits(c)
    want = {0: wa[[0, 29]], 1: wa[[30]], 2: np.concatenate([wb[[20, 22]], wa[[39]]]), 3: wc[[8]]}
    for i in range(4):
        np.testing.assert_allclose(rows[i], want[i], atol=3e-4 * np.abs(wa).max(), rtol=0)


def drawn_config(rng):
    """A configuration drawn at random: any order of the mixers and feed-forwards, sizes that the matrix cores take or
    not, any loop or none."""
    width = int(rng.choice([40, 64, 72, 96, 136]))
    decays = lambda: [float(rng.choice([0.3, 0.6, 0.9, 0.97, 0.999, 1.0])) for _ in range(3)]
    even = lambda dim: int(rng.choice([r for r in (2, 4, 8, 16, 20, 32, 64) if r <= dim]))
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        if rng.random() < 0.5:
            layer = lightning(int(rng.integers(1, 6)), int(rng.choice([6, 16, 24, 32, 64])), int(rng.choice([10, 16, 32, 48, 80])), decays())
        else:
            kv, dim, keys = int(rng.choice([1, 2, 3, 4])), int(rng.choice([8, 16, 20, 32, 64])), int(rng.choice([8, 16, 22, 64]))
            layer = parallel(window(kv * int(rng.choice([1, 2, 3, 4])), kv, dim, int(rng.choice([8, 16, 32, 80])), even(dim),
                                    int(rng.choice([1, 7, 16, 33, 60])), int(rng.choice([0, 1, 4, 9, 32, 40])), cap=float(rng.choice([5.0, 20.0, 60.0])),
                                    base=float(rng.choice([100.0, 1e4, 1e6])), scale=float(rng.uniform(0.05, 0.4))),
                             retention(int(rng.integers(1, 6)), keys, int(rng.choice([16, 20, 32, 64])), even(keys), decays()))
        kind = rng.random()
        if kind < 0.4:
            layers.append(dense(layer, None if kind < 0.15 else int(rng.choice([24, 64, 100]))))
        else:
            experts, identity = int(rng.integers(1, 9)), int(rng.integers(0, 5))
            layers.append(moe(layer, int(rng.choice([16, 20, 64])), experts, identity, int(rng.integers(1, min(4, experts + identity) + 1)),
                              [None, 8, 33, 64][int(rng.integers(4))]))
    loop = None
    if rng.random() < 0.7:
        start = int(rng.integers(0, len(layers)))
        loop = (start, int(rng.integers(start + 1, len(layers) + 1)), int(rng.integers(1, 4)))
    return model(int(rng.choice([33, 100, 257])), width, layers, eps=float(rng.choice([1e-6, 1e-5, 1e-3])), mult=float(rng.choice([0.2, 0.5, 1.0])), loop=loop)


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    from mini_llm_runtime_amd.engine import Runner
    from mini_llm_runtime_amd.parts import DecoderModel
    rng = np.random.default_rng(8000 + seed)
    cfg = drawn_config(rng)
    folder = write_model(str(tmp_path), cfg, seed=seed, matrix_std=0.1)
    oracle = P.PlainSagopel(folder)
    reqs = decisive_requests(oracle, cfg["vocab"], [90, 37, 5, 64], seed=seed)
    want = plain_logits(oracle, reqs)
    scale = max(float(np.abs(v).max()) for v in want.values())
    page = int(rng.choice([4, 8, 16, 24, 32]))
    steps, peak = mixed(reqs, seed=seed)
    for dtype_name in DTYPES:
        loaded = DecoderModel.load(folder, DTYPES[dtype_name])
        results = {}
        for mode, trace, pool in (("whole", whole(reqs), 128), ("portions", portions(reqs), 128), ("mixed", steps, peak)):
            r = Runner(loaded, max_tokens=pool, max_slots=4, page_size=page, max_length=256, split_keys=64)
            results[mode] = run_steps(r, trace)
            close(results[mode], want, dtype_name, scale)
            r.cache.check()
            assert r.free_slots() == 4
        if dtype_name == "float32":
            assert max_difference(results["whole"], results["portions"]) == 0.0, cfg
            assert max_difference(results["whole"], results["mixed"]) == 0.0, cfg
