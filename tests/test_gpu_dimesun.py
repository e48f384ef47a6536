"""Dimesun on the GPU against the plain oracle: mechanisms alone, portions, decoding, states and cache given back,
generation, replay."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import dimesun_forward as df
from tests.dimesun_fixture import (HUGE, LARGE, LONG_ROWS, MANY_VALUES, ODD, SMALL, TOL, WIDE, Truth, attention, config, mlstm, moe,
                                   row_errors, write_model)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CONFIGS = {"small": SMALL, "odd": ODD, "wide": WIDE, "large": LARGE, "huge": HUGE, "long_rows": LONG_ROWS, "many_values": MANY_VALUES}
OPTIONS = ("unfused", "attention", "attention_split", "memory", "keep_states")


@pytest.fixture(scope="module")
def built(pkg, tmp_path_factory):
    """(name, dtype) -> (model, oracle, folder), made once."""
    made, oracles, dirs = {}, {}, {}

    def get(name, dtype):
        if name not in oracles:
            w = df.random_weights(CONFIGS[name], 100 + len(name))
            oracles[name] = df.DimesunOracle(CONFIGS[name], w)
            dirs[name] = str(tmp_path_factory.mktemp(name))
            write_model(dirs[name], CONFIGS[name], w)
        if (name, dtype) not in made:
            made[name, dtype] = pkg.Model.load(dirs[name], 400, dtype)
        m = made[name, dtype]
        m.reset()
        for option in OPTIONS:
            m.set_option(option, 0)
        return m, oracles[name], dirs[name]
    return get


_truth = {}


def truth(name, oracle, n, seed=1):
    key = (name, n, seed)
    if key not in _truth:
        _truth[key] = Truth(oracle, n, seed)
    return _truth[key]


def close(got, want, tol, what=""):
    """tol: one limit, or one for every row"""
    err = row_errors(got, want)
    worst = int((err / tol).argmax())
    assert (err <= tol).all(), (what, worst, float(err.reshape(-1)[worst]))


def feed(model, ids, sizes):
    """Portions of the given sizes, the last one repeated; every token's logits."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(sizes[min(k, len(sizes) - 1)], len(ids) - at)
        out.append(model.forward(ids[at:at + n], range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)


# ---- mechanisms alone ------------------------------------------------------------------------

def _grouped_case(M, heads, kv_heads, dim, vdim, pos, chunk, seed):
    """Queries of which each is aimed at one key, at an edge of its chunk or of a tile; what nobody may see would win every
    softmax.  Some queries are aimed away from all keys, so that the sink takes most of the weight."""
    rng = np.random.default_rng(seed)
    max_seq = pos + M + 70
    k = rng.standard_normal((max_seq, kv_heads, dim))
    k /= np.linalg.norm(k, axis=2, keepdims=True)
    v = rng.standard_normal((max_seq, kv_heads, vdim))
    q = np.zeros((M, heads, dim))
    for m in range(M):
        last = pos + m
        first = last - last % chunk if chunk else 0
        for h in range(heads):
            edge = [last, first, first + 31, first + 63, first + 64, last - 1, int(rng.integers(first, last + 1)), first + 1][(m + h) % 8]
            q[m, h] = 8.0 * k[min(max(edge, first), last), h // (heads // kv_heads)]
            if (m + 3 * h) % 5 == 4:
                q[m, h] *= -0.5
    return q, k, v


def _grouped_reference(q, k, v, pos, scale, chunk, sink):
    M, heads, _ = q.shape
    group = heads // k.shape[1]
    out = np.empty((M, heads, v.shape[2]))
    for m in range(M):
        seen = [j for j in range(pos + m + 1) if not chunk or df.sees(pos + m, j, chunk)]
        for h in range(heads):
            s = k[seen, h // group] @ q[m, h] * scale
            p = df.sink_softmax(s) if sink else np.exp(s - s.max()) / np.exp(s - s.max()).sum()
            out[m, h] = p @ v[seen, h // group]
    return out


@pytest.mark.parametrize("M,heads,kv_heads,dim,vdim,pos,chunk", [
    (1, 4, 2, 24, 40, 0, 7), (1, 6, 1, 64, 64, 255, 64), (1, 16, 2, 128, 128, 256, 64), (1, 8, 1, 128, 96, 300, 128), (1, 40, 2, 96, 96, 190, 0),
    (2, 3, 3, 8, 16, 62, 63), (3, 20, 5, 136, 256, 200, 100), (5, 12, 4, 64, 8, 130, 1), (40, 6, 1, 56, 120, 0, 11), (65, 2, 2, 128, 64, 33, 32),
    (130, 8, 2, 64, 64, 127, 65), (200, 5, 1, 200, 136, 0, 0), (90, 4, 4, 264, 272, 10, 40), (150, 6, 2, 72, 128, 64, 128)])
@pytest.mark.parametrize("sink", [True, False])
def test_grouped_attention(pkg, M, heads, kv_heads, dim, vdim, pos, chunk, sink):
    import torch
    q, k, v = _grouped_case(M, heads, kv_heads, dim, vdim, pos, chunk, 17)
    key, value = (dim + 7) // 8 * 8, (vdim + 7) // 8 * 8
    row = kv_heads * (key + value)
    ld = (row + 63) // 64 * 64
    rows = np.zeros((k.shape[0], ld))
    parts = rows[:, :row].reshape(-1, kv_heads, key + value)
    parts[:, :, :vdim], parts[:, :, value:value + dim] = v, k
    queries = np.zeros((M, heads, key))
    queries[:, :, :dim] = q
    for kind, tol in ((torch.bfloat16, 0.02), (torch.float32, 1e-5)):
        tq, tr = torch.from_numpy(queries).to(kind), torch.from_numpy(rows).to(kind)
        fq, fr = tq.double().numpy()[:, :, :dim], tr.double().numpy()[:, :row].reshape(-1, kv_heads, key + value)
        want = _grouped_reference(fq, fr[:, :, value:value + dim], fr[:, :, :vdim], pos, 1.0, chunk, sink)
        unseen = rows.copy()
        unseen[pos + M:] *= 1e4
        if chunk:
            unseen[:pos - pos % chunk] *= 1e4
        tu = torch.from_numpy(unseen).to(kind).cuda()
        choices = [(0, 1)]
        if kind == torch.bfloat16 and max(key, value) <= 256:
            choices += [(1, 1), (1, 2), (1, 5), (1, 64)]
        for variant, splits in choices:
            got = pkg.ops.grouped_attention(tq.cuda(), tu, pos, kv_heads, key, vdim, 1.0, chunk, sink, variant, splits).double().cpu().numpy()
            # where the sink has nearly all the weight the result is small: an absolute part for it
            err = np.linalg.norm(got - want, axis=2) / (np.linalg.norm(want, axis=2) + 0.05 * math.sqrt(vdim))
            assert err.max() <= tol, (kind, variant, splits, err.max(), np.unravel_index(err.argmax(), err.shape))


def _memory_rows(T, heads, dim, vdim, seed, shift_i=0.0, shift_f=2.0, spread=2.0):
    rng = np.random.default_rng(seed)
    n = heads * (2 * dim + 2 * vdim + 2)
    rows = rng.standard_normal((T, (n + 3) // 4 * 4)).astype(np.float32)
    rows[:, n - 2 * heads:n] *= spread
    bias_i = (shift_i + rng.standard_normal(heads)).astype(np.float32)
    bias_f = (shift_f + rng.standard_normal(heads)).astype(np.float32)
    return rows, bias_i, bias_f, (1 + 0.3 * rng.standard_normal(heads * vdim)).astype(np.float32)


def _memory_reference(rows, heads, dim, vdim, cap, eps, bias_i, bias_f, norm):
    rows = rows.astype(np.float64)
    T = len(rows)
    at = np.cumsum([0, heads * dim, heads * dim, heads * vdim, heads * vdim, heads, heads])
    q, k, v, g, zi, zf = (rows[:, a:b] for a, b in zip(at[:-1], at[1:]))
    log_in, log_keep = df.soft_cap(zi + bias_i, cap), df.log_sigmoid(df.soft_cap(zf + bias_f, cap))
    out = np.empty((T, heads, vdim))
    for h in range(heads):
        memory = df.MatrixMemory(dim, vdim)
        for t in range(T):
            d, e = slice(h * dim, (h + 1) * dim), slice(h * vdim, (h + 1) * vdim)
            out[t, h] = memory.step(q[t, d] / math.sqrt(dim), k[t, d], v[t, e], log_in[t, h], log_keep[t, h])
    return df.unit_rms(out, eps).reshape(T, -1) * norm * df.sigmoid(g)


GATES = {"mixed": (0.0, 2.0, 2.0), "keep for long": (-2.0, 12.0, 0.5), "forget at once": (0.0, -20.0, 6.0), "sudden inputs": (0.0, 3.0, 12.0)}


@pytest.mark.parametrize("gates", sorted(GATES))
@pytest.mark.parametrize("heads,dim,vdim", [(2, 12, 20), (1, 3, 5), (3, 128, 128), (2, 72, 160), (1, 130, 260), (1, 33, 512), (2, 256, 30)])
def test_matrix_memory(pkg, heads, dim, vdim, gates):
    """Both kernels, whole and in portions that hand the state on, single tokens among them; eps large, so that the
    denominator shows."""
    import torch
    T, cap, eps = 200, 15.0, 0.3
    rows, bi, bf, norm = _memory_rows(T, heads, dim, vdim, dim + vdim, *GATES[gates])
    want = _memory_reference(rows, heads, dim, vdim, cap, eps, bi, bf, norm)
    dev = [torch.from_numpy(x).cuda() for x in (bi, bf, norm)]
    for variants, sizes in (([0], [T]), ([1], [T]), ([1, 0], [64, 1, 63, 1, 2, 65]), ([1], [1, 3, 130, 2]), ([0, 1], [5, 100, 1]),
                            ([1, 1, 0], [127, 1, 1])):
        state, out, at, k = pkg.ops.matrix_memory_state(heads, dim, vdim), [], 0, 0
        while at < T:
            n = min(sizes[k % len(sizes)], T - at)
            part = torch.from_numpy(rows[at:at + n]).cuda().contiguous()
            out.append(pkg.ops.matrix_memory(part, heads, dim, vdim, cap, eps, *dev, state, at, variants[k % len(variants)]).cpu().numpy())
            at, k = at + n, k + 1
        got = np.concatenate(out)
        scale = np.sqrt((want ** 2).mean())
        assert np.abs(got - want).max() <= 5e-5 * max(scale, 1.0) * 10, (variants, sizes, np.abs(got - want).max())
        close(got, want, 5e-5, (variants, sizes))


def test_matrix_memory_finds_a_far_token(pkg):
    """One key among hundreds is asked for again, across chunks and portions: a lost or decayed state would not have it."""
    import torch
    T, dim, vdim, cap, eps = 420, 64, 96, 15.0, 1e-5
    rng = np.random.default_rng(8)
    n = 2 * dim + 2 * vdim + 2
    rows = np.zeros((T, n), np.float32)
    rows[:, :2 * dim] = 0.01 * rng.standard_normal((T, 2 * dim))
    rows[:, 2 * dim:2 * dim + vdim] = rng.standard_normal((T, vdim))
    rows[:, -1] = 20.0                       # nothing is forgotten
    asked = {100: 3, 128: 63, 129: 64, 300: 3, 333: 255, 419: 64}
    keys, _ = np.linalg.qr(rng.standard_normal((dim, len(asked))))
    for k, s in enumerate(sorted(set(asked.values()))):
        rows[s, dim:2 * dim] = 8 * keys[:, k]
    for t, s in asked.items():
        rows[t, :dim] = rows[s, dim:2 * dim]
    zero, one = np.zeros(1, np.float32), np.ones(vdim, np.float32)
    want = _memory_reference(rows, 1, dim, vdim, cap, eps, zero, zero, one)
    for t, s in asked.items():               # the oracle finds it: the value of token s, up to its length and sign
        v = rows[s, 2 * dim:2 * dim + vdim]
        assert abs(v @ want[t]) / np.linalg.norm(v) / np.linalg.norm(want[t]) > 0.8
    dev = [torch.from_numpy(x).cuda() for x in (zero, zero, one)]
    for variants, sizes in (([1], [420]), ([1, 0], [65, 1]), ([0], [420]), ([1], [2])):
        state, out, at, k = pkg.ops.matrix_memory_state(1, dim, vdim), [], 0, 0
        while at < T:
            m = min(sizes[k % len(sizes)], T - at)
            part = torch.from_numpy(rows[at:at + m]).cuda().contiguous()
            out.append(pkg.ops.matrix_memory(part, 1, dim, vdim, cap, eps, *dev, state, at, variants[k % len(variants)]).cpu().numpy())
            at, k = at + m, k + 1
        close(np.concatenate(out), want, 1e-4, (variants, sizes))


@pytest.mark.parametrize("M,experts,top", [(1, 1, 1), (7, 5, 5), (130, 12, 3), (9, 64, 6), (5, 65, 64), (33, 300, 8), (3, 2048, 17)])
def test_router(pkg, M, experts, top):
    import torch
    rng = np.random.default_rng(M)
    z, bias = rng.standard_normal((M, experts)).astype(np.float32) * 3, rng.standard_normal(experts).astype(np.float32)
    if experts >= 5:
        z[0] = 0.0
        bias[1] = bias[3] = bias.max() + 1.0   # equals: the lower number comes first
    chosen, weights = (x.cpu().numpy() for x in pkg.ops.router(torch.from_numpy(z).cuda(), torch.from_numpy(bias).cuda(), top))
    for m in range(M):
        best, w = df.choose((z[m] + bias).astype(np.float64), top)
        assert chosen[m].tolist() == best
        assert np.abs(weights[m] - w).max() <= 1e-6


# ---- the model -------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n", [("small", 1), ("small", 2), ("small", 75), ("odd", 40), ("wide", 150), ("large", 120), ("huge", 40),
                                    ("long_rows", 9), ("many_values", 9)])
def test_whole_prompt(built, name, n, dtype):
    model, oracle, _ = built(name, dtype)
    t = truth(name, oracle, n)
    model.set_option("keep_states", 1)
    close(model.forward(t.ids, range(n)), t.logits, t.limits[dtype])
    for i, state in enumerate(t.states):
        close(model.read_buffer(f"state{i}", n, oracle.cfg["width"]), state, t.limits[dtype], f"layer run {i}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n", [("small", 75), ("odd", 40), ("wide", 150), ("large", 120), ("huge", 40), ("long_rows", 9),
                                    ("many_values", 9)])
@pytest.mark.parametrize("sizes", [[1], [2], [3], [31, 1, 2, 33, 1], [64, 2, 1], [5, 17, 1], [70, 1, 66]])
def test_portions(built, name, n, dtype, sizes):
    model, oracle, _ = built(name, dtype)
    t = truth(name, oracle, n)
    model.set_option("keep_states", 1)
    close(feed(model, t.ids, sizes), t.logits, t.limits[dtype])
    assert model.position == n
    last = last_portion(n, sizes)
    for i, state in enumerate(t.states):
        close(model.read_buffer(f"state{i}", last, oracle.cfg["width"]), state[n - last:], t.limits[dtype][n - last:], f"layer run {i}")


def last_portion(n, sizes):
    k, last = 0, 0
    while n > 0:
        last = min(sizes[min(k, len(sizes) - 1)], n)
        n, k = n - last, k + 1
    return last


@pytest.mark.parametrize("name", ["wide", "large"])
@pytest.mark.parametrize("option", [("unfused", 1), ("attention", 1), ("attention_split", 1), ("attention_split", 7), ("memory", 1), ("memory", 2)])
def test_kernel_choices_agree(built, option, name):
    for dtype in ("bfloat16", "float32"):
        model, oracle, _ = built(name, dtype)
        t = truth(name, oracle, 120)
        model.set_option(*option)
        if option[0] == "memory":
            model.set_option("unfused", 1)
        close(feed(model, t.ids, [50, 3, 9, 1]), t.logits, t.limits[dtype], (option, dtype))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_and_chunk_edges_show(pkg, tmp_path, dtype):
    """Sharp attention: some queries are aimed at one earlier token, just inside or just outside their chunk."""
    W, V, chunk = 64, 600, 90
    cfg = config(V, W, [attention(2, 1, 40, 40, chunk, 1.0, rot_dims=8)], (0, 1, 1), residual_mult=1.0)
    rng = np.random.default_rng(21)
    w = df.random_weights(cfg, 22)
    w["loop.step"] = np.zeros_like(w["loop.step"])
    w["l0.norm1"] = np.zeros_like(w["l0.norm1"])
    eye = np.eye(W)
    q, k, v = np.zeros((80, W)), np.zeros((40, W)), np.zeros((40, W))
    k[8:40] = eye[:32]                                            # a key is the first half of a token's row, not rotated
    q[8:40], q[48:80] = eye[32:], eye[32:]                        # a query the second half
    v[:32] = np.roll(eye, 5, axis=0)[:32]
    for name, a in (("q", q), ("k", k), ("v", v)):
        w["l0.mix." + name] = a.astype(np.float32)
    e = rng.standard_normal((V, W))
    e[:, 32:] *= 0.05
    ids = np.arange(420)
    far = {31: 0, 62: 0, 88: 0, 89: 0, 90: 89, 91: 0, 95: 90, 153: 90, 154: 90, 179: 90, 180: 90, 181: 180, 269: 180, 270: 180, 300: 265,
           359: 270, 360: 359, 400: 360, 419: 364}
    for i, target in far.items():                                 # token i looks for token `target`, if it may see it
        e[i, 32:] = 3.0 * e[target, :32] / np.linalg.norm(e[target, :32])
    w["embed"] = df.round_bf16(e / np.sqrt((e * e).mean(1, keepdims=True)))
    write_model(str(tmp_path), cfg, w)
    oracle = df.DimesunOracle(cfg, w)
    want = oracle.forward(ids)
    model = pkg.Model.load(str(tmp_path), 512, dtype)
    for sizes in ([420], [300, 1], [89, 1, 2, 88, 1, 1, 2, 100, 7, 2]):
        model.reset()
        close(feed(model, ids, sizes), want, 2e-5 if dtype == "float32" else 0.03, sizes)
    # a window that is one token off must show at that limit (the mistake is planted in the oracle)
    for off in (1, -1):
        cfg["layers"][0]["mixer"]["mask"]["size"] = chunk + off
        err = np.linalg.norm(df.DimesunOracle(cfg, w).forward(ids) - want, axis=1) / np.linalg.norm(want, axis=1)
        assert sum(err[i] > 0.1 for i in (89, 90, 179, 180, 269, 270, 359, 360)) >= 3, err


def test_state_and_cache_are_given_back(built):
    for name in ("small", "wide"):
        for dtype in ("float32", "bfloat16"):
            model, oracle, _ = built(name, dtype)
            a, b = truth(name, oracle, 75), truth(name, oracle, 33, seed=2)
            close(feed(model, a.ids, [40, 1]), a.logits, a.limits[dtype])
            model.reset()
            assert model.position == 0
            first = feed(model, b.ids, [20, 1])
            close(first, b.logits, b.limits[dtype])
            model.reset()
            assert np.array_equal(feed(model, b.ids, [20, 1]), first)
            model.reset()
            feed(model, a.ids[:7], [1])          # an odd number of tokens leaves the other copies of n and m in use
            model.reset()
            assert np.array_equal(feed(model, b.ids, [20, 1]), first)


def test_long_decoding(built):
    for name in ("small", "odd"):
        model, oracle, _ = built(name, "float32")
        t = truth(name, oracle, 320)
        close(feed(model, t.ids, [3, 1]), t.logits, TOL["float32"])


def test_portions_beyond_one_pass(pkg, tmp_path):
    """A prompt longer than a pass is cut inside the model; the wanted places and the state follow."""
    cfg = config(61, 32, [attention(2, 1, 8, 8, 700, 0.4, mlp=moe(3, 2, 16)), mlstm(1, 16, 8)], (0, 2, 2))
    write_model(str(tmp_path), cfg, df.random_weights(cfg, 8))
    ids = np.random.default_rng(4).integers(0, 61, 8300)
    for dtype in ("float32", "bfloat16"):
        model = pkg.Model.load(str(tmp_path), 8300, dtype)
        want = [0, 4095, 4096, 4097, 8191, 8192, 8299]
        whole = model.forward(ids, want)
        model.reset()
        out = []
        for at in range(0, 8300, 1000):
            n = min(1000, 8300 - at)
            out.append(model.forward(ids[at:at + n], range(n)))
        close(whole, np.concatenate(out)[want], 1e-4 if dtype == "float32" else 0.03)


@pytest.mark.parametrize("name", ["small", "odd", "large"])
def test_greedy_generation(built, name):
    """The framework's own generation (graph replays) against the oracle."""
    model, oracle, _ = built(name, "float32")
    ids = truth(name, oracle, 20).ids
    want = df.greedy(oracle, ids, 24)
    for _ in range(2):
        model.reset()
        got, _, _ = model.generate_greedy(ids, 24)
        assert got.tolist() == want
    assert model.position == 20 + 23
    more, _, _ = model.generate_greedy(got[-1:], 5)      # on top of what is cached
    assert more.tolist() == df.greedy(oracle, list(ids) + want, 5)


def test_greedy_generation_in_bfloat16_replays_its_own_steps(built):
    model, oracle, _ = built("wide", "bfloat16")
    ids = truth("wide", oracle, 150).ids
    got, _, _ = model.generate_greedy(ids, 30)
    model.reset()
    again, _, _ = model.generate_greedy(ids, 30)
    assert np.array_equal(got, again)
    model.reset()
    logits, out = model.forward(ids), []
    for _ in range(30):
        out.append(int(logits[0].argmax()))
        logits = model.forward([out[-1]])
    assert got[0] == out[0] and got.tolist()[:10] == out[:10]


def test_two_sequences_side_by_side(pkg, built):
    """Sessions share nothing: interleaved calls of unequal requests give what each gives alone."""
    _, oracle, root = built("small", "float32")
    seqs = [truth("small", oracle, 75), truth("small", oracle, 33, seed=2)]
    models = [pkg.Model.load(root, 80, "float32") for _ in seqs]
    got = [[], []]
    for at in range(0, 75, 5):
        for k, t in enumerate(seqs):
            part = t.ids[at:at + 5]
            if len(part):
                got[k].append(models[k].forward(part, range(len(part))))
    for k, t in enumerate(seqs):
        close(np.concatenate(got[k]), t.logits, TOL["float32"])


def test_bad_requests_are_errors(built, pkg):
    model, _, _ = built("small", "bfloat16")
    for ids, want in (([1] * 401, [0]), ([], []), ([1, 2, 3], [3]), ([1, 2, 3], [2, 1])):
        with pytest.raises(pkg.capi.A81W41Error):
            model.forward(ids, want)
    assert model.position == 0
    for option in (("no such", 1), ("memory", 3), ("attention", 2)):
        with pytest.raises(pkg.capi.A81W41Error):
            model.set_option(*option)
    with pytest.raises(pkg.capi.A81W41Error):
        model.generate_greedy([1] * 390, 20)


def test_a_pass_without_wanted_logits_carries_on(built):
    for dtype in ("float32", "bfloat16"):
        model, oracle, _ = built("wide", dtype)
        t = truth("wide", oracle, 75)
        for a, b in ((0, 40), (40, 41), (41, 43), (43, 44)):
            assert model.forward(t.ids[a:b], []).shape == (0, 300)
        close(model.forward(t.ids[44:], range(31)), t.logits[44:], t.limits[dtype][44:])


def test_trace_run(built, tmp_path):
    _, oracle, root = built("small", "float32")
    a, b = truth("small", oracle, 75), truth("small", oracle, 33, seed=2)
    steps, expected = [], {}
    for rid, t, sizes in (("a", a, [40, 2, 1, 1, 31]), ("b", b, [32, 1])):
        at = 0
        for n in sizes:
            w = [] if n == 2 else sorted({0, n - 1})
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": t.ids[at:at + n].tolist(), "want": w}],
                          "end": [rid] if at + n == len(t.ids) else []})
            expected[len(steps) - 1] = (t, [at + k for k in w])
            at += n
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", root, "--dtype", dtype, "--out", str(out),
                            "--max-tokens", "80"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                           timeout=100)
        assert r.returncode == 0, r.stderr
        assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {k}" for k in range(len(steps))]
        for k, (t, places) in expected.items():
            path = out / f"{k}.f32"
            assert path.exists() == bool(places)
            if places:
                close(np.fromfile(path, "<f4").reshape(len(places), -1), t.logits[places], t.limits[dtype][places], k)


def test_generate_command(built):
    _, oracle, root = built("small", "float32")
    prompt = [5, 17, 3, 101, 64]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", root, "--dtype", "float32", "--tokens",
                        ",".join(map(str, prompt)), "--new", "9"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split(",")] == df.greedy(oracle, prompt, 9)
