"""Takosun on the GPU against the plain oracle: mechanisms alone, portions, decoding, cache reuse, generation, replay."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import takosun_forward as tf
from tests.takosun_fixture import HUGE_LATENT, LONG_ROWS, LONGER_ROWS, ODD, SMALL, WIDE, config, dense, layer, mixer, moe, write_model

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CONFIGS = {"small": SMALL, "odd": ODD, "wide": WIDE, "huge_latent": HUGE_LATENT, "long_rows": LONG_ROWS,
           "longer_rows": LONGER_ROWS}
TOL = {"float32": 3e-5, "bfloat16": 0.06}


@pytest.fixture(scope="module")
def built(pkg, tmp_path_factory):
    """(name, dtype) -> (model, oracle), made once."""
    made, oracles, dirs = {}, {}, {}

    def get(name, dtype):
        if name not in oracles:
            w = tf.random_weights(CONFIGS[name], 100 + len(name))
            oracles[name] = tf.TakosunOracle(CONFIGS[name], w)
            dirs[name] = str(tmp_path_factory.mktemp(name))
            write_model(dirs[name], CONFIGS[name], w)
        if (name, dtype) not in made:
            made[name, dtype] = pkg.Model.load(dirs[name], 700, dtype)
        m = made[name, dtype]
        m.reset()
        for option in ("unfused", "attention", "attention_split"):
            m.set_option(option, 0)
        return m, oracles[name], dirs[name]
    return get


_truth = {}


def truth(name, oracle, n, seed=1):
    """Ids and the oracle's logits (and states after every layer) for n tokens, kept."""
    key = (name, n, seed)
    if key not in _truth:
        ids = np.random.default_rng(seed).integers(0, oracle.cfg["vocab"], n).astype(np.int32)
        states = []
        _truth[key] = (ids, oracle.forward(ids, states), states)
    return _truth[key]


def close(got, want, tol, what=""):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    err = np.linalg.norm(got - want, axis=-1) / np.linalg.norm(want, axis=-1)
    assert err.max() <= tol, (what, int(err.argmax()), float(err.max()))


def feed(model, ids, sizes):
    """Portions of the given sizes, the last one repeated; every token's logits."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(sizes[min(k, len(sizes) - 1)], len(ids) - at)
        out.append(model.forward(ids[at:at + n], range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)


# ---- mechanisms alone ------------------------------------------------------------------------

@pytest.mark.parametrize("bf16", [True, False])
@pytest.mark.parametrize("M,N,K", [(1, 1, 1), (2, 33, 7), (63, 65, 64), (64, 64, 65), (65, 200, 130), (300, 1000, 320), (2050, 1537, 96)])
def test_dense_gemm(pkg, bf16, M, N, K):
    import torch
    rng = np.random.default_rng(M + N)
    step = 64 if bf16 else 32
    ld = (K + step - 1) // step * step
    a, w = np.full((M, ld), 7.0, np.float32), np.zeros((N, ld), np.float32)   # padding of A is finite, of W zero
    a[:, :K], w[:, :K] = rng.standard_normal((M, K)), rng.standard_normal((N, K))
    kind = torch.bfloat16 if bf16 else torch.float32
    ta, tw = torch.from_numpy(a).to(kind), torch.from_numpy(w).to(kind)
    got = pkg.ops.dense_gemm(ta.cuda(), tw.cuda(), K).cpu().numpy()
    want = ta[:, :K].double().numpy() @ tw[:, :K].double().numpy().T
    scale = np.sqrt(K)
    assert np.abs(got - want).max() <= 3e-6 * scale * 4


def _latent_case(M, heads, rank, rot, pos, max_seq, seed, bf16):
    """Queries and a cache in which query row r is aimed at one far key, so that one score stands out."""
    rng = np.random.default_rng(seed)
    width, step = rank + rot, 64 if bf16 else 32
    ld = (width + step - 1) // step * step
    q, cache = np.zeros((M * heads, ld), np.float32), np.zeros((max_seq, ld), np.float32)
    cache[:, :width] = rng.standard_normal((max_seq, width))
    cache[:, :width] /= np.linalg.norm(cache[:, :width], axis=1, keepdims=True)
    cache[pos + M:] *= 1e4   # keys that nobody may see would win every softmax
    target = np.array([rng.integers(0, pos + r // heads + 1) for r in range(M * heads)])
    for r in range(M * heads):   # edges: the newest key, the first, the last of a 32- or 64-key tile, the next
        last = pos + r // heads
        edge = [last, 0, 31, 32, 63, 64, last - 1, int(target[r])][r % 8]
        target[r] = min(max(edge, 0), last)
        q[r, :width] = 12.0 * cache[target[r], :width]
    return q, cache, target


def _latent_reference(q, cache, heads, rank, rot, pos, scale):
    q, cache = q.astype(np.float64), cache.astype(np.float64)
    out = np.empty((q.shape[0], rank))
    for r in range(q.shape[0]):
        n = pos + r // heads + 1
        s = cache[:n, :rank + rot] @ q[r, :rank + rot] * scale
        p = np.exp(s - s.max())
        out[r] = p @ cache[:n, :rank] / p.sum()
    return out


@pytest.mark.parametrize("M,heads,rank,rot,pos", [
    (1, 4, 56, 8, 0), (1, 4, 56, 8, 31), (1, 16, 128, 16, 32), (1, 5, 512, 64, 63), (1, 33, 256, 16, 64), (2, 3, 11, 2, 90),
    (3, 20, 300, 20, 200), (40, 6, 120, 24, 0), (65, 2, 512, 64, 33), (130, 1, 128, 64, 127)])
def test_latent_attention(pkg, M, heads, rank, rot, pos):
    import torch
    for bf16 in (True, False):
        q, cache, target = _latent_case(M, heads, rank, rot, pos, pos + M + 70, 17, bf16)
        kind = torch.bfloat16 if bf16 else torch.float32
        tq, tc = torch.from_numpy(q).to(kind), torch.from_numpy(cache).to(kind)
        want = _latent_reference(tq.float().numpy(), tc.float().numpy(), heads, rank, rot, pos, 1.5)
        for variant, splits in [(0, 1)] + ([(1, 1), (1, 2), (1, 5), (1, 64)] if bf16 else []):
            got = pkg.ops.latent_attention(tq.cuda(), tc.cuda(), pos, rank, rot, heads, 1.5, variant, splits).float().cpu().numpy()
            close(got, want, 0.02 if bf16 else 1e-5, (bf16, variant, splits))


@pytest.mark.parametrize("M,heads,dim,rot,vdim,pos", [
    (1, 2, 16, 8, 24, 0), (64, 3, 64, 16, 64, 0), (65, 2, 128, 64, 128, 63), (130, 1, 40, 24, 33, 200), (200, 2, 192, 64, 256, 1),
    (129, 2, 56, 8, 128, 64), (17, 5, 24, 8, 7, 300)])
def test_formed_attention(pkg, M, heads, dim, rot, vdim, pos):
    import torch
    rng = np.random.default_rng(5)
    max_seq = pos + M + 40
    ld_v, ld_rot = (max_seq + 63) // 64 * 64, rot + 8
    k = rng.standard_normal((max_seq, heads, dim)).astype(np.float32)
    kr = rng.standard_normal((max_seq, ld_rot)).astype(np.float32)
    v = rng.standard_normal((heads, vdim, ld_v)).astype(np.float32)
    gates = rng.standard_normal((M, heads)).astype(np.float32)
    q = np.empty((M, heads, dim + rot), np.float32)
    for m in range(M):
        for h in range(heads):
            last = pos + m
            t = min(max([last, 0, 63, 64, last - 1, int(rng.integers(0, last + 1)), 127, 128][(m + h) % 8], 0), last)
            full = np.concatenate([k[t, h], kr[t, :rot]])
            q[m, h] = 12.0 * full / np.linalg.norm(full)
    k[pos + M:] *= 1e4
    B = torch.bfloat16
    tq, tk, tr, tv = (torch.from_numpy(x).to(B) for x in (q, k.reshape(max_seq, -1), kr, v.reshape(heads * vdim, ld_v)))
    got = pkg.ops.formed_attention(tq.cuda(), tk.cuda(), tr.cuda(), tv.cuda(), torch.from_numpy(gates).cuda(), pos, vdim, 0.3)
    fq, fk, fr = tq.double().numpy(), tk.double().numpy().reshape(max_seq, heads, dim), tr.double().numpy()[:, :rot]
    fv = tv.double().numpy().reshape(heads, vdim, ld_v)
    want = np.empty((M, heads, vdim))
    for m in range(M):
        n = pos + m + 1
        for h in range(heads):
            s = (fk[:n, h] @ fq[m, h, :dim] + fr[:n] @ fq[m, h, dim:]) * 0.3
            p = np.exp(s - s.max())
            want[m, h] = fv[h, :, :n] @ p / p.sum() / (1 + np.exp(-gates[m, h]))
    close(got.float().cpu().numpy().reshape(M, heads, vdim), want, 0.02)


# ---- the model -------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n", [("small", 1), ("small", 2), ("small", 75), ("odd", 40), ("wide", 150), ("huge_latent", 20), ("long_rows", 9),
                                    ("longer_rows", 9)])
def test_whole_prompt(built, name, n, dtype):
    model, oracle, _ = built(name, dtype)
    ids, want, states = truth(name, oracle, n)
    close(model.forward(ids, range(n)), want, TOL[dtype])
    # the stream after every layer: the mean over depth of what the model holds before it
    width, pre = oracle.cfg["width"], []
    for i in range(len(states) + 1):
        pre.append(model.read_buffer(f"state{i}", n, width).astype(np.float64))
        if i:
            close(tf.depth_average(pre, oracle.w[f"l{i - 1}.dwa"]), states[i - 1], TOL[dtype], f"layer {i - 1}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n", [("small", 75), ("odd", 40), ("wide", 70), ("huge_latent", 20), ("long_rows", 9), ("longer_rows", 9)])
@pytest.mark.parametrize("sizes", [[1], [2], [3], [31, 1, 2, 33, 1], [64, 2, 1], [5, 17, 1]])
def test_portions(built, name, n, dtype, sizes):
    model, oracle, _ = built(name, dtype)
    ids, want, _ = truth(name, oracle, n)
    close(feed(model, ids, sizes), want, TOL[dtype])
    assert model.position == n


@pytest.mark.parametrize("option", [("unfused", 1), ("attention", 1), ("attention", 2), ("attention", 3), ("attention_split", 1),
                                    ("attention_split", 7)])
def test_kernel_choices_agree(built, option):
    model, oracle, _ = built("wide", "bfloat16")
    ids, want, _ = truth("wide", oracle, 70)
    model.set_option(*option)
    close(feed(model, ids, [50, 3, 9, 1]), want, TOL["bfloat16"], option)


def test_unfused_one_token_pass_in_32_bit(built):
    for name, n in (("small", 75), ("odd", 40)):
        model, oracle, _ = built(name, "float32")
        ids, want, _ = truth(name, oracle, n)
        model.set_option("unfused", 1)
        close(feed(model, ids, [n - 6, 1]), want, TOL["float32"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_far_keys_show(pkg, tmp_path, dtype):
    """Sharp attention: some queries are aimed at one earlier token, hundreds of keys away or at a tile's edge."""
    W, V = 64, 600
    cfg = config(V, W, 1, [layer(mixer(2, 32, 8, 32, 64, 64, 1.0), None)])
    rng = np.random.default_rng(21)
    w = tf.random_weights(cfg, 22)
    e = rng.standard_normal((V, W))
    w["embed"] = tf.round_bf16(e / np.sqrt((e * e).mean(1, keepdims=True)))
    for n in ("norm1", "mix.dq.norm", "mix.dkv.norm"):
        w["l0." + n] = np.ones_like(w["l0." + n])
    eye = np.eye(64)
    w["l0.mix.dq"] = np.roll(eye, 7, axis=1).astype(np.float32)   # a query latent is the token's row shifted by 7
    dkv = np.zeros((72, W)); dkv[:64] = eye
    w["l0.mix.dkv"] = dkv.astype(np.float32)                      # a key latent is the row itself; no rotated part
    w["l0.mix.uk"] = eye.astype(np.float32)
    uq = np.zeros((80, 64)); uq[0:32] = eye[:32]; uq[40:72] = eye[32:]
    w["l0.mix.uq"] = uq.astype(np.float32)
    w["l0.dwa"] = np.array([0.0, 1.0], np.float32)
    ids = np.arange(420)
    far = {331: 0, 332: 31, 340: 32, 350: 63, 360: 64, 370: 127, 380: 128, 390: 255, 400: 256, 419: 5}
    for i, target in far.items():                                 # token i looks for token `target`, and finds it alone
        w["embed"][i] = np.roll(w["embed"][target], 7)
    write_model(str(tmp_path), cfg, w)
    oracle = tf.TakosunOracle(cfg, w)
    want = oracle.forward(ids)
    model = pkg.Model.load(str(tmp_path), 512, dtype)
    for sizes in ([420], [300, 1], [200, 64, 7, 2]):
        model.reset()
        close(feed(model, ids, sizes), want, 2e-5 if dtype == "float32" else 0.03, sizes)
    # a missing far key must show at that limit (the mistake is planted in the oracle; nothing here rotates)
    for i, target in far.items():
        short = oracle.forward(np.delete(ids[:i + 1], target))[-1]
        assert np.linalg.norm(short - want[i]) / np.linalg.norm(want[i]) > 0.3


def test_cache_is_given_back(built):
    for dtype in ("float32", "bfloat16"):
        model, oracle, _ = built("small", dtype)
        a = truth("small", oracle, 75)
        b = truth("small", oracle, 33, seed=2)
        close(feed(model, a[0], [40, 1]), a[1], TOL[dtype])
        model.reset()
        assert model.position == 0
        first = feed(model, b[0], [20, 1])
        close(first, b[1], TOL[dtype])
        model.reset()
        assert np.array_equal(feed(model, b[0], [20, 1]), first)


def test_long_decoding(built):
    model, oracle, _ = built("small", "float32")
    ids, want, _ = truth("small", oracle, 320)
    close(feed(model, ids, [3, 1]), want, TOL["float32"])


def test_portions_beyond_one_pass(pkg, tmp_path):
    """A prompt longer than a pass is cut inside the model; the wanted places follow."""
    cfg = config(61, 32, 2, [layer(mixer(1, 8, 8, 8, 16, 24, 0.4), moe(3, 2, 16)), layer(mixer(1, 8, 8, 8, 8, 24, 0.4, kv_from=0), None)])
    write_model(str(tmp_path), cfg, tf.random_weights(cfg, 8))
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


@pytest.mark.parametrize("name", ["small", "odd"])
def test_greedy_generation(built, name):
    """The framework's own generation (graph replays) against the oracle, and against single steps of the same model."""
    model, oracle, _ = built(name, "float32")
    ids = truth(name, oracle, 20)[0]
    want = tf.greedy(oracle, ids, 24)
    for _ in range(2):
        model.reset()
        got, _, _ = model.generate_greedy(ids, 24)
        assert got.tolist() == want
    assert model.position == 20 + 23
    more, _, _ = model.generate_greedy(got[-1:], 5)      # on top of what is cached
    assert more.tolist() == tf.greedy(oracle, list(ids) + want, 5)


def test_greedy_generation_in_bfloat16_replays_its_own_steps(built):
    model, oracle, _ = built("wide", "bfloat16")
    ids = truth("wide", oracle, 150)[0]
    got, _, _ = model.generate_greedy(ids, 30)
    model.reset()
    model.set_option("attention_split", 0)
    logits, out = model.forward(ids), []
    for _ in range(30):
        out.append(int(logits[0].argmax()))
        logits = model.forward([out[-1]])
    close_calls = sum(a != b for a, b in zip(got.tolist(), out))
    assert got[0] == out[0] and (close_calls == 0 or got.tolist()[:10] == out[:10])


def test_bad_requests_are_errors(built, pkg):
    model, _, _ = built("small", "bfloat16")
    for ids, want in (([1] * 701, [0]), ([], []), ([1, 2, 3], [3]), ([1, 2, 3], [2, 1])):
        with pytest.raises(pkg.capi.A81W41Error):
            model.forward(ids, want)
    assert model.position == 0
    with pytest.raises(pkg.capi.A81W41Error):
        model.set_option("no such", 1)
    with pytest.raises(pkg.capi.A81W41Error):
        model.generate_greedy([1] * 690, 20)


def test_trace_run(built, tmp_path):
    model, oracle, root = built("small", "float32")
    a, b = truth("small", oracle, 75), truth("small", oracle, 33, seed=2)
    steps, expected = [], {}
    for rid, (ids, want, _), sizes in (("a", a, [40, 2, 1, 1, 31]), ("b", b, [32, 1])):
        at = 0
        for n in sizes:
            w = [] if n == 2 else sorted({0, n - 1})
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": ids[at:at + n].tolist(), "want": w}],
                          "end": [rid] if at + n == len(ids) else []})
            expected[len(steps) - 1] = want[[at + k for k in w]]
            at += n
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", root, "--dtype", dtype, "--out", str(out),
                            "--max-tokens", "80"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                           timeout=100)
        assert r.returncode == 0, r.stderr
        assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {k}" for k in range(len(steps))]
        for k, want in expected.items():
            path = out / f"{k}.f32"
            assert path.exists() == bool(len(want))
            if len(want):
                close(np.fromfile(path, "<f4").reshape(len(want), -1), want, TOL[dtype], k)
