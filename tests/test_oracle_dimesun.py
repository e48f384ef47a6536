"""The Dimesun oracle against properties that the mathematics fixes, and mistakes planted in it: what the tolerances of the
GPU tests can tell apart (no GPU)."""
import copy
import math

import numpy as np
import pytest

from oracle import dimesun_forward as df
from tests.dimesun_fixture import ODD, SMALL, WIDE, Truth, attention, config, mlstm, moe, row_errors

RNG = np.random.default_rng(3)


def tensors(cfg, seed, layer=0, part="mix."):
    w = {k: np.asarray(v, np.float64) for k, v in df.random_weights(cfg, seed).items()}
    return lambda name: w[f"l{layer}.{part}{name}"]


def test_norm_weight_is_a_distance_from_one():
    x = RNG.standard_normal((3, 10))
    assert np.allclose((df.norm_around_zero(x, np.zeros(10), 0.0) ** 2).mean(-1), 1.0)
    assert np.allclose(df.norm_around_zero(x, np.full(10, -1.0), 0.1), 0.0)
    assert np.allclose(df.norm_around_zero(np.full((1, 4), 1e-3), np.ones(4), 1.0), 2e-3 / np.sqrt(1 + 1e-6))   # eps in the root


def test_memory_equals_its_sum_over_tokens():
    """o_t = sum_s D_ts (q_t . k_s) v_s / max(|sum_s D_ts (q_t . k_s)|, 1) with D_ts = e^(f_{s+1} + .. + f_t + i_s): the scale m
    cancels but for the small constant in the denominator."""
    T, D, V = 9, 4, 6
    q, k, v = (RNG.standard_normal((T, n)) for n in (D, D, V))
    log_in, log_keep = RNG.standard_normal(T), -RNG.random(T)
    memory = df.MatrixMemory(D, V)
    for t in range(T):
        got = memory.step(q[t], k[t], v[t], log_in[t], log_keep[t])
        weight = np.array([math.exp(log_keep[s + 1:t + 1].sum() + log_in[s]) * (q[t] @ k[s]) for s in range(t + 1)])
        assert np.allclose(got, weight @ v[:t + 1] / max(abs(weight.sum()), 1.0), rtol=1e-4)


def test_memory_scale_starts_at_zero():
    """A first input gate below zero leaves m at f, not at i: the denominator's floor e^-m shows which."""
    memory = df.MatrixMemory(1, 1)
    out = memory.step(np.array([1.0]), np.array([1.0]), np.array([1.0]), -3.0, -0.5)
    assert memory.m == -0.5 and np.isclose(out[0], math.exp(-2.5) / (math.exp(0.5) + 1e-6))


def test_denominator_shows_only_beside_a_large_eps(monkeypatch):
    """The norm over a head takes every factor of its output away, up to eps: tests of the denominator use a large one."""
    cfg = config(11, 16, [mlstm(2, 6, 10)], (0, 1, 1))
    tensor, m, h = tensors(cfg, 4), cfg["layers"][0]["mixer"], RNG.standard_normal((7, 16))
    small, large = df.mlstm(h, m, tensor, 1e-9), df.mlstm(h, m, tensor, 1.0)
    step = df.MatrixMemory.step

    def no_floor(self, q, *a):
        out = step(self, q, *a)
        return out * max(abs(self.n @ q), math.exp(-self.m)) / abs(self.n @ q)
    monkeypatch.setattr(df.MatrixMemory, "step", no_floor)
    assert np.allclose(df.mlstm(h, m, tensor, 1e-9), small, atol=1e-4)
    assert np.abs(df.mlstm(h, m, tensor, 1.0) - large).max() > 0.05


def test_gates():
    m = {"gate_cap": 2.0}
    w = {"i": np.array([[100.0]]), "i.b": np.array([0.0]), "f": np.array([[0.0]]), "f.b": np.array([1.0])}
    log_in, log_keep = df.gates_of(np.array([[1.0]]), m, w.__getitem__)
    assert np.isclose(log_in[0, 0], 2.0)
    assert np.isclose(log_keep[0, 0], -math.log1p(math.exp(-2 * math.tanh(0.5))))
    assert np.allclose(df.log_sigmoid(np.array([-800.0, 0.0, 800.0])), [-800.0, -math.log(2), 0.0])


def test_sink_takes_its_share():
    p = df.sink_softmax(np.array([0.0, 0.0, 0.0]))
    assert np.allclose(p, 0.25)
    assert df.sink_softmax(np.array([-50.0, -60.0])).sum() < 1e-20
    assert np.isclose(df.sink_softmax(np.array([900.0, 0.0])).sum(), 1.0)


def test_chunks_count_from_position_zero():
    seen = [[j for j in range(10) if df.sees(i, j, 4)] for i in range(10)]
    assert seen[3] == [0, 1, 2, 3] and seen[4] == [4] and seen[9] == [8, 9]


def test_rotation_leaves_the_rest_and_depends_on_distance_only():
    rot = {"dims": 4, "base": 30.0}
    q, k = RNG.standard_normal((1, 7)), RNG.standard_normal((1, 7))
    assert np.allclose(df.rotate_first(q, [50], rot)[:, 4:], q[:, 4:])

    def score(p, j):
        return float((df.rotate_first(q, [p], rot) @ df.rotate_first(k, [j], rot).T)[0, 0])
    assert np.isclose(score(9, 4), score(105, 100)) and not np.isclose(score(9, 4), score(9, 5))
    one = np.zeros((1, 7)); one[0, 0] = 1
    r = df.rotate_first(one, [1], rot)[0]
    assert np.isclose(r[0], np.cos(1)) and np.isclose(r[2], np.sin(1))


def test_queries_share_their_groups_keys():
    cfg = config(11, 16, [attention(4, 2, 6, 5, 100, 0.4)], (0, 1, 1))
    tensor = tensors(cfg, 5)
    h = RNG.standard_normal((6, 16))
    out = df.attention(h, cfg["layers"][0]["mixer"], tensor, np.arange(6))
    heads = {"q": tensor("q"), "k": np.repeat(tensor("k").reshape(2, 6, 16), 2, axis=0).reshape(24, 16),
             "v": np.repeat(tensor("v").reshape(2, 5, 16), 2, axis=0).reshape(20, 16), "o": tensor("o")}
    alone = dict(cfg["layers"][0]["mixer"], kv_heads=4)
    assert np.allclose(out, df.attention(h, alone, heads.__getitem__, np.arange(6)))


def test_router_and_clamped_expert():
    best, w = df.choose(np.array([1.0, 3.0, 2.0, 3.0]), 2)
    assert best == [1, 3] and np.allclose(w, 0.5)
    best, w = df.choose(np.array([0.0, 2.0, 1.0]), 2)
    assert best == [1, 2] and np.isclose(w[0], 1 / (1 + math.exp(-1)))
    one = {"e.gate": np.array([[1.0]]), "e.up": np.array([[1.0]]), "e.down": np.array([[1.0]])}

    def expert(x, limit):
        return df.clamped_expert(np.array([x]), one.__getitem__, "e.", limit)[0]
    assert np.isclose(expert(5.0, 2.0), 2 / (1 + math.exp(-3.404)) * 3)
    assert np.isclose(expert(-5.0, 2.0), -5 / (1 + math.exp(8.51)) * -1)   # the gate has no lower limit
    assert np.isclose(expert(0.5, 2.0), 0.5 / (1 + math.exp(-0.851)) * 1.5)


def test_layer_runs():
    assert df.layer_runs(SMALL) == [(0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (1, 2), (2, None), (3, None),
                                    (4, None)]
    assert df.layer_runs(ODD) == [(0, 0), (1, None), (2, None), (3, None)]


@pytest.mark.parametrize("cfg", [SMALL, ODD])
def test_causal_and_every_part_matters(cfg):
    w = df.random_weights(cfg, 9)
    ids = RNG.integers(0, cfg["vocab"], 14)
    base = df.DimesunOracle(cfg, w).forward(ids)
    other = ids.copy(); other[9] = (other[9] + 1) % cfg["vocab"]
    changed = np.abs(df.DimesunOracle(cfg, w).forward(other) - base).max(axis=1)
    assert (changed[:9] == 0).all() and (changed[9:] > 1e-6).all()
    for name in w:   # a tensor that no output depends on would be a mechanism the forward pass leaves out
        if ".mlp.e" in name:
            continue
        by, ramp = (-3.0, 9.0) if ".router" in name else (1.3, 0.05)   # where one expert is chosen only another choice shows
        v = dict(w); v[name] = v[name] * by + ramp * np.arange(w[name].size).reshape(w[name].shape) / w[name].size
        assert np.abs(df.DimesunOracle(cfg, v).forward(ids) - base).max() > 1e-7, name


def planted(cfg, mistake):
    """The same configuration with one thing wrong: an edited configuration, or a patch of the oracle."""
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        m = l["mixer"]
        if "mask" in m:
            m["mask"]["size"] += {"chunk + 1": 1, "chunk - 1": -1}.get(mistake, 0)
            m["rot"]["base"] *= 1.5 if mistake == "rotation" else 1
        elif mistake == "cap":
            m["gate_cap"] = 2.0
        if l["mlp"] and mistake == "limit":
            l["mlp"]["expert"]["limit"] = 100.0
    if mistake == "times":
        out["loop"]["times"] = max(1, out["loop"]["times"] - 1)
    if mistake == "multiplier":
        out["residual_mult"] *= 0.8
    return out


MISTAKES = ["chunk + 1", "chunk - 1", "rotation", "limit", "multiplier", "no sink", "norm without one", "no loop vector"]


@pytest.mark.parametrize("name,mistake", [(name, m) for name in ("small", "odd", "wide") for m in MISTAKES] +
                         [("small", "cap"), ("small", "lost state"), ("small", "times"), ("odd", "weights over all experts"),
                          ("wide", "cap"), ("wide", "lost state"), ("wide", "times")])
def test_mistakes_show_in_the_logits(monkeypatch, name, mistake):
    """The configurations of the GPU tests with their weights: a planted mistake moves some logits by more than the limit."""
    cfg = {"small": SMALL, "odd": ODD, "wide": WIDE}[name]
    n = {"small": 75, "odd": 75, "wide": 150}[name]
    w = df.random_weights(cfg, 100 + len(name))
    right = Truth(df.DimesunOracle(cfg, w), n)
    if mistake == "no sink":
        monkeypatch.setattr(df, "sink_softmax", lambda s: np.exp(s - s.max()) / np.exp(s - s.max()).sum())
    elif mistake == "lost state":
        step = df.MatrixMemory.step

        def forgetful(self, *a):
            self.count = getattr(self, "count", 0) + 1
            if self.count == 41:
                self.S[:], self.n[:], self.m = 0, 0, 0.0
            return step(self, *a)
        monkeypatch.setattr(df.MatrixMemory, "step", forgetful)
    elif mistake == "weights over all experts":
        choose = df.choose

        def all_of_them(z, top):
            best, _ = choose(z, top)
            return best, (np.exp(z - z.max()) / np.exp(z - z.max()).sum())[best]
        monkeypatch.setattr(df, "choose", all_of_them)
    elif mistake == "norm without one":
        monkeypatch.setattr(df, "norm_around_zero", lambda x, v, eps: df.unit_rms(x, eps) * v)
    elif mistake == "no loop vector":
        w = dict(w); w["loop.step"] = w["loop.step"] * 0
    err = row_errors(df.DimesunOracle(planted(cfg, mistake), w).forward(right.ids), right.logits)
    assert (err > 1.5 * right.limits["bfloat16"]).any(), (err / right.limits["bfloat16"]).max()


def test_greedy_repeats_the_argmax():
    cfg = config(31, 24, [mlstm(2, 4, 6, mlp=moe(3, 2, 8)), attention(2, 1, 6, 4, 5, 0.5)], (0, 2, 2))
    oracle = df.DimesunOracle(cfg, df.random_weights(cfg, 13))
    out = df.greedy(oracle, [1, 2, 3], 4)
    logits = oracle.forward([1, 2, 3] + out)
    assert out == [int(logits[2 + i].argmax()) for i in range(4)]
