"""The Takosun oracle against properties that the mathematics fixes (no GPU)."""
import numpy as np
import pytest

from oracle import takosun_forward as tf
from tests.takosun_fixture import ODD, SMALL, config, dense, layer, mixer

RNG = np.random.default_rng(3)


def test_grouped_norm_scales_every_part_alone():
    x = RNG.standard_normal((4, 12)) * np.repeat([1.0, 100.0, 0.01], 4)
    y = tf.grouped_rms_norm(x, np.ones(12), 0.0, 3)
    assert np.allclose((y.reshape(4, 3, 4) ** 2).mean(-1), 1.0)
    assert np.allclose(tf.grouped_rms_norm(x, np.ones(12), 0.5, 1), tf.rms_norm(x, np.ones(12), 0.5))
    # eps is inside the root
    assert np.allclose(tf.rms_norm(np.zeros((1, 3)) + 1e-3, np.ones(3), 1.0), 1e-3 / np.sqrt(1 + 1e-6))


def test_rotation_keeps_norms_and_depends_on_distance_only():
    q, k = RNG.standard_normal((1, 8)), RNG.standard_normal((1, 8))
    def score(p, j):
        return float((tf.rotate_half(q, [p], 30.0) @ tf.rotate_half(k, [j], 30.0).T)[0, 0])
    assert np.isclose(np.linalg.norm(tf.rotate_half(q, [77], 30.0)), np.linalg.norm(q))
    assert np.isclose(score(9, 4), score(105, 100)) and not np.isclose(score(9, 4), score(9, 5))
    assert np.allclose(tf.rotate_half(q, [0], 30.0), q)
    # component i turns with i + R/2, the first pair by the position itself
    one = np.zeros((1, 8)); one[0, 0] = 1
    r = tf.rotate_half(one, [1], 30.0)[0]
    assert np.isclose(r[0], np.cos(1)) and np.isclose(r[4], np.sin(1)) and np.allclose(np.delete(r, [0, 4]), 0)


def test_one_key_gives_its_value_and_absorbed_equals_formed():
    m = mixer(2, 6, 4, 5, 7, 9, 0.3)
    w = tf.random_weights(config(11, 16, 4, [layer(m, dense(8))]), 5)
    def tensor(n):
        return np.asarray(w["l0.mix." + n], np.float64)
    h = RNG.standard_normal((6, 16))
    lat = tf.latent_of(h, m, tensor, 1e-5, np.arange(6))
    out = tf.latent_attention(h, m, tensor, 1e-5, np.arange(6), lat)
    gate = 1 / (1 + np.exp(-(h @ tensor("g").T)))
    v0 = (lat[0][:1] @ tensor("uv").T).reshape(2, 5) * gate[0][:, None]
    assert np.allclose(out[0], v0.reshape(-1) @ tensor("o").T)
    # the last row with the up-projections moved into query and output
    q = (tf.rms_norm(h @ tensor("dq").T, tensor("dq.norm"), 1e-5) @ tensor("uq").T).reshape(6, 2, 10)
    heads = []
    for a in range(2):
        uk, uv = tensor("uk")[a * 6:a * 6 + 6], tensor("uv")[a * 5:a * 5 + 5]
        s = (q[5, a, :6] @ uk) @ lat[0].T + tf.rotate_half(q[5:6, a, 6:], [5], m["rot"]["base"])[0] @ lat[1].T
        p = np.exp(s * m["scale"]); p /= p.sum()
        heads.append(uv @ (p @ lat[0]) * gate[5, a])
    assert np.allclose(out[5], np.concatenate(heads) @ tensor("o").T)


def test_experts_count_equally_and_follow_the_table():
    cfg = SMALL
    w = {k: np.asarray(v, np.float64) for k, v in tf.random_weights(cfg, 7).items()}
    h = RNG.standard_normal((1, cfg["width"]))
    def tensor(n):
        return w["l0.mlp." + n]
    got = tf.table_moe(h, [42], cfg["layers"][0]["mlp"], tensor)
    e = w["l0.mlp.table"][42].astype(int)
    want = (tf.gated_ff(h, tensor, f"e{e[0]}.") + tf.gated_ff(h, tensor, f"e{e[1]}.")) / 2 + tf.gated_ff(h, tensor, "shared.")
    assert np.allclose(got, want) and e[0] != e[1]


@pytest.mark.parametrize("cfg", [SMALL, ODD])
def test_causal_and_every_part_matters(cfg):
    w = tf.random_weights(cfg, 9)
    o = tf.TakosunOracle(cfg, w)
    ids = RNG.integers(0, cfg["vocab"], 14)
    base = o.forward(ids)
    other = ids.copy(); other[9] = (other[9] + 1) % cfg["vocab"]
    changed = np.abs(o.forward(other) - base).max(axis=1)
    assert (changed[:9] == 0).all() and (changed[9:] > 1e-6).all()
    for name in w:   # a tensor that no output depends on would be a mechanism the forward pass leaves out
        if name.endswith("table") or ".e" in name:
            continue
        v = dict(w); v[name] = v[name] * 1.3 + 0.05
        assert np.abs(tf.TakosunOracle(cfg, v).forward(ids) - base).max() > 1e-7, name


def test_depth_average_of_the_last_state_alone_is_a_plain_stack():
    cfg = config(31, 24, 2, [layer(mixer(2, 4, 2, 4, 6, 8, 0.4), dense(12))] * 2)
    w = tf.random_weights(cfg, 13)
    for i in range(2):
        w[f"l{i}.dwa"] = np.eye(i + 2)[-1]
    states = []
    tf.TakosunOracle(cfg, w).forward([1, 2, 3], states)
    w2 = dict(w); w2["l1.dwa"] = np.array([0.0, 1.0, 0.0])   # what goes on is the first layer's result
    again = []
    tf.TakosunOracle(cfg, w2).forward([1, 2, 3], again)
    assert np.allclose(again[1], states[0])
