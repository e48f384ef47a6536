"""The model interface over both model families: Qwen3 through the registry, and the generation command."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from oracle import takosun_forward as tf
from tests.qwen3_fixture import TINY, arrays, build, write_reference_tree
from tests.takosun_fixture import SMALL, write_model

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def qwen_dir(synth, tmp_path_factory):
    root = str(tmp_path_factory.mktemp("qwen"))
    write_reference_tree(root, arrays(synth, TINY, 900), TINY)
    with open(os.path.join(root, "config.json"), "w") as f:
        json.dump({"architecture": "Qwen3", "num_hidden_layers": TINY["n_layers"], "hidden_size": TINY["hidden"],
                   "num_attention_heads": TINY["n_q_heads"], "num_key_value_heads": TINY["n_kv_heads"],
                   "intermediate_size": TINY["intermediate"], "vocab_size": TINY["vocab"], "rope_theta": 1e6, "rms_norm_eps": 1e-6}, f)
    return root


def test_qwen3_through_the_registry(pkg, synth, ora, qwen_dir):
    direct = pkg.Qwen3Model(**TINY)
    build(synth, ora, TINY, 900, gpu_model=direct)
    model = pkg.Model.load(qwen_dir, TINY["max_seq"])
    ids = [3, 99, 500, 7, 7, 123, 45, 256, 31, 8]
    assert np.array_equal(model.forward(ids)[0], direct.forward(ids))
    assert np.array_equal(model.forward([17])[0], direct.forward([17]))
    model.reset(), direct.reset()
    # several wanted places of one pass are what shorter prompts end with
    got = model.forward(ids, [2, 6, 9])
    for row, n in zip(got, (3, 7, 10)):
        direct.reset()
        want = direct.forward(ids[:n])
        assert np.linalg.norm(row - want) <= 5e-3 * np.linalg.norm(want)
    model.reset(), direct.reset()
    assert np.array_equal(model.generate_greedy(ids, 12)[0], direct.generate_greedy(ids, 12)[0])
    sizes = model.resident_bytes()
    assert sizes["cache"] == 2 * 2 * TINY["n_layers"] * TINY["n_kv_heads"] * TINY["max_seq"] * 128 and sizes["weights"] > 0


def test_trace_run_on_qwen3(pkg, synth, ora, qwen_dir, tmp_path):
    direct = pkg.Qwen3Model(**TINY)
    build(synth, ora, TINY, 900, gpu_model=direct)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": [3, 99, 500], "want": [2]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": [7], "want": [0]}], "end": ["x"]}]
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", qwen_dir, "--out", str(tmp_path), "--max-tokens", "16"]
    text = "".join(json.dumps(s) + "\n" for s in steps)
    assert subprocess.run(cmd + ["--dtype", "float32"], input=text, capture_output=True, text=True, timeout=100).returncode == 3
    r = subprocess.run(cmd + ["--dtype", "bfloat16"], input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    for k, ids in enumerate(([3, 99, 500], [7])):
        assert np.array_equal(np.fromfile(tmp_path / f"{k}.f32", "<f4"), direct.forward(ids))


def test_generate_command(pkg, tmp_path):
    w = tf.random_weights(SMALL, 77)
    write_model(str(tmp_path), SMALL, w)
    prompt = [5, 17, 3, 101, 64]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", str(tmp_path), "--dtype", "float32", "--tokens",
                        ",".join(map(str, prompt)), "--new", "9"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split(",")] == tf.greedy(tf.TakosunOracle(SMALL, w), prompt, 9)


def test_two_models_side_by_side(pkg, tmp_path):
    """Sessions share nothing: interleaved calls give what each gives alone."""
    w = tf.random_weights(SMALL, 5)
    write_model(str(tmp_path), SMALL, w)
    oracle = tf.TakosunOracle(SMALL, w)
    rng = np.random.default_rng(2)
    seqs = [rng.integers(0, SMALL["vocab"], n) for n in (30, 21)]
    models = [pkg.Model.load(str(tmp_path), 40, "float32") for _ in seqs]
    got = [[], []]
    for at in range(0, 30, 5):
        for k, ids in enumerate(seqs):
            part = ids[at:at + 5]
            if len(part):
                got[k].append(models[k].forward(part, range(len(part))))
    for k, ids in enumerate(seqs):
        want = oracle.forward(ids)
        err = np.linalg.norm(np.concatenate(got[k]) - want, axis=1) / np.linalg.norm(want, axis=1)
        assert err.max() <= 3e-5
