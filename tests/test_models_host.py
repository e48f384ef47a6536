"""The model registry without a GPU: configurations that are refused, with the reason, before any device work."""
import copy
import json
import os
import stat

import numpy as np
import pytest

from oracle import takosun_forward as tf
from tests import dimesun_fixture
from tests.takosun_fixture import SMALL, write_model

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def refused(pkg, cfg, match):
    with pytest.raises(pkg.capi.A81W41Error, match=match):
        pkg.Model.random(cfg, 16)


def edit(path, value, of=SMALL):
    cfg = copy.deepcopy(of)
    at = cfg
    for k in path[:-1]:
        at = at[k]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return cfg


@pytest.mark.parametrize("path,value,match", [
    (["width"], None, "missing key 'width'"),
    (["norm", "groups"], 7, "multiple of norm.groups"),
    (["layers", 0, "type"], "window_attention", "unknown type"),
    (["layers", 0, "mixer", "rot", "dims"], 6, "rot.dims must equal rot_dim"),
    (["layers", 1, "mixer", "kv_from"], 1, "kv_from must name an earlier layer"),
    (["layers", 3, "mixer", "kv_from"], 1, "of its own"),
    (["layers", 1, "mixer", "kv_rank"], 48, "of the same sizes"),
    (["layers", 1, "mixer", "rot", "base"], 501.0, "of the same sizes"),
    (["layers", 0, "mlp", "kind"], "sparse", "unknown feed-forward"),
    (["layers", 0, "mlp", "router", "top"], 6, "router out of range"),
    (["layers"], [], "no layers"),
    (["vocab"], 2.5, "whole number"),
])
def test_bad_configurations_are_refused(pkg, path, value, match):
    refused(pkg, edit(path, value), match)


@pytest.mark.parametrize("path,value,match", [
    (["residual_mult"], None, "missing key 'residual_mult'"),
    (["norm", "eps"], -1.0, "norm.eps"),
    (["layers", 1, "type"], "latent_attention", "layer 1: unknown type"),
    (["layers", 1, "mixer", "kv_heads"], 4, "multiple of kv_heads"),
    (["layers", 1, "mixer", "rot", "dims"], 26, "rot.dims"),
    (["layers", 1, "mixer", "rot", "dims"], 3, "rot.dims"),
    (["layers", 1, "mixer", "mask"], None, "missing key 'mask'"),
    (["layers", 1, "mixer", "mask", "size"], 0, "'size' is out of range"),
    (["layers", 0, "mixer", "gate_cap"], 0.0, "gate_cap"),
    (["layers", 0, "mixer", "vdim"], None, "missing key 'vdim'"),
    (["layers", 0, "mlp", "kind"], "dense", "unknown feed-forward"),
    (["layers", 0, "mlp", "router", "top"], 6, "router out of range"),
    (["layers", 0, "mlp", "expert", "limit"], None, "missing key 'limit'"),
    (["loop", "stop"], 6, "loop.start"),
    (["loop", "start"], 4, "loop.start"),
    (["loop", "times"], 0, "'times' is out of range"),
    (["layers"], [], "no layers"),
])
def test_bad_dimesun_configurations_are_refused(pkg, path, value, match):
    refused(pkg, edit(path, value, dimesun_fixture.SMALL), match)


def test_unknown_architecture(pkg):
    with pytest.raises(ValueError, match="Takosun"):
        pkg.Model.random({"architecture": "Nobody"}, 16)


def test_folder_errors(pkg, tmp_path):
    with pytest.raises(FileNotFoundError):
        pkg.Model.load(str(tmp_path), 16)
    (tmp_path / "config.json").write_text(json.dumps(SMALL))
    with pytest.raises(pkg.capi.A81W41Error, match="cannot open"):
        pkg.Model.load(str(tmp_path), 16)
    (tmp_path / "model.safetensors").write_bytes(b"\xff" * 20)
    with pytest.raises(pkg.capi.A81W41Error, match="header is longer"):
        pkg.Model.load(str(tmp_path), 16)
    with pytest.raises(pkg.capi.A81W41Error, match="dtype"):
        pkg.Model.load(str(tmp_path), 16, "float64")


def test_qwen3_is_registered_and_has_no_32_bit_path(pkg, tmp_path):
    cfg = {"architecture": "Qwen3", "num_hidden_layers": 1, "hidden_size": 64, "num_attention_heads": 1, "num_key_value_heads": 1,
           "intermediate_size": 64, "vocab_size": 64, "rope_theta": 1e6, "rms_norm_eps": 1e-6}
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(pkg.capi.A81W41Error) as e:
        pkg.Model.load(str(tmp_path), 16, "float32")
    assert e.value.status == pkg.capi.ERR_UNSUPPORTED


def test_fixture_round_trip(tmp_path):
    w = tf.random_weights(SMALL, 1)
    write_model(str(tmp_path), SMALL, w)
    from safetensors import safe_open  # an independent reader of the same format
    with safe_open(str(tmp_path / "model.safetensors"), "pt") as f:
        assert set(f.keys()) == set(w)
        assert np.array_equal(f.get_tensor("l2.mix.dkv").float().numpy(), w["l2.mix.dkv"])
        assert np.array_equal(f.get_tensor("l0.mlp.table").numpy(), w["l0.mlp.table"])


def test_trace_run_is_executable():
    assert os.stat(os.path.join(ROOT, "bin", "trace_run")).st_mode & stat.S_IXUSR
