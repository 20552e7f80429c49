"""The plain Nafevik functions against numbers worked out by hand, and the loader's refusals (no GPU)."""
import json
import math
import subprocess

import numpy as np
import pytest

import nafevik_ref as R
import nafevik_util as U
from cera_amd import _build, llama_api


def test_visible_is_causal_and_stays_in_its_chunk():
    v = R.visible(7, 3)
    assert [list(np.flatnonzero(r)) for r in v] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert R.visible(4, None).sum() == 10


def test_conv_reads_the_newest_row_with_its_last_tap():
    h, w = np.array([[1.0], [10.0], [100.0]]), np.array([[2.0, 3.0, 5.0]])
    assert R.causal_conv(h, w)[:, 0].tolist() == [5.0, 53.0, 532.0]


def test_rotation_pairs_neighbours_and_leaves_the_rest():
    x = np.array([1.0, 0.0, 0.0, 1.0, 7.0]).reshape(1, 1, 5)
    y = R.rotate(x, [2], {"dims": 4, "base": 16.0})[0, 0]      # frequencies 1 and 1/4
    assert np.allclose(y, [math.cos(2), math.sin(2), -math.sin(0.5), math.cos(0.5), 7.0])


def test_yarn_frequencies():
    f, mag = R.rotary_frequencies({"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "original": 2 * math.pi * 1000, "fast": 1000.0, "slow": 1.0}})
    # turns over the original length: 1000 at pair 0 (lo = 0), 1 at dimension 8 ln(1000) / (2 ln 100) = 6 (hi)
    ramp = np.array([0, 1 / 6, 2 / 6, 3 / 6])
    base = 100.0 ** (-np.arange(4) / 4)
    assert np.allclose(f, base / 4 * ramp + base * (1 - ramp)) and math.isclose(mag, 0.1 * math.log(4) + 1)


def test_attention_weights_are_not_normalised():
    q = k = np.zeros((3, 1, 2))
    v = np.ones((3, 1, 1))
    assert np.allclose(R.sigmoid_attention(q, k, v, 1.0, np.array([0.0]), 2)[:, 0, 0], [0.5, 1.0, 0.5])


def test_layer_runs_and_pass_starts():
    assert R.layer_runs({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert R.layer_runs({"layers": [0] * 2}) == [(0, None), (1, None)]


def _open_error(path):
    with pytest.raises(llama_api.BackendError) as e:
        llama_api.HipLlama(str(path), 64)
    return str(e.value)


def test_loader_refuses_what_it_cannot_run(tmp_path):
    cfg = U.CONFIGS["plain"]
    w = R.random_model(cfg, 1)
    bad = json.loads(json.dumps(cfg))
    bad["architecture"] = "Other"
    assert "unsupported architecture" in _open_error(U.save(tmp_path / "arch", bad, w))
    bad = json.loads(json.dumps(cfg))
    bad["layers"][1]["type"] = "convolution"
    assert "layers[1].type" in _open_error(U.save(tmp_path / "type", bad, w))
    bad = json.loads(json.dumps(cfg))
    bad["layers"][1]["mlp"]["kind"] = "routed"
    assert "layers[1].mlp.kind" in _open_error(U.save(tmp_path / "kind", bad, w))
    bad = json.loads(json.dumps(cfg))
    del bad["layers"][0]["mixer"]["vdim"]
    assert "missing layers[0].mixer.vdim" in _open_error(U.save(tmp_path / "key", bad, w))
    bad = json.loads(json.dumps(cfg))
    bad["loop"] = {"start": 1, "stop": 5, "times": 2}
    assert "loop" in _open_error(U.save(tmp_path / "loop", bad, w))
    less = {k: v for k, v in w.items() if k != "l1.mix.pb"}
    assert "l1.mix.pb is missing" in _open_error(U.save(tmp_path / "tensor", cfg, less))
    other = dict(w, **{"head": w["head"][:-1]})
    assert "tensor head has shape" in _open_error(U.save(tmp_path / "shape", cfg, other))
    assert "expected BF16" in _open_error(U.save(tmp_path / "dtype", cfg, w, {"embed": "F16"}))
    (tmp_path / "none").mkdir()
    assert "config.json" in _open_error(tmp_path / "none")
    d = U.save(tmp_path / "json", cfg, w)
    (d / "config.json").write_text('{"architecture": "Nafevik",}')
    assert "JSON" in _open_error(d)
    d = U.save(tmp_path / "cut", cfg, w)
    raw = (d / "model.safetensors").read_bytes()
    (d / "model.safetensors").write_bytes(raw[:-2])
    assert "offsets outside the file" in _open_error(d)


def test_inspect_lists_a_model_directory(tmp_path):
    cfg = U.CONFIGS["plain"]
    d = U.save(tmp_path / "m", cfg, R.random_model(cfg, 2))
    r = subprocess.run([str(_build.CLI_BIN), "inspect", "--model", str(d)], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0 and '"architecture": "Nafevik"' in r.stdout
    assert [line.split()[:2] for line in r.stdout.splitlines() if line.startswith("l1.mix.o")] == [["l1.mix.o", "BF16"]]


def test_trace_runner_arguments():
    assert _build.TRACE_BIN.exists(), "cera-trace missing: run __graft_entry__.build()"
    run = lambda *a: subprocess.run([str(_build.TRACE_BIN), *a], capture_output=True, text=True, input="", timeout=60)  # noqa: E731
    assert run("--model", "/nowhere").returncode == 2
    assert run("--model", "/nowhere", "--out", "/tmp", "--dtype", "int8").returncode == 2
    r = run("--model", "/nowhere", "--out", "/tmp")
    assert r.returncode == 1 and "config.json" in r.stderr
