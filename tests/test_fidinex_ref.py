"""The plain Fidinex functions against numbers worked out by hand, and the loader's refusals (no GPU)."""
import json
import math
import subprocess

import numpy as np
import pytest

import fidinex_ref as R
import fidinex_util as U
from cera_amd import _build, llama_api


def test_rms_norm_has_eps_inside_the_root():
    assert np.allclose(R.rms_norm(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), 12.5), [[3 / 5, 8 / 5]])


def test_rotation_pairs_neighbours_and_leaves_the_rest():
    x = np.array([1.0, 0.0, 0.0, 1.0, 7.0]).reshape(1, 1, 5)
    y = R.rotate_pairs(x, [2], 16.0, 4)[0, 0]      # frequencies 1 and 1/4
    assert np.allclose(y, [math.cos(2), math.sin(2), -math.sin(0.5), math.cos(0.5), 7.0])


def test_query_temperature_steps_behind_every_nth_position():
    f = R.query_temperature(range(8), {"coef": 0.5, "every": 4})
    assert np.allclose(f, [1, 1, 1] + [1 + 0.5 * math.log(2)] * 4 + [1 + 0.5 * math.log(3)])
    assert R.query_temperature(range(3), None).tolist() == [1, 1, 1]


def test_the_sink_takes_its_share_and_has_no_value():
    s = np.array([[math.log(2.0), 99.0], [0.0, math.log(3.0)]])
    w = R.sink_softmax(s, math.log(4.0))
    assert np.allclose(w, [[2 / 6, 0], [1 / 8, 3 / 8]])


def test_values_mix_with_the_first_layers():
    assert R.mix_values(np.array([2.0]), np.array([10.0]), 0.25).tolist() == [4.0]


def test_streams_are_written_from_the_old_ones():
    xs, mix = [np.array([1.0]), np.array([10.0])], np.array([[2.0, 3.0], [5.0, 7.0]])      # [from, to]
    assert R.read_streams(xs, np.array([4.0, 0.5])).tolist() == [9.0]
    out = R.write_streams(xs, np.array([100.0]), np.array([1.0, -1.0]), mix)
    assert [o.tolist() for o in out] == [[2 + 50 + 100], [3 + 70 - 100]]


def test_squared_relu():
    w = {"up": np.array([[1.0], [-1.0]]), "down": np.array([[1.0, 100.0]])}
    assert R.dense_ff(np.array([[3.0]]), "", w).tolist() == [[9.0]]


def test_absorbed_and_expanded_latent_attention_are_the_same_numbers():
    rng = np.random.default_rng(1)
    q, uk, c = rng.standard_normal(5), rng.standard_normal((5, 9)), rng.standard_normal(9)
    assert math.isclose(q @ (uk @ c), (uk.T @ q) @ c)


def _open_error(path):
    with pytest.raises(llama_api.BackendError) as e:
        llama_api.HipLlama(str(path), 64)
    return str(e.value)


def test_loader_refuses_what_it_cannot_run(tmp_path):
    cfg = U.CONFIGS["mixed"]
    w = U.random_model(cfg, 1)

    def broken(name, edit):
        bad = json.loads(json.dumps(cfg))
        edit(bad)
        return _open_error(U.save(tmp_path / name, bad, w))

    assert "layers[1].type" in broken("type", lambda c: c["layers"][1].update(type="convolution"))
    assert "layers[1].mlp.kind" in broken("kind", lambda c: c["layers"][1]["mlp"].update(kind="routed"))
    assert "missing layers[0].mixer.kv_rank" in broken("key", lambda c: c["layers"][0]["mixer"].pop("kv_rank"))
    assert "missing layers[1].mixer.kv_heads" in broken("groups", lambda c: c["layers"][1]["mixer"].pop("kv_heads"))
    assert "q_temp.every" in broken("temp", lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0))
    assert "v_mix must be" in broken("vmix", lambda c: c["layers"][1]["mixer"].update(v_mix=3))
    assert "missing norm" in broken("norm", lambda c: c.pop("norm"))
    for name in ("l0.mix.dkv.norm", "l1.mix.sink", "l3.mix.vmix", "l1.hc2.mix", "final.norm"):
        less = {k: v for k, v in w.items() if k != name}
        assert name + " is missing" in _open_error(U.save(tmp_path / ("no_" + name), cfg, less))
    assert "tensor l0.mix.uk has shape" in _open_error(U.save(tmp_path / "shape", cfg, dict(w, **{"l0.mix.uk": w["l0.mix.uk"][:-1]})))
    assert "expected BF16" in _open_error(U.save(tmp_path / "dtype", cfg, w, {"embed": "F16"}))


def test_inspect_lists_a_model_directory(tmp_path):
    cfg = U.CONFIGS["plain"]
    d = U.save(tmp_path / "m", cfg, U.random_model(cfg, 2))
    r = subprocess.run([str(_build.CLI_BIN), "inspect", "--model", str(d)], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0 and '"architecture": "Fidinex"' in r.stdout
    assert [line.split()[:3] for line in r.stdout.splitlines() if line.startswith("l1.mix.vmix")] == [["l1.mix.vmix", "BF16", "[]"]]
