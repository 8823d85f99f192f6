"""CPU-side checks of the Rapitar design: the plain forward pass the GPU tests compare with, and what the library does with
a model directory before it needs a GPU (config.json, safetensors headers, the registry)."""
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest

import kagalorn_case as KC
import rapitar_case as RC
import rapitar_oracle as R
from blok_amd.lib import KxModelShape, KxOpenOptions, kx

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EXEC = os.path.join(ROOT, "blok_amd", "kx-kimi-exec")
CFG = RC.config([RC.mamba2(mlp=RC.dense()), RC.wkv(mlp=RC.moe()), RC.latent(mlp=None), RC.latent(mlp=RC.moe(experts=3, top=3))], vocab=40, width=32)


def test_state_space_recurrence_is_its_sum_and_carries_its_state():
    r = np.random.default_rng(0)
    x, b, c, dt, a = r.standard_normal((9, 3)), r.standard_normal((9, 4)), r.standard_normal((9, 4)), r.uniform(0, 1, 9), r.uniform(0.3, 1, 9)
    y, s = R.ssd(x, b, c, dt, a, 0.7)
    for t in range(9):
        want = 0.7 * x[t] + sum(np.prod(a[j + 1:t + 1]) * dt[j] * (b[j] @ c[t]) * x[j] for j in range(t + 1))
        assert np.allclose(y[t], want)
    y1, s1 = R.ssd(x[:4], b[:4], c[:4], dt[:4], a[:4], 0.7)
    y2, s2 = R.ssd(x[4:], b[4:], c[4:], dt[4:], a[4:], 0.7, s1)
    assert np.allclose(np.concatenate([y1, y2]), y) and np.allclose(s2, s)


def test_time_mixing_recurrence_is_its_sum_and_the_bonus_is_the_current_tokens():
    r = np.random.default_rng(1)
    q, k, v, w, u = r.standard_normal((8, 4)), r.standard_normal((8, 4)), r.standard_normal((8, 4)), r.uniform(0.2, 1, (8, 4)), r.standard_normal(4)
    o, _ = R.wkv(q, k, v, w, u)
    for t in range(8):
        want = (q[t] * u * k[t]).sum() * v[t] + sum((q[t] * np.prod(w[j + 1:t], 0) * k[j]).sum() * v[j] for j in range(t))
        assert np.allclose(o[t], want)


def test_shifted_mix_convolution_and_norms():
    h = np.array([[1.0, 2.0], [3.0, 5.0]])
    assert np.allclose(R.shifted_mix(h, np.array([1.0, 0.5])), [[0.0, 1.0], [1.0, 3.5]])
    y = R.causal_conv(np.arange(12.0).reshape(6, 2), np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]]), np.array([0.5, 0.0]))
    assert y[0, 0] == 0.5 and y[1, 0] == 200.5 and y[2, 0] == 420.5 and y[3, 0] == 642.5
    x = np.array([[3.0, 4.0, 0.0, 0.5]])
    assert np.allclose(R.grouped_rms(x, 2, 0.0), [[3 / np.sqrt(12.5), 4 / np.sqrt(12.5), 0, np.sqrt(2)]])
    assert np.allclose(R.norm_about_one(x, np.array([1.0, 0, 0, -1.0]), 0.0) * np.sqrt(np.mean(x * x)), [[6.0, 4.0, 0.0, 0.0]])


def test_rotation_keeps_relative_positions_and_passes_the_rest():
    r = np.random.default_rng(2)
    a, b = r.standard_normal(10), r.standard_normal(10)
    turn = lambda x, p: R.rotate_half(x[None], np.array([float(p)]), 6, 50.0)[0]
    assert np.allclose(turn(a, 9) @ turn(b, 4), turn(a, 25) @ turn(b, 20)) and np.allclose(turn(a, 7)[6:], a[6:]) and np.allclose(turn(a, 0), a)
    assert np.allclose(turn(np.eye(10)[0], 1.3)[[0, 3]], [np.cos(1.3), np.sin(1.3)])       # dimension 0 goes with dimension 3


def test_sink_takes_its_share_and_routing_its_order():
    v = np.ones((3, 2))
    out = R.sink_attention(np.zeros((3, 4)), np.zeros((3, 4)), v, 1.0, np.log(2.0))
    assert np.allclose(out[:, 0], [1 / 3, 2 / 4, 3 / 5])
    ids, w = R.route(np.array([[1.0, 3.0, 3.0, 0.0]]), 3)
    assert list(ids[0]) == [1, 2, 0] and np.allclose(w[0], np.exp([3, 3, 1]) / np.exp([3, 3, 1]).sum())
    assert abs(R.gelu_tanh(np.array(1.0)) - 0.841192) < 1e-6


def _probe(path):
    shape = KxModelShape()
    rc = kx().kx_model_probe(str(path).encode(), C.byref(shape))
    return rc, shape, kx().kx_last_error().decode()


def _open_error(path, **opt):
    o = KxOpenOptions()
    assert kx().kx_open_options_default(C.byref(o)) == 0
    for k, v in opt.items():
        setattr(o, k, v)
    m = C.c_void_p()
    assert kx().kx_model_open(str(path).encode(), C.byref(o), C.byref(m)) != 0 and not m
    return kx().kx_last_error().decode()


def test_registry_knows_the_design_by_its_config(tmp_path):
    KC.write(tmp_path / "m", CFG, RC.weights(CFG, 1))
    rc, shape, err = _probe(tmp_path / "m")
    assert rc == 0, err
    assert (shape.design, shape.n_layers, shape.hidden, shape.vocab) == (b"Rapitar", 4, 32, 40)


@pytest.mark.parametrize("edit, message", [
    (lambda c: c.pop("vocab"), "model.vocab"),
    (lambda c: c["norm"].pop("eps"), "norm.eps"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="mamba"), "layers[0].type is mamba"),
    (lambda c: c["layers"][0]["mixer"].update(groups=4), "6 heads in 4 groups"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=7), "7 norm_groups"),
    (lambda c: c["layers"][0]["mixer"].update(state=513), "state=513"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "layers[0].mixer.conv"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "kind is glu"),
    (lambda c: c["layers"][1]["mixer"].update(dim=0), "layers[1].mixer.dim"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=8), "8 of 7 experts"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(experts=2000), "2000 experts"),
    (lambda c: c["layers"][1]["mlp"].pop("expert"), "layers[1].mlp.expert"),
    (lambda c: c["layers"][2]["mixer"].pop("rot"), "layers[2].mixer.rot"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=13), "13 of 12"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(base=0), "base 0"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=3000), "kv_rank=3000"),
    (lambda c: c["layers"][2]["mixer"].pop("scale"), "layers[2].mixer.scale"),
])
def test_configuration_errors_name_the_field(tmp_path, edit, message):
    cfg = json.loads(json.dumps(CFG))
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    rc, _, err = _probe(tmp_path)
    assert rc != 0 and message in err, err


def test_weight_files_are_checked_before_anything_is_allocated(tmp_path):
    w = RC.weights(CFG, 1)
    for gone in ("l1.mlp.e6.down", "l1.mix.w1", "l0.mix.conv.b", "l3.mix.sink", "l2.norm1"):
        path = KC.write(tmp_path / "m", CFG, {k: v for k, v in w.items() if k != gone})
        assert "missing tensor: " + gone in _open_error(path)
    path = KC.write(tmp_path / "m", CFG, dict(w, **{"l0.mix.in": w["l0.mix.in"][:-1]}))
    assert "tensor l0.mix.in is bf16" in _open_error(path)
    path = KC.write(tmp_path / "m", CFG, dict(w, **{"l1.mix.w1": w["l1.mix.w1"][:-1]}))      # its rows are the rank that w2 has to have
    assert f"tensor l1.mix.w2 is bf16 72x{RC.RANK}, expected bf16 or f32 72x{RC.RANK - 1}" in _open_error(path)
    assert "4 layers, 5 asked" in _open_error(path, layers=5)


def test_executor_takes_a_model_directory(tmp_path):
    path = KC.write(tmp_path / "m", CFG, RC.weights(CFG, 1))
    r = subprocess.run([EXEC, "--model", path, "--prompt-tokens", "1,2,3", "--tokens", "5", "--print-config"], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0, r.stderr
    assert json.loads(r.stdout) == {"design": "Rapitar", "n_layers": 4, "layers_in_checkpoint": 4, "hidden": 32, "vocab": 40, "max_context": 8, "dtype": "bfloat16"}
