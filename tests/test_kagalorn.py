"""CPU-side checks of the Kagalorn design: the plain forward pass the GPU tests compare with, and what the library does
with a model directory before it needs a GPU (config.json, safetensors headers, the registry)."""
import ctypes as C
import json
import os
import struct
import subprocess

import numpy as np
import pytest

import kagalorn_case as KC
import kagalorn_oracle as K
from blok_amd.lib import KxModelShape, KxOpenOptions, kx

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EXEC = os.path.join(ROOT, "blok_amd", "kx-kimi-exec")
CFG = KC.config([KC.delta(), KC.attention(), KC.delta(ff=0)], vocab=40, width=32)


def test_window_and_blocks_partition_what_is_seen():
    for size, pool in ((1, 1), (5, 1), (5, 3), (3, 8), (8, 4), (7, 4)):
        for i in range(60):
            toks, blocks = K.visible(i, size, pool)
            assert toks == [j for j in range(i + 1) if 0 <= i - j < size]
            covered = [j for b in blocks for j in range(b * pool, (b + 1) * pool)]
            assert covered == list(range(len(covered))) and (not covered or covered[-1] <= i - size)
            assert len(covered) > i - size + 1 - pool        # less than a block is missing between blocks and window


def test_attention_with_blocks_of_one_and_no_sink_weight_is_full_attention():
    r = np.random.default_rng(0)
    q, k, v = r.standard_normal((20, 6)), r.standard_normal((20, 6)), r.standard_normal((20, 5))
    got = K.pooled_window_attention(q, k, v, 0.7, 4, 1)
    for i in range(20):
        e = np.exp(k[:i + 1] @ q[i] * 0.7)
        assert np.allclose(got[i], e @ v[:i + 1] / (1 + e.sum()))


def test_delta_rule_is_its_matrix_form_and_carries_its_state():
    r = np.random.default_rng(1)
    q, k, v = K.unit(r.standard_normal((9, 4))), K.unit(r.standard_normal((9, 4))), r.standard_normal((9, 3))
    beta, g = r.uniform(0, 1, 9), r.uniform(0.5, 1, 9)
    o, s = K.delta_rule(q, k, v, beta, g)
    m = np.zeros((4, 3))
    for t in range(9):                                       # S <- (I - beta k k^T) g S + beta k v^T
        m = (np.eye(4) - beta[t] * np.outer(k[t], k[t])) @ (g[t] * m) + beta[t] * np.outer(k[t], v[t])
        assert np.allclose(o[t], m.T @ q[t])
    a, s1 = K.delta_rule(q[:4], k[:4], v[:4], beta[:4], g[:4])
    b, s2 = K.delta_rule(q[4:], k[4:], v[4:], beta[4:], g[4:], s1)
    assert np.allclose(np.concatenate([a, b]), o) and np.allclose(s2, s)


def test_convolution_taps_and_hyper_connections():
    x = np.arange(12.0).reshape(6, 2)
    y = K.causal_conv(x, np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]]))
    assert y[0, 0] == 0 and y[1, 0] == 200 and y[2, 0] == 400 + 20 and y[3, 0] == 600 + 40 + 2 and (y[:, 1] == x[:, 1]).all()
    s = np.stack([np.full((1, 2), 1.0), np.full((1, 2), 10.0)])
    new = K.hyper_write(s, np.array([[1.0, 2.0], [3.0, 4.0]]), np.array([5.0, 6.0]), np.ones((1, 2)))   # mix[from, to]
    assert (new[0] == 1 + 30 + 5).all() and (new[1] == 2 + 40 + 6).all()
    assert (K.hyper_read(s, np.array([2.0, 1.0])) == 12).all()


def test_grouped_norm_and_clamped_glu():
    x = np.array([3.0, 4.0, 0.0, 0.5])
    assert np.allclose(K.grouped_rms_norm(x, np.ones(4), 2, 0.0), [3 / np.sqrt(12.5), 4 / np.sqrt(12.5), 0, np.sqrt(2)])
    eye = {"gate": np.eye(1), "up": np.eye(1), "down": np.eye(1)}
    for z, want in ((5.0, 1 / (1 + np.exp(-1.702)) * 2), (-5.0, -5 / (1 + np.exp(1.702 * 5)) * 0)):
        assert np.allclose(K.clamped_glu(np.array([[z]]), eye, "", 1.0), want)    # gate has no lower bound, up has


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
    KC.write(tmp_path / "m", CFG, KC.weights(CFG, 1))
    rc, shape, err = _probe(tmp_path / "m")
    assert rc == 0, err
    assert (shape.design, shape.n_layers, shape.hidden, shape.vocab) == (b"Kagalorn", 3, 32, 40)
    (tmp_path / "x").mkdir()
    assert "config.json" in _probe(tmp_path / "x")[2]
    (tmp_path / "x" / "config.json").write_text('{"architecture": "Other"}')
    rc, _, err = _probe(tmp_path / "x")
    assert rc != 0 and "Kimi-K2" in err and "Kagalorn" in err
    (tmp_path / "x" / "config.json").write_text('{"text_config": {"model_type": "kimi_k2"}}')
    assert "runtime-index.blok" in _probe(tmp_path / "x")[2]


@pytest.mark.parametrize("edit, message", [
    (lambda c: c.pop("vocab"), "model.vocab"),
    (lambda c: c.update(width="96"), "model.width"),
    (lambda c: c.update(streams=0), "model.streams"),
    (lambda c: c["norm"].update(groups=5), "5 groups"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="linear"), "layers[0].type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"].pop("mask"), "layers[1].mixer.mask"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=2.5), "mask.size"),
    (lambda c: c["layers"][1]["mlp"].update(kind="experts"), "mlp.kind"),
    (lambda c: c["layers"][0]["mixer"].update(dim=300), "dim=300"),
])
def test_configuration_errors_name_the_field(tmp_path, edit, message):
    cfg = json.loads(json.dumps(CFG))
    edit(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    rc, _, err = _probe(tmp_path)
    assert rc != 0 and message in err, err


@pytest.mark.parametrize("text", ["", "{", '{"a": 1,}', '{"a" 1}', '["x", 01x]', '{"a": "\\q"}', '{"a": "\\ud800"}', "[" * 100, "{} {}", '{"a": nul}', '"open'])
def test_malformed_json_is_an_error(tmp_path, text):
    (tmp_path / "config.json").write_text(text)
    rc, _, err = _probe(tmp_path)
    assert rc != 0 and "config.json" in err


def test_json_reader_takes_what_json_allows(tmp_path):
    text = json.dumps(dict(CFG, note="tab\t quote\" slash\\ é \U0001f600 €"), indent=3)
    (tmp_path / "config.json").write_text(text)
    assert _probe(tmp_path)[0] == 0
    (tmp_path / "config.json").write_text(text.replace('"width": 32', '"width": 3.2e1').replace('"architecture"', '"\\u0061rchitecture"'))
    rc, shape, err = _probe(tmp_path)
    assert rc == 0 and shape.hidden == 32, err


def test_weight_files_are_checked_before_anything_is_allocated(tmp_path):
    w = KC.weights(CFG, 1)
    path = KC.write(tmp_path / "m", CFG, {k: v for k, v in w.items() if k != "l1.mix.k.norm"})
    assert "missing tensor: l1.mix.k.norm" in _open_error(path)
    path = KC.write(tmp_path / "m", CFG, dict(w, head=w["head"][:, :-1]))
    assert "tensor head is bf16 40x31" in _open_error(path)
    assert "3 layers, 4 asked" in _open_error(path, layers=4)
    assert "max_batch" in _open_error(path, max_batch=0)
    good = KC.write(tmp_path / "m", CFG, w)
    blob = open(os.path.join(good, "model.safetensors"), "rb").read()
    for bad in (b"", blob[:6], struct.pack("<Q", 1 << 40) + blob[8:], blob[:8] + b"[" + blob[9:], blob[:-2], blob.replace(b'"BF16"', b'"XF16"', 1)):
        with open(os.path.join(good, "model.safetensors"), "wb") as f:
            f.write(bad)
        assert "model.safetensors" in _open_error(good)
    os.unlink(os.path.join(good, "model.safetensors"))
    assert "no safetensors files" in _open_error(good)


def test_executor_takes_a_model_directory(tmp_path):
    path = KC.write(tmp_path / "m", CFG, KC.weights(CFG, 1))

    def run(*a):
        return subprocess.run([EXEC, *a], capture_output=True, text=True, timeout=60)
    r = run("--model", path, "--prompt-tokens", "1,2,3", "--tokens", "5", "--dtype", "float32", "--print-config")
    assert r.returncode == 0, r.stderr
    doc = json.loads(r.stdout)
    assert doc == {"design": "Kagalorn", "n_layers": 3, "layers_in_checkpoint": 3, "hidden": 32, "vocab": 40, "max_context": 8, "dtype": "float32"}
    for extra, msg in ((("--prompt-tokens", "1,40"), "prompt token outside vocabulary"), (("--prompt-tokens", "1", "--dtype", "half"), "bad dtype"),
                       (("--prompt-tokens", "1", "--index", "x"), "--model takes none of"), (("--prompt-tokens", "1", "--prefill-chunk", "0"), "bad prefill chunk")):
        r = run("--model", path, "--tokens", "5", *extra)
        assert r.returncode == 1 and msg in r.stderr and r.stdout == "", (extra, r)
    r = run("--prompt-tokens", "1", "--tokens", "1", "--dtype", "float32")
    assert r.returncode == 1 and "--model" in r.stderr
