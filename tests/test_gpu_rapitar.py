"""The Rapitar design on the GPU against the plain forward pass of rapitar_oracle.py: each mechanism through its operator, then
whole models through the library's own step, cache, state, sampling and command line."""
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest

import kagalorn_case as KC
import rapitar_case as RC
import rapitar_oracle as R
from blok_amd import runtime
from blok_amd.lib import DevBuf, KxExpertsConfig, KxLatentConfig, KxLinearArgs, KxSsdConfig, KxWkvConfig, check
from kxt import dev, say
from test_gpu_kagalorn import SCHEDULES, _matrix, _rounded, portions, rel, to_f32

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EXEC = os.path.join(ROOT, "blok_amd", "kx-kimi-exec")
pytestmark = pytest.mark.gpu

BF16_LOGITS, F32_LOGITS = 0.05, 3e-5   # logit_error of a whole model
FORMATS = pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])


class Op:
    """An operator that keeps something from call to call: portions of position-major rows in, rows out."""

    def over(self, rows, cuts, cols, es, call):
        """rows [batch][n][...]; call(at, count, device rows, leading dimension, output)"""
        batch, n = rows.shape[:2]
        out = np.empty((batch, n, cols), np.float32)
        for at, c in portions(n, cuts):
            part = np.ascontiguousarray(rows[:, at:at + c].transpose(1, 0, 2), np.float32)
            d, o = dev(part), DevBuf(batch * c * cols * es)
            call(at, c, d.ptr, part.shape[2], o.ptr)
            out[:, at:at + c] = to_f32(o.to_numpy(np.float32 if es == 4 else np.uint16, (c, batch, cols))).transpose(1, 0, 2)
        return out


# ---- state-space duality ----------------------------------------------------------------------------------------

class Ssd(Op):
    def __init__(self, lib, heads, vdim, state, groups, taps, batch=1, positions=512, seed=0, decay=0.7, bias=True):
        self.lib, self.shape = lib, (heads, vdim, state, groups, taps)
        c = KxSsdConfig(heads, vdim, state, groups, taps)
        self.h = C.c_void_p()
        check(lib.kx_ssd_create(C.byref(c), batch, positions, C.byref(self.h)))
        self.inner, self.channels = heads * vdim, heads * vdim + 2 * groups * state
        r = np.random.default_rng(seed)
        self.conv, self.bias = r.standard_normal((self.channels, taps)).astype(np.float32), (0.3 * r.standard_normal(self.channels)).astype(np.float32)
        self.a_log, self.dt, self.skip = [(s * r.standard_normal(heads) + m).astype(np.float32) for s, m in ((decay, -1.0), (1.0, -1.0), (1.0, 0.0))]
        if not bias:
            self.bias[:] = 0
        self.has_bias = bias
        self.push()

    def push(self):
        self.d = [dev(x) for x in (self.conv, self.bias, self.a_log, self.dt, self.skip)]

    def cols(self):
        return 3 + self.channels + 2 + self.shape[0]       # something before, between and nothing behind

    def run(self, proj, cuts):
        check(self.lib.kx_ssd_restart(self.h, None))
        d = [x.ptr for x in self.d]
        if not self.has_bias:
            d[1] = None
        return self.over(proj, cuts, self.inner, 4, lambda at, c, x, ld, o: check(
            self.lib.kx_ssd_run(self.h, x, ld, 3, 3 + self.channels + 2, *d, proj.shape[0], c, o, None)))

    def oracle(self, proj):
        heads, vdim, n, g, _ = self.shape
        p, t = proj.astype(np.float64), len(proj)
        xbc = R.silu(R.causal_conv(p[:, 3:3 + self.channels], self.conv.astype(np.float64), self.bias.astype(np.float64)))
        x, b, c = np.split(xbc, [self.inner, self.inner + g * n], axis=1)
        x, b, c = x.reshape(t, heads, vdim), b.reshape(t, g, n), c.reshape(t, g, n)
        dt = R.softplus(p[:, -heads:] + self.dt)
        a = np.exp(-np.exp(self.a_log.astype(np.float64)) * dt)
        return np.stack([R.ssd(x[:, h], b[:, h // (heads // g)], c[:, h // (heads // g)], dt[:, h], a[:, h], self.skip[h])[0] for h in range(heads)], 1).reshape(t, -1)

    def close(self):
        check(self.lib.kx_ssd_destroy(self.h))


# heads, vdim, state, groups, taps: one to many heads per group (more than the 16 that share a launch of the coefficients), every
# size of the state's tiles, columns off and on a wave's 16, no history at all, more taps than a portion has positions
SSDS = [(4, 24, 16, 2, 4), (3, 5, 8, 3, 1), (6, 33, 40, 1, 2), (2, 64, 64, 2, 3), (4, 70, 100, 4, 4), (8, 64, 128, 2, 4), (1, 17, 200, 1, 7), (2, 40, 256, 2, 3),
        (1, 8, 300, 1, 2), (2, 130, 512, 1, 4), (20, 16, 48, 1, 3), (66, 8, 20, 2, 4), (1, 1, 1, 1, 5)]


@pytest.mark.parametrize("case", SSDS, ids=lambda c: "-".join(map(str, c)))
def test_state_space_in_portions_of_every_kind(kxlib, case):
    d = Ssd(kxlib, *case, bias=case[0] != 3)
    proj = np.random.default_rng(4).standard_normal((1, 150, d.cols())).astype(np.float32)
    want = d.oracle(proj[0])
    for name, cuts in SCHEDULES.items():
        say(f"state space {case} {name}")
        assert rel(d.run(proj, cuts)[0], want) < 3e-5, name
    d.close()


def test_state_space_on_many_workgroups(kxlib):
    """More column groups than CUs: a wave then has all rows of its columns (state of 64 and of 96)."""
    for case in ((280, 10, 64, 4, 4), (300, 16, 96, 2, 2)):
        d = Ssd(kxlib, *case)
        proj = np.random.default_rng(5).standard_normal((1, 40, d.cols())).astype(np.float32)
        assert rel(d.run(proj, [40])[0], d.oracle(proj[0])) < 3e-5, case
        d.close()


def test_state_space_holds_a_write_for_long_and_strong_decays_forget(kxlib):
    heads, vdim, state = 2, 8, 32
    d = Ssd(kxlib, heads, vdim, state, 1, 1)
    d.conv[:], d.bias[:], d.skip[:], d.dt[:] = 1.0, 0.0, 0.0, 0.0
    d.a_log[:] = (-30.0, 4.0)                                       # head 0 keeps everything, head 1 nothing
    d.push()
    n, x0 = 400, 3
    proj = np.zeros((1, n, d.cols()), np.float32)
    proj[..., -heads:] = 2.0
    b0 = x0 + heads * vdim
    proj[0, 5, x0:b0] = 3.0                                         # one write under key 7 ...
    proj[0, 5, b0 + 7] = 4.0
    proj[..., b0 + state + 7] = 5.0                                 # ... that every query reads
    want = d.oracle(proj[0])
    assert want[399, 0] > 50 and want[5, vdim] > 50 and abs(want[6, vdim]) < 1e-20
    for name, cuts in SCHEDULES.items():
        got = d.run(proj, cuts)[0]
        assert np.isfinite(got).all() and rel(got, want) < 1e-5, name
    d.close()


def test_state_space_batch_equals_each_alone(kxlib):
    d = Ssd(kxlib, 4, 40, 48, 2, 4, batch=5)
    proj = np.random.default_rng(6).standard_normal((5, 90, d.cols())).astype(np.float32)
    for s in ("whole", "mixed", "decoded"):
        together = d.run(proj, SCHEDULES[s])
        for b in range(5):
            assert rel(together[b], d.run(proj[b:b + 1], SCHEDULES[s])[0]) < 1e-6, (s, b)
    d.close()


# ---- time mixing ------------------------------------------------------------------------------------------------

class Wkv(Op):
    def __init__(self, lib, heads, dim, rank, f32, batch=1, positions=512, seed=0):
        self.lib, self.f32, self.shape = lib, f32, (heads, dim, rank)
        c = KxWkvConfig(heads, dim, rank)
        self.h = C.c_void_p()
        check(lib.kx_wkv_create(C.byref(c), f32, batch, positions, C.byref(self.h)))
        self.hd = heads * dim
        r = np.random.default_rng(seed)
        self.w2 = KC.bf16(r.standard_normal((self.hd, rank)) * rank ** -0.5)
        self.w0, self.u = (1.2 * r.standard_normal(self.hd) - 1.5).astype(np.float32), r.standard_normal(self.hd).astype(np.float32)
        self.push()

    def push(self):
        self.d = [_matrix(self.w2, self.f32)[0], dev(self.w0), dev(self.u)]

    def cols(self):
        return 3 * self.hd + self.shape[2] + 5

    def run(self, proj, cuts):
        check(self.lib.kx_wkv_restart(self.h, None))
        hd = self.hd
        return self.over(proj, cuts, hd, 4, lambda at, c, x, ld, o: check(
            self.lib.kx_wkv_run(self.h, x, ld, 0, hd, 2 * hd, 3 * hd + 5, *[y.ptr for y in self.d], proj.shape[0], c, o, None)))

    def oracle(self, proj, rounded=False):
        """rounded: the rank's tanh in bf16, as a product's rows are"""
        heads, dim, _ = self.shape
        t, p = len(proj), proj.astype(np.float64)
        r, k, v = (p[:, i * self.hd:(i + 1) * self.hd].reshape(t, heads, dim) for i in range(3))
        low = np.tanh(p[:, 3 * self.hd + 5:])
        low = KC.bf16(low).astype(np.float64) if rounded else low
        w = np.exp(-np.exp(low @ self.w2.T.astype(np.float64) + self.w0)).reshape(t, heads, dim)
        u = self.u.reshape(heads, dim).astype(np.float64)
        return np.stack([R.wkv(r[:, h], k[:, h], v[:, h], w[:, h], u[h])[0] for h in range(heads)], 1).reshape(t, -1)

    def close(self):
        check(self.lib.kx_wkv_destroy(self.h))


WKVS = [(2, 16, 8), (3, 33, 16), (1, 64, 64), (2, 128, 20), (1, 200, 70), (1, 260, 5), (5, 48, 100), (4, 4, 1), (2, 96, 33)]


@FORMATS
@pytest.mark.parametrize("case", WKVS, ids=lambda c: "-".join(map(str, c)))
def test_time_mixing_in_portions_of_every_kind(kxlib, case, f32):
    d = Wkv(kxlib, *case, f32)
    proj = np.random.default_rng(4).standard_normal((1, 150, d.cols())).astype(np.float32)
    want, near = d.oracle(proj[0]), d.oracle(proj[0], not f32)
    for name, cuts in SCHEDULES.items():
        say(f"time mixing {case} f32={f32} {name}")
        got = d.run(proj, cuts)[0]
        if name == "decoded":                                       # nothing is rounded on the way to a single token's decay
            assert rel(got, want) < 3e-5
        elif name == "mixed":
            assert rel(got, want) < (3e-5 if f32 else 2e-2)
        else:
            assert rel(got, near) < (3e-5 if f32 else 2e-4), name
    d.close()


def test_time_mixing_keeps_and_forgets_per_channel_and_the_bonus_is_for_the_current_token(kxlib):
    d = Wkv(kxlib, 1, 32, 1, 1)
    d.w2[:], d.u[:] = 0.0, 0.0
    d.w0[:] = np.where(np.arange(32) % 2, -40.0, 5.0)               # odd channels keep everything, even ones nothing
    d.u[4] = 6.0
    d.push()
    proj = np.zeros((1, 300, d.cols()), np.float32)
    proj[..., :32] = 1.0                                            # every query reads all channels
    for t, ch in ((3, 5), (3, 8), (100, 4), (150, 7)):
        proj[0, t, 32 + ch] = 2.0
        proj[0, t, 64:96] = 1.0 + np.arange(32)
    want = d.oracle(proj[0])
    assert np.allclose(want[3], 0) and np.allclose(want[4, 0], 4) and np.allclose(want[5, 0], 2) and np.allclose(want[100, 0], 2 + 12) and np.allclose(want[299, 0], 4)
    for name, cuts in SCHEDULES.items():
        got = d.run(proj, cuts)[0]
        assert np.isfinite(got).all() and rel(got, want) < 1e-5, name
    d.close()


def test_time_mixing_batch_equals_each_alone(kxlib):
    d = Wkv(kxlib, 3, 40, 20, 1, batch=5)
    proj = np.random.default_rng(6).standard_normal((5, 90, d.cols())).astype(np.float32)
    for s in ("whole", "mixed", "decoded"):
        together = d.run(proj, SCHEDULES[s])
        for b in range(5):
            assert rel(together[b], d.run(proj[b:b + 1], SCHEDULES[s])[0]) < 1e-5, (s, b)
    d.close()


# ---- latent attention -------------------------------------------------------------------------------------------

class Latent(Op):
    def __init__(self, lib, heads, dim, rot_dim, rot, vdim, rank, f32, batch=1, context=512, positions=512, sink=1, gate=1, scale=None, base=300.0,
                 no_expand=0, seed=0):
        self.lib, self.f32, self.shape, self.gate, self.sink, self.base, self.eps = lib, f32, (heads, dim, rot_dim, rot, vdim, rank), gate, sink, base, 1e-5
        self.scale = (dim + rot_dim) ** -0.5 if scale is None else scale
        c = KxLatentConfig(heads, dim, rot_dim, rot, vdim, rank, sink, gate, no_expand, self.scale, self.eps, base)
        self.h = C.c_void_p()
        check(lib.kx_latent_create(C.byref(c), f32, batch, context, positions, C.byref(self.h)))
        r = np.random.default_rng(seed)
        self.norm = (1 + 0.3 * r.standard_normal(rank)).astype(np.float32)
        self.uk, self.uv = [KC.bf16(s * r.standard_normal((heads * n, rank)) * rank ** -0.5) for s, n in ((1.5, dim), (1.0, vdim))]
        self.sinks = r.standard_normal(heads).astype(np.float32)
        self.push()

    def push(self):
        self.d = [dev(self.norm), _matrix(self.uk, self.f32)[0], _matrix(self.uv, self.f32)[0], dev(self.sinks)]

    def cols(self):
        heads, dim, rot_dim, _, vdim, rank = self.shape
        return np.cumsum([0, heads * (dim + rot_dim), rank + rot_dim, heads * vdim])      # queries, latent and shared key, gate

    def run(self, rows, cuts):
        heads, _, _, _, vdim, _ = self.shape
        c = list(map(int, self.cols()))
        batch = rows.shape[0]
        return self.over(rows, cuts, heads * vdim, 4 if self.f32 else 2, lambda at, n, x, ld, o: check(
            self.lib.kx_latent_run(self.h, x, ld, x, ld, c[1], c[2], *[y.ptr for y in self.d], batch, n, at, o, heads * vdim, None)))

    def keys(self, rows):
        """(queries, keys, values) [T][heads][...] in the number format's precision"""
        heads, dim, rot_dim, rot, vdim, rank = self.shape
        t, p = len(rows), rows.astype(np.float64)
        pos = np.arange(t, dtype=np.float64)
        r = (lambda x: x) if self.f32 else (lambda x: KC.bf16(x).astype(np.float64))
        q, kv, _ = np.split(p, self.cols()[1:3], axis=1)
        q = q.reshape(t, heads, dim + rot_dim)
        turn = (lambda x: R.rotate_half(x, pos, rot, self.base)) if rot else (lambda x: x)
        q = np.concatenate([q[..., :dim], turn(q[..., dim:])], -1)
        c, shared = r(R.rms(kv[:, :rank], self.eps) * self.norm), r(turn(kv[:, rank:]))
        k = (c @ self.uk.T.astype(np.float64)).reshape(t, heads, dim)
        return q, np.concatenate([k, np.repeat(shared[:, None], heads, 1)], -1), (c @ self.uv.T.astype(np.float64)).reshape(t, heads, vdim)

    def oracle(self, rows):
        heads = self.shape[0]
        q, k, v = self.keys(rows)
        o = np.stack([R.sink_attention(q[:, h], k[:, h], v[:, h], self.scale, float(self.sinks[h]) if self.sink else -np.inf) for h in range(heads)], 1)
        o = o.reshape(len(rows), -1)
        return o * R.sigmoid(rows[:, self.cols()[2]:].astype(np.float64)) if self.gate else o

    def close(self):
        check(self.lib.kx_latent_destroy(self.h))


# heads, dim, rot_dim, rotated of them, vdim, rank: sizes off every tile; heads off the groups of 8; nothing rotated and part of it;
# keys and values wider than the matrix-core kernel takes; latents of one, two and more passes of a workgroup's columns
LATENTS = [(4, 24, 16, 16, 40, 32), (2, 40, 8, 4, 16, 100), (3, 33, 6, 6, 31, 130), (16, 64, 32, 32, 64, 128), (5, 128, 64, 64, 128, 512), (1, 16, 0, 0, 8, 20),
           (12, 96, 32, 16, 160, 260), (2, 300, 10, 10, 20, 70), (2, 16, 8, 8, 270, 700), (9, 16, 8, 8, 16, 1100), (1, 1, 2, 2, 1, 1)]


def _bar(f32):
    return 4e-5 if f32 else 3e-2


@FORMATS
@pytest.mark.parametrize("case", LATENTS, ids=lambda c: "-".join(map(str, c)))
def test_latent_attention_in_portions_of_every_kind(kxlib, case, f32):
    a = Latent(kxlib, *case, f32)
    rows = np.random.default_rng(5).standard_normal((1, 200, a.cols()[-1])).astype(np.float32)
    want = a.oracle(rows[0])
    for name, cuts in dict(SCHEDULES, eights=[8], nines=[9, 3]).items():
        say(f"latent {case} f32={f32} {name}")
        assert rel(a.run(rows, cuts)[0], want) < _bar(f32), name
    a.close()


@FORMATS
def test_latent_attention_without_room_for_expanded_keys(kxlib, f32):
    a = Latent(kxlib, 6, 24, 12, 12, 20, 48, f32, batch=3, no_expand=1)
    rows = np.random.default_rng(7).standard_normal((3, 120, a.cols()[-1])).astype(np.float32)
    for cuts in ([120], [50, 30, 1]):
        got = a.run(rows, cuts)
        for b in range(3):
            assert rel(got[b], a.oracle(rows[b])) < _bar(f32), (cuts, b)
    a.close()


@FORMATS
def test_latent_tiles_one_after_the_other(kxlib, f32):
    """Enough tokens, heads and keys that a workgroup goes through several tiles of keys."""
    a = Latent(kxlib, 24, 16, 8, 8, 16, 64, f32, batch=6, context=640, positions=8)
    rows = np.random.default_rng(8).standard_normal((6, 640, a.cols()[-1])).astype(np.float32)
    got = a.run(rows, [8])
    for b in (0, 5):
        assert rel(got[b], a.oracle(rows[b])) < _bar(f32), b
    a.close()


@FORMATS
@pytest.mark.parametrize("part", ["unrotated", "rotated"])
def test_one_key_that_stands_out_wherever_it_is(kxlib, part, f32):
    """Query i meets one key that scores far above hundreds of others: at the start, at both sides of every tile's edge, the last
    but one, itself.  With the rotated part it does so at that distance only."""
    heads, dim, rot_dim, n = 2, 32, 16, 330
    a = Latent(kxlib, heads, dim, rot_dim, rot_dim, 24, 40, f32, gate=0, scale=1.0)
    a.sinks[:] = 0.5
    a.push()
    c = a.cols()
    r = np.random.default_rng(3)
    for i, j in ((329, 0), (329, 1), (300, 31), (300, 32), (310, 63), (310, 64), (311, 127), (311, 128), (328, 255), (328, 256), (327, 326), (200, 200), (15, 0), (16, 1)):
        say(f"stands out: {part} {i} -> {j} f32={f32}")
        rows = (0.05 * r.standard_normal((n, c[-1]))).astype(np.float32)
        rows[:, c[1]:c[1] + 40] = r.standard_normal((n, 40))        # the latents differ
        if part == "unrotated":
            k = a.keys(rows)[1][j, :, :dim]
            rows[i, :c[1]] = 0
            for h in range(heads):
                rows[i, h * (dim + rot_dim):h * (dim + rot_dim) + dim] = 14.0 * k[h] / (k[h] @ k[h])
        else:
            shared = r.standard_normal(rot_dim)
            rows[j, c[1] + 40:c[2]] = 2.5 * shared / np.linalg.norm(shared)
            turned = R.rotate_half(shared[None], np.array([float(j - i)]), rot_dim, a.base)[0]      # the query that meets it best from i
            for h in range(heads):
                rows[i, h * (dim + rot_dim):(h + 1) * (dim + rot_dim)] = np.concatenate([np.zeros(dim), 5.0 * turned / np.linalg.norm(turned)])
        want = a.oracle(rows)
        q, k, _ = a.keys(rows)
        score = np.einsum("hd,jhd->hj", q[i], k[:i + 1])
        assert (score.argmax(1) == j).all() and (np.exp(score[:, j]) > 0.6 * np.exp(score).sum(1)).all()
        for s in ("whole", "decoded", "mixed"):
            got = a.run(rows[None], SCHEDULES[s])[0]
            assert rel(got[i], want[i]) < _bar(f32), (i, j, s)
    a.close()


@FORMATS
def test_sink_gate_and_rotation_are_parameters(kxlib, f32):
    for sink, gate, sinks, base in ((0, 1, 0.0, 50.0), (1, 0, 6.0, 1e6), (1, 1, -20.0, 2.0), (0, 0, 3.0, 1e4)):
        a = Latent(kxlib, 4, 24, 16, 16, 24, 40, f32, sink=sink, gate=gate, scale=0.4, base=base)
        a.sinks[:] = sinks + 0.1 * np.arange(4)
        a.push()
        rows = np.random.default_rng(9).standard_normal((1, 90, a.cols()[-1])).astype(np.float32)
        want = a.oracle(rows[0])
        for s in ("whole", "decoded", "mixed"):
            assert rel(a.run(rows, SCHEDULES[s])[0], want) < _bar(f32), (sink, gate, sinks, s)
        a.close()


def test_latent_batch_equals_each_alone(kxlib):
    for f32, exact in ((1, 1e-5), (0, 1e-2)):
        a = Latent(kxlib, 4, 24, 8, 8, 40, 48, f32, batch=6, context=160, positions=160)
        rows = np.random.default_rng(2).standard_normal((6, 150, a.cols()[-1])).astype(np.float32)
        together = {s: a.run(rows, SCHEDULES[s]) for s in ("whole", "mixed", "decoded")}
        for b in range(6):
            for s, t in together.items():
                assert rel(t[b], a.run(rows[b:b + 1], SCHEDULES[s])[0]) < exact, (f32, s, b)
        a.close()


# ---- experts ----------------------------------------------------------------------------------------------------

def _packed(gate, up):
    """[experts][ff][cols] twice -> the library's blocks of 32 gate and 32 up rows"""
    e, ff, cols = gate.shape
    blocks = -(-ff // 32)
    out = np.zeros((e, blocks, 2, 32, cols), np.float32)
    for half, m in ((0, gate), (1, up)):
        full = np.zeros((e, blocks * 32, cols), np.float32)
        full[:, :ff] = m
        out[:, :, half] = full.reshape(e, blocks, 32, cols)
    return out.reshape(e, blocks * 64, cols)


def _stack(m, f32):
    """[experts][rows][cols] on the device with padded rows"""
    return _matrix(m.reshape(-1, m.shape[-1]), f32)[0]


class Experts:
    def __init__(self, lib, width, ff, experts, top, cols, f32, tokens, seed=0):
        self.lib, self.shape, self.f32 = lib, (width, ff, experts, top, cols), f32
        c = KxExpertsConfig(width, ff, experts, top, cols, np.inf, 1.0, 0.0)
        self.h = C.c_void_p()
        check(lib.kx_experts_create(C.byref(c), f32, tokens, C.byref(self.h)))
        r = np.random.default_rng(seed)
        self.router, self.bias = KC.bf16(2.0 * r.standard_normal((experts, width)) * width ** -0.5), r.standard_normal(experts).astype(np.float32)
        self.gate, self.up = [KC.bf16(1.5 * r.standard_normal((experts, ff, width)) * width ** -0.5) for _ in range(2)]
        self.down = KC.bf16(r.standard_normal((experts, width, ff)) * ff ** -0.5)
        self.w = KC.bf16(0.5 * r.standard_normal((width, cols)) * cols ** -0.5)
        self.norm = (1 + 0.3 * r.standard_normal(width)).astype(np.float32)
        self.push()

    def push(self):
        self.d = [dev(self.norm), _matrix(self.router, self.f32)[0], dev(self.bias), _stack(_packed(self.gate, self.up), self.f32), _stack(self.down, self.f32),
                  _matrix(self.w, self.f32)[0]]

    def run(self, x, rows):
        """(x afterwards, chosen experts)"""
        n, top, cols = len(x), self.shape[3], self.shape[4]
        pad = np.zeros((n, -(-cols // 64) * 64), np.float32)
        pad[:, :cols] = rows
        dx, dr, ids = dev(x), dev(pad if self.f32 else (pad.view(np.uint32) >> 16).astype(np.uint16)), DevBuf(4 * n * top)
        d = [y.ptr for y in self.d]
        check(self.lib.kx_experts_run(self.h, dx.ptr, d[0], 1e-5, d[1], d[2], d[3], d[4], d[5], dr.ptr, n, ids.ptr, None))
        check(self.lib.kx_sync(None))
        return dx.to_numpy(np.float32, x.shape), ids.to_numpy(np.int32, (n, top))

    def oracle(self, x, rows, ids):
        """with the device's choice, which has to be one that rounding allows"""
        h = R.rms(x.astype(np.float64), 1e-5) * self.norm
        z = _rounded(h, self.f32) @ self.router.T.astype(np.float64) + self.bias
        kth = np.sort(z, 1)[:, -self.shape[3]]
        mine = np.take_along_axis(z, ids.astype(np.int64), 1)
        assert (mine >= kth[:, None] - (1e-4 if self.f32 else 3e-2)).all() and (np.diff(mine, axis=1) <= (1e-4 if self.f32 else 3e-2)).all()
        assert all(len(set(row)) == len(row) for row in ids)
        weight = np.exp(mine - mine.max(1, keepdims=True))
        weight /= weight.sum(1, keepdims=True)
        out = x + rows.astype(np.float64) @ self.w.T
        for e in range(self.shape[2]):
            tok, slot = np.nonzero(ids == e)
            w = {"gate": self.gate[e].astype(np.float64), "up": self.up[e].astype(np.float64), "down": self.down[e].astype(np.float64)}
            out[tok] += weight[tok, slot][:, None] * R.expert(_rounded(h[tok], self.f32), w, "")
        return out

    def close(self):
        check(self.lib.kx_experts_destroy(self.h))


# width, ff, experts, top, cols of the product beside them; the last does not fit a workgroup's rows in f32
EXPERTS = [(96, 40, 16, 2, 70), (120, 32, 5, 5, 64), (64, 100, 70, 3, 130), (200, 33, 1, 1, 20), (128, 48, 200, 8, 2100), (96, 40, 4, 2, 33), (64, 2048, 24, 20, 64)]


@FORMATS
@pytest.mark.parametrize("case", EXPERTS, ids=lambda c: "-".join(map(str, c)))
def test_experts_for_few_and_many_tokens(kxlib, case, f32):
    a = Experts(kxlib, *case, f32, 700)
    r = np.random.default_rng(1)
    for n in (1, 2, 3, 4, 5, 33, 130, 700):
        say(f"experts {case} f32={f32} tokens={n}")
        x, rows = r.standard_normal((n, case[0])).astype(np.float32), KC.bf16(r.standard_normal((n, case[4])))
        got, ids = a.run(x, rows)
        assert rel(got, a.oracle(x, rows, ids)) < (3e-5 if f32 else 2e-2), n
    a.close()


@FORMATS
def test_equal_logits_choose_the_lower_index_and_one_expert_may_have_every_token(kxlib, f32):
    a = Experts(kxlib, 64, 32, 100, 3, 64, f32, 300)
    a.router[:], a.bias[:] = 0.0, 0.0
    for n in (2, 300):
        for bias, want in ((None, [0, 1, 2]), (77, [77, 0, 1])):
            a.bias[:] = 0.0
            if bias is not None:
                a.bias[bias] = 2.0
            a.push()
            r = np.random.default_rng(n)
            x, rows = r.standard_normal((n, 64)).astype(np.float32), KC.bf16(r.standard_normal((n, 64)))
            got, ids = a.run(x, rows)
            assert (ids == want).all()
            assert rel(got, a.oracle(x, rows, ids)) < (3e-5 if f32 else 2e-2)
    a.close()


# ---- products with their rows and epilogues ----------------------------------------------------------------------

@FORMATS
@pytest.mark.parametrize("tokens", [1, 2, 3, 4, 5, 33, 130])
def test_rows_of_this_designs_products(kxlib, tokens, f32):
    r = np.random.default_rng(tokens)
    tol, es = (2e-5, 4) if f32 else (1.5e-2, 2)
    as_format = lambda x: dev(x if f32 else (np.ascontiguousarray(x).view(np.uint32) >> 16).astype(np.uint16))

    def run(**kw):
        a = KxLinearArgs(f32=f32, tokens=tokens, streams=1, groups=1, eps=1e-5)
        for k, v in kw.items():
            if k == "var_row":
                a.var_row[:len(v)] = v
            else:
                setattr(a, k, v)
        scratch = DevBuf(tokens * a.ld * es * 8)
        check(kxlib.kx_linear_run(C.byref(a), scratch.ptr, None))
        check(kxlib.kx_sync(None))

    # mixes of neighbouring positions, several sequences, plain rows behind them and an activation for the last ones
    for batch in (1, tokens) if tokens > 1 else (1,):
        for cols, n_mix, sizes in ((96, 2, (100, 40, 60)), (300, 5, (33, 128, 7, 150, 20, 90))):
            starts = np.cumsum([0] + [-(-s // 128) * 128 for s in sizes])
            rows = int(starts[-2]) + sizes[-1]
            w = np.zeros((rows, cols), np.float32)
            for s, n in zip(starts, sizes):
                w[s:s + n] = KC.bf16(r.standard_normal((n, cols)) * cols ** -0.5)
            dw, ld = _matrix(w, f32)
            x, prev = r.standard_normal((tokens // batch, batch, cols)).astype(np.float32), r.standard_normal((batch, cols)).astype(np.float32)
            norm, mu = (1 + 0.3 * r.standard_normal(cols)).astype(np.float32), r.standard_normal((n_mix, cols)).astype(np.float32)
            act = sizes[-1] - 10
            d = [dev(y) for y in (x, norm, mu, prev)]
            kept, out, mid = DevBuf(prev.nbytes), DevBuf(tokens * rows * 4), DevBuf(tokens * (act + 3) * es)
            run(rows=rows, cols=cols, ld=ld, row_kind=3, epilogue=0, d_w=dw.ptr, d_streams_in=d[0].ptr, d_norm=d[1].ptr, d_mu=d[2].ptr, d_prev=d[3].ptr,
                d_prev_out=kept.ptr, n_mix=n_mix, batch=batch, var_row=[int(s) for s in starts[:n_mix + 1]], d_out=out.ptr, out_ld=rows, act_rows=act,
                d_mid=mid.ptr, mid_ld=act + 3)
            h = R.rms(x.astype(np.float64), 1e-5) * norm
            before = np.concatenate([prev[None].astype(np.float64), h[:-1]])
            got = out.to_numpy(np.float32, (tokens // batch, batch, rows))
            for m, (s, n) in enumerate(zip(starts, sizes)):
                hm = _rounded(h + (before - h) * mu[m] if m < n_mix else h, f32)
                want = hm @ w[s:s + n].T
                if m < n_mix:
                    assert rel(got[..., s:s + n], want) < tol, (cols, batch, m)
                else:
                    assert rel(got[..., s:s + 10], want[..., :10]) < tol
                    y = to_f32(mid.to_numpy(np.float32 if f32 else np.uint16, (tokens, act + 3)))[:, :act].reshape(tokens // batch, batch, act)
                    assert rel(y, R.gelu_tanh(want[..., 10:])) < tol
            assert rel(kept.to_numpy(np.float32, prev.shape), h[-1]) < 1e-5

    # a read-out: gate in front of the norm or behind it, few long parts or many, a weight per column, a tail behind it
    for heads, vdim, first, tail in ((1, 150, 1, 0), (3, 40, 1, 50), (12, 20, 1, 0), (10, 24, 0, 33), (2, 64, 0, 130), (7, 9, 1, 1)):
        head_ld = -(-heads * vdim // 64) * 64
        cols = head_ld + tail if tail else heads * vdim
        w = KC.bf16(r.standard_normal((70, cols)) * cols ** -0.5)
        w[:, heads * vdim:head_ld] = 0
        dw, ld = _matrix(w, f32)
        o, g = r.standard_normal((tokens, heads * vdim)).astype(np.float32), r.standard_normal((tokens, heads * vdim + 5)).astype(np.float32)
        wc = (1 + 0.3 * r.standard_normal(heads * vdim)).astype(np.float32)
        t = np.zeros((tokens, max(ld - head_ld, 64)), np.float32)
        t[:, :tail] = KC.bf16(r.standard_normal((tokens, tail)))
        d = [dev(o), dev(g), dev(wc), as_format(t)]
        out = DevBuf(tokens * 70 * 4)
        kw = dict(d_tail=d[3].ptr, tail_ld=t.shape[1], head_ld=head_ld) if tail else {}
        run(rows=70, cols=cols, ld=ld, row_kind=2, epilogue=0, d_w=dw.ptr, d_o=d[0].ptr, d_gate=d[1].ptr, gate_ld=heads * vdim + 5, heads=heads, vdim=vdim,
            d_norm=d[2].ptr, w_per_column=1, gate_first=first, d_out=out.ptr, out_ld=70, **kw)
        z, y = g[:, :heads * vdim].astype(np.float64), o.astype(np.float64)
        h = R.gated_then_normed(y, z, wc, heads, 1e-5) if first else R.grouped_rms(y, heads, 1e-5) * wc * R.silu(z)
        want = _rounded(h, f32) @ w[:, :heads * vdim].T + (t[:, :tail].astype(np.float64) @ w[:, head_ld:].T if tail else 0)
        assert rel(out.to_numpy(np.float32, (tokens, 70)), want) < tol, (heads, vdim, first, tail)

    # tanh of 32-bit rows; a block per head
    x = r.standard_normal((tokens, 50)).astype(np.float32)
    w = KC.bf16(r.standard_normal((96, 40)) * 40 ** -0.5)
    dw, ld = _matrix(w, f32)
    dx, out = dev(x), dev(np.full((4, tokens, 30), 7.0, np.float32) if f32 else np.full((4, tokens, 30), 0x40e0, np.uint16))
    run(rows=96, cols=40, ld=ld, row_kind=4, epilogue=3, d_w=dw.ptr, d_streams_in=dx.ptr, streams_ld=50, d_out=out.ptr, out_ld=30, head_dim=24, head_stride=tokens * 30)
    got = to_f32(out.to_numpy(np.float32 if f32 else np.uint16, (4, tokens, 30)))
    want = (_rounded(np.tanh(x[:, :40].astype(np.float64)), f32) @ w.T).reshape(tokens, 4, 24).transpose(1, 0, 2)
    assert rel(got[..., :24], want) < tol and (got[..., 24:] == 7.0).all()


# ---- models -----------------------------------------------------------------------------------------------------

MODELS = {
    "all kinds": RC.config([RC.mamba2(mlp=RC.dense()), RC.wkv(mlp=RC.moe()), RC.latent(mlp=RC.moe(experts=10, top=3)), RC.mamba2(groups=1, norm_groups=1, conv=2, mlp=RC.moe()),
                            RC.latent(heads=10, rot_dim=8, dims=4, base=77.0, mlp=RC.dense(50)), RC.wkv(heads=2, dim=40, mlp=RC.dense(33))]),
    "no feed-forward": RC.config([RC.wkv(), RC.latent(), RC.mamba2(heads=4, groups=4, norm_groups=2, state=70, conv=1), RC.wkv(heads=5, dim=8, mlp=RC.dense(20))], width=120),
    "other sizes": RC.config([RC.latent(heads=1, dim=8, rot_dim=2, vdim=70, q_rank=9, kv_rank=150, scale=0.3, mlp=RC.moe(ff=70, experts=1, top=1)),
                              RC.mamba2(heads=1, vdim=64, state=130, groups=1, norm_groups=4, conv=6, mlp=RC.moe(ff=9, experts=70, top=6)),
                              RC.wkv(heads=1, dim=66, mlp=RC.moe(ff=40, experts=3, top=3))], width=200, vocab=301, eps=1e-3),
    # (a part of one element over its own root mean square is a step at zero: a large eps makes it a slope)
    "heads of one": RC.config([RC.mamba2(heads=33, vdim=1, state=1, groups=1, norm_groups=33, conv=3, mlp=RC.dense(32)), RC.wkv(heads=40, dim=1),
                               RC.latent(heads=33, dim=4, rot_dim=2, vdim=3, q_rank=16, kv_rank=12)], width=64, vocab=33, eps=0.3),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            cfg = MODELS[name]
            w = RC.weights(cfg, sum(map(ord, name)))
            made[name] = cfg, w, KC.write(tmp_path_factory.mktemp("rapitar"), cfg, w)
        return made[name]
    return get


DTYPES = pytest.mark.parametrize("dtype, bar", [("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)])


@DTYPES
@pytest.mark.parametrize("name", MODELS)
def test_model_whole_decoded_and_in_portions(kxlib, models, name, dtype, bar):
    cfg, w, path = models(name)
    ids = KC.tokens(cfg, 170, 1)
    record = []
    want = R.forward(cfg, w, ids, record)
    with KC.Model(path, dtype, context=170) as m:
        check(kxlib.kx_model_set_residual_record(m.h, 1))
        for s, cuts in dict(SCHEDULES, late=[140, 1], nines=[9, 3, 8]).items():
            got = m.run(ids, cuts)[:, 0]
            err = KC.logit_error(got, want)
            say(f"{name} {dtype} {s}: worst {err.max():.1e} at {err.argmax()}")
            assert err.max() < bar, (s, int(err.argmax()))
            for layer, ref in enumerate(record):
                x = np.empty(ref.shape, np.float32)
                check(kxlib.kx_model_residual(m.h, layer, 0, len(ids), x.ctypes.data))
                assert rel(x, ref) < bar, (s, layer)
            hid = np.empty(cfg["width"], np.uint16)
            check(kxlib.kx_model_hidden(m.h, hid.ctypes.data))
            assert rel(to_f32(hid), record[-1][-1]) < max(bar, 1e-2)


@DTYPES
def test_model_long_decoding(kxlib, models, dtype, bar):
    cfg, w, path = models("all kinds")
    ids = KC.tokens(cfg, 500, 2)
    want = R.forward(cfg, w, ids)
    with KC.Model(path, dtype, context=500, step_tokens=40) as m:
        for cuts in ([500], [3, 1], [100, 2, 1]):
            err = KC.logit_error(m.run(ids, cuts)[:, 0], want)
            say(f"long {dtype} {cuts}: worst {err.max():.1e} at {err.argmax()}")
            assert err.max() < bar, cuts


@DTYPES
def test_model_batches_and_sequences_that_follow_each_other(kxlib, models, dtype, bar):
    cfg, w, path = models("all kinds")
    n = 60
    ids = np.stack([KC.tokens(cfg, n, 10 + b) for b in range(6)])
    want = np.stack([R.forward(cfg, w, s) for s in ids], 1)
    with KC.Model(path, dtype, batch=6, context=80) as m:
        for batch in (6, 2, 1, 5):                                    # cache rows and state of longer-gone sequences are taken over
            for cuts in ([n], [7, 1, 1, 20, 2], [1]):
                err = KC.logit_error(m.run(ids[:batch], cuts, batch), want[:, :batch])
                say(f"batch {batch} {dtype} {cuts}: worst {err.max():.1e}")
                assert err.max() < bar, (batch, cuts)
        short = m.run(ids[3][:9], [4])[:, 0]                          # shorter than what was there before
        assert KC.logit_error(short, want[:9, 3]).max() < bar


def test_wanted_places_and_the_sampled_position(kxlib, models):
    cfg, w, path = models("all kinds")
    ids = KC.tokens(cfg, 100, 3)
    want = R.forward(cfg, w, ids)
    with KC.Model(path, "float32", context=100, step_tokens=30) as m:
        m.restart()
        places = [99, 0, 31, 31, 29, 30, 5]
        assert KC.logit_error(m.extend(ids, places)[:, 0], want[places]).max() < F32_LOGITS
        last, out = np.empty((1, cfg["vocab"]), np.float32), np.zeros(1, np.uint32)
        check(kxlib.kx_model_logits(m.h, last.ctypes.data))
        check(kxlib.kx_greedy_sample(m.h, out.ctypes.data))
        assert KC.logit_error(last, want[99:]).max() < F32_LOGITS and out[0] == want[99].argmax()


def test_greedy_generation_by_library_command_line_and_host_api(kxlib, models):
    cfg, w, path = models("all kinds")
    for seed in range(20):
        p = KC.tokens(cfg, 25, 100 + seed)
        ids, gap = KC.greedy(cfg, w, p, 12, R.forward)
        if gap > 0.02:
            break
    assert gap > 0.02, "no prompt without a near-tie"
    with KC.Model(path, "float32", context=64, batch=3) as m:
        assert m.generate(p, 12)[0] == ids
        check(kxlib.kx_model_set_prefill_chunk(m.h, 2))
        assert m.generate([p, p[::-1], p], 12, batch=3)[::2] == [ids, ids]
        check(kxlib.kx_prefill(m.h, np.ascontiguousarray(p, np.uint32).ctypes.data, 1, len(p)))
        got, out = [], np.zeros(1, np.uint32)
        for _ in range(12):                                           # step by step, feeding what was sampled
            check(kxlib.kx_greedy_sample(m.h, out.ctypes.data))
            got.append(int(out[0]))
            check(kxlib.kx_decode_step(m.h, None))
        assert got == ids
    with KC.Model(path, "float32", context=64, eos_id=ids[5]) as m:
        assert m.generate(p, 12, ignore_eos=0)[0] == ids[:ids.index(ids[5])]
    arg = ["--model", path, "--prompt-tokens", ",".join(map(str, p)), "--tokens", "12", "--dtype", "float32"]
    r = subprocess.run([EXEC, *arg], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and json.loads(r.stdout) == {"status": "ok", "token_ids": ids}, r
    r = subprocess.run([EXEC, *arg, "--layers", "2", "--prefill-chunk", "5"], capture_output=True, text=True, timeout=100)
    doc = json.loads(r.stdout)
    assert (doc["layers_run"], doc["layers_in_checkpoint"]) == (2, 6) and doc["token_ids"] != ids
    assert runtime.generate_ids(model_dir=path, prompt_ids=list(map(int, p)), max_tokens=12, max_time=100, dtype="float32") == ids


def test_weights_in_32_bit_files_and_random_weights(kxlib, models, tmp_path):
    cfg, w, path = models("other sizes")
    ids = KC.tokens(cfg, 30, 4)
    mixed = KC.write(tmp_path / "m", cfg, w, f32=[n for i, n in enumerate(w) if i % 2])
    with KC.Model(path, "float32") as a, KC.Model(mixed, "float32") as b:
        assert (a.run(ids, [30]) == b.run(ids, [30])).all()
    os.unlink(tmp_path / "m" / "model.safetensors")
    with KC.Model(tmp_path / "m", "bfloat16", random_init=1, seed=7) as a:
        x = a.run(ids, [30])
        assert np.isfinite(x).all() and x.std() > 0.01 and a.shape.weight_bytes > 0


def test_what_the_design_does_not_have_is_refused(kxlib, models):
    cfg, _, path = models("heads of one")
    with KC.Model(path, "bfloat16", context=32) as m:
        m.run(KC.tokens(cfg, 5, 1), [5])
        assert kxlib.kx_model_rewind(m.h, 1) != 0 and b"recurrent" in kxlib.kx_last_error()
        assert kxlib.kx_model_set_fusion(m.h, 0) != 0 and b"not available" in kxlib.kx_last_error()


def test_trace_replay(kxlib, models, tmp_path):
    cfg, w, path = models("all kinds")
    a, b = KC.tokens(cfg, 50, 20), KC.tokens(cfg, 20, 21)
    steps = [("x", a[:30], [29, 3], []), ("x", a[30:32], [], []), ("x", a[32:], [0, 17], ["x"]), ("y", b, [19], ["y"]), ("x", b[:4], [3], ["x"])]
    lines = "".join(json.dumps({"step": i, "entries": [{"id": r, "tokens": list(map(int, t)), "want": q}], "end": e}) + "\n" for i, (r, t, q, e) in enumerate(steps))
    fa, fb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    want = {0: fa[[29, 3]], 2: fa[[32, 49]], 3: fb[[19]], 4: fb[[3]]}
    for dtype, bar in (("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)):
        out = tmp_path / dtype
        out.mkdir()
        cmd = [os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "64"]
        r = subprocess.run(cmd, input=lines, capture_output=True, text=True, timeout=100)
        assert r.returncode == 0 and r.stdout.split("\n")[:-1] == [f"done {i}" for i in range(5)], r
        assert sorted(os.listdir(out)) == [f"{i}.f32" for i in want]
        for i, ref in want.items():
            assert KC.logit_error(np.fromfile(out / f"{i}.f32", np.float32).reshape(ref.shape), ref).max() < bar, (dtype, i)
