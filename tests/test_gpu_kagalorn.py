"""The Kagalorn design on the GPU against the plain forward pass of kagalorn_oracle.py: each mechanism through its operator,
then whole models through the library's own step, cache, state, sampling and command line."""
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest

import kagalorn_case as KC
import kagalorn_oracle as K
from blok_amd import runtime
from blok_amd.lib import DevBuf, KxDeltaConfig, KxLinearArgs, KxWindowConfig, check
from kxt import dev, say

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EXEC = os.path.join(ROOT, "blok_amd", "kx-kimi-exec")
pytestmark = pytest.mark.gpu

BF16_LOGITS, F32_LOGITS = 0.04, 2e-5   # logit_error of a whole model


def portions(n, cuts):
    at, k = 0, 0
    while at < n:
        c = min(cuts[min(k, len(cuts) - 1)], n - at)
        yield at, c
        at, k = at + c, k + 1


def to_f32(a):
    return a if a.dtype == np.float32 else (a.astype(np.uint32) << 16).view(np.float32)


def rel(got, want):
    return float(np.max(np.abs(got - want)) / np.max(np.abs(want)))


# ---- attention over window and pooled blocks ------------------------------------------------------------------

class Window:
    def __init__(self, lib, heads, kv, dim, vdim, size, pool, f32, batch=1, context=512, positions=512, sink=1, gate=1, scale=None, norm=True, seed=0):
        self.lib, self.f32, self.norm, self.gate = lib, f32, norm, gate
        self.heads, self.kv, self.dim, self.vdim, self.size, self.pool, self.sink = heads, kv, dim, vdim, size, pool, sink
        self.scale, self.eps = dim ** -0.5 if scale is None else scale, 1e-5
        c = KxWindowConfig(heads, kv, dim, vdim, size, pool, sink, gate, self.scale, self.eps)
        self.h = C.c_void_p()
        check(lib.kx_window_create(C.byref(c), f32, batch, context, positions, C.byref(self.h)))
        self.cols = np.cumsum([0, heads * dim, kv * dim, kv * vdim, heads * vdim])
        r = np.random.default_rng(seed)
        self.qn, self.kn = [(1 + 0.3 * r.standard_normal(n * dim)).astype(np.float32) for n in (heads, kv)]
        self.dqn, self.dkn = dev(self.qn), dev(self.kn)

    def run(self, proj, cuts, batch=1):
        """proj [batch][n][cols]; [batch][n][heads * vdim]"""
        n, hv = proj.shape[1], self.heads * self.vdim
        out = np.empty((batch, n, hv), np.float32)
        for at, c in portions(n, cuts):
            rows = np.ascontiguousarray(proj[:, at:at + c].transpose(1, 0, 2), np.float32)     # position-major
            d = dev(rows)
            o = DevBuf(batch * c * hv * (4 if self.f32 else 2))
            check(self.lib.kx_window_run(self.h, d.ptr, rows.shape[2], *map(int, self.cols[:4]), self.dqn.ptr if self.norm else None,
                                         self.dkn.ptr if self.norm else None, batch, c, at, o.ptr, hv, None))
            got = to_f32(o.to_numpy(np.float32 if self.f32 else np.uint16, (c, batch, hv)))
            out[:, at:at + c] = got.transpose(1, 0, 2)
        return out

    def oracle(self, proj, size=None, pool=None):
        """proj [n][cols] of one sequence, in the number format's cache precision"""
        q, k, v, g = np.split(proj.astype(np.float64), self.cols[1:4], axis=1)
        if self.norm:
            q, k = K.rms(q, self.eps) * self.qn, K.rms(k, self.eps) * self.kn
        r = (lambda x: x) if self.f32 else (lambda x: KC.bf16(x).astype(np.float64))
        n = len(proj)
        q, k, v = r(q).reshape(n, self.heads, -1), r(k).reshape(n, self.kv, -1), r(v).reshape(n, self.kv, -1)
        o = np.stack([self.head(q[:, a], k[:, a // (self.heads // self.kv)], v[:, a // (self.heads // self.kv)], size or self.size, pool or self.pool)
                      for a in range(self.heads)], 1).reshape(n, -1)
        return o * K.sigmoid(g) if self.gate else o

    def head(self, q, k, v, size, pool):
        if self.sink:
            return K.pooled_window_attention(q, k, v, self.scale, size, pool)
        out = np.empty((len(q), v.shape[1]))                      # no sink: an ordinary softmax over the same keys
        for i in range(len(q)):
            toks, blocks = K.visible(i, size, pool)
            ks = [k[j] for j in toks] + [k[b * pool:(b + 1) * pool].mean(0) for b in blocks]
            vs = [v[j] for j in toks] + [v[b * pool:(b + 1) * pool].mean(0) for b in blocks]
            s = np.array(ks) @ q[i] * self.scale
            e = np.exp(s - s.max())
            out[i] = e / e.sum() @ np.array(vs)
        return out

    def close(self):
        check(self.lib.kx_window_destroy(self.h))


SCHEDULES = {"whole": [10 ** 6], "decoded": [1], "twos": [2], "mixed": [37, 2, 64, 1, 3, 129, 1, 1, 5]}

# heads, kv, dim, vdim, size, pool: sizes off every tile, windows shorter and longer than a block and than a tile of 64 keys,
# blocks of 1, many query heads per key head, keys and values wider than the matrix-core kernel takes
WINDOWS = [(4, 1, 24, 40, 10, 4), (6, 2, 40, 16, 7, 3), (2, 2, 64, 64, 16, 1), (8, 8, 33, 31, 5, 8), (3, 1, 128, 128, 64, 16), (5, 5, 96, 160, 100, 7),
           (32, 1, 16, 8, 1, 5), (4, 2, 300, 20, 70, 6), (2, 1, 20, 270, 33, 2), (4, 4, 130, 250, 65, 64)]


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("case", WINDOWS, ids=lambda c: "-".join(map(str, c)))
def test_window_attention_in_portions_of_every_kind(kxlib, case, f32):
    n = 200
    r = np.random.default_rng(5)
    w = Window(kxlib, *case, f32)
    proj = r.standard_normal((1, n, w.cols[-1])).astype(np.float32)
    proj[..., :w.cols[2]] *= 1.7
    want = w.oracle(proj[0])
    for name, cuts in SCHEDULES.items():
        say(f"window {case} f32={f32} {name}")
        assert rel(w.run(proj, cuts)[0], want) < (3e-5 if f32 else 2e-2), name
    w.close()


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("size, pool", [(12, 4), (9, 5), (64, 16), (70, 64)])
def test_one_key_that_stands_out_at_every_edge(kxlib, size, pool, f32):
    """Position i's query meets one early key that scores far above all others: with the key just inside the window, just
    outside, in the last block that is seen, in the first that is not, in the first block and at position 0; once where a
    block has just come into sight, once where the next position brings one."""
    n, dim, vdim = 260, 48, 16
    w = Window(kxlib, 1, 1, dim, vdim, size, pool, f32, norm=False, gate=0, scale=1.0)
    r = np.random.default_rng(3)
    just = next(i for i in range(n - 3, 0, -1) if (i - size + 1) % pool == 0)          # its last block has just come into sight
    early = next(i for i in range(n - 3, 0, -1) if (i - size + 2) % pool == 0)         # the next position will see one block more
    cases = [(just, "inside", just - size + 1), (just, "outside", just - size), (just, "own", just), (just, "start", 0), (just, "first block", pool - 1),
             (just, "block start", just - size + 1 - pool), (early, "inside", early - size + 1), (early, "outside", early - size),
             (early, "first unseen", early - size + 2 - pool), (early, "last block", early - size + 1 - pool)]
    for i, name, j in cases:
        say(f"edge {name} of {i} size={size} pool={pool} f32={f32}")
        proj = np.concatenate([0.05 * r.standard_normal((n, 2 * dim)), r.standard_normal((n, vdim)), np.zeros((n, vdim))], 1).astype(np.float32)
        e = np.eye(dim)[7]
        proj[i, :dim] = 4.0 * e
        proj[j, dim:2 * dim] += (2.0 if j >= i - size + 1 else 2.0 * pool) * e        # a block's mean has it over pool
        want = w.oracle(proj)
        if name not in ("own", "start", "first block", "last block"):               # the case tells a window or a block that is off by one
            assert max(rel(w.oracle(proj, size=x)[i], want[i]) for x in (size - 1, size + 1)) > 0.2, name
        for s in ("whole", "decoded", "mixed"):
            got = w.run(proj[None], SCHEDULES[s])[0]
            assert rel(got[i], want[i]) < (3e-5 if f32 else 2e-2), (name, s)
    w.close()


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
def test_ring_that_is_written_over_many_times(kxlib, f32):
    """A cache for steps of few positions: its ring is a few tiles long and goes round under a long sequence."""
    for size, pool, positions in ((20, 8, 3), (64, 4, 64), (5, 40, 2), (100, 16, 30)):
        n = 700
        w = Window(kxlib, 2, 1, 20, 12, size, pool, f32, context=n, positions=positions)
        proj = np.random.default_rng(size).standard_normal((1, n, w.cols[-1])).astype(np.float32)
        want = w.oracle(proj[0])
        for cuts in ([positions], [1], [positions, 1, 2, 1]):
            say(f"ring size={size} pool={pool} positions={positions} cuts={cuts} f32={f32}")
            assert rel(w.run(proj, cuts)[0], want) < (3e-5 if f32 else 2e-2)
        w.close()


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
def test_sink_gate_norm_and_pool_are_parameters(kxlib, f32):
    n = 90
    for sink, gate, norm, pool in ((0, 1, True, 3), (1, 0, False, 3), (0, 0, False, 0), (1, 1, True, 0)):
        w = Window(kxlib, 4, 2, 24, 24, 20, pool, f32, sink=sink, gate=gate, norm=norm, scale=0.4)
        proj = np.random.default_rng(9).standard_normal((1, n, w.cols[-1])).astype(np.float32)
        want = w.oracle(proj[0], pool=pool or 10 ** 6)
        for s in ("whole", "decoded", "mixed"):
            assert rel(w.run(proj, SCHEDULES[s])[0], want) < (3e-5 if f32 else 2e-2), (sink, gate, norm, pool, s)
        w.close()


def test_sink_shows_where_every_score_is_low(kxlib):
    w = Window(kxlib, 1, 1, 16, 8, 6, 2, 1, norm=False, gate=0, scale=1.0)
    proj = np.zeros((1, 40, w.cols[-1]), np.float32)
    proj[..., 0], proj[..., 16], proj[..., 32:40] = 1.0, -6.0, 1.0                 # every score is -6, every value 1
    got = w.run(proj, [10 ** 6])[0]
    keys = np.array([sum(map(len, K.visible(i, 6, 2))) for i in range(40)])
    assert np.allclose(got[:, 0], keys * np.exp(-6.0) / (1 + keys * np.exp(-6.0)), rtol=1e-4)
    w.close()


def test_window_batch_equals_each_alone(kxlib):
    for f32, exact in ((1, 1e-5), (0, 1e-2)):
        w = Window(kxlib, 4, 2, 24, 40, 30, 4, f32, batch=6, context=160, positions=160)
        proj = np.random.default_rng(2).standard_normal((6, 150, w.cols[-1])).astype(np.float32)
        together = {s: w.run(proj, SCHEDULES[s], 6) for s in ("whole", "mixed", "decoded")}
        for b in range(6):
            alone = w.run(proj[b:b + 1], [10 ** 6])[0]
            for s, t in together.items():
                assert rel(t[b], alone) < exact, (f32, s, b)
        w.close()


# ---- delta rule -----------------------------------------------------------------------------------------------

class Delta:
    def __init__(self, lib, heads, kv, dim, vdim, taps, batch=1, positions=512, seed=0):
        self.lib, self.shape = lib, (heads, kv, dim, vdim, taps)
        c = KxDeltaConfig(heads, kv, dim, vdim, taps, 1e-6)
        self.h = C.c_void_p()
        check(lib.kx_delta_create(C.byref(c), batch, positions, C.byref(self.h)))
        self.cols = np.cumsum([0, kv * dim, kv * dim, heads * vdim, heads, heads])
        r = np.random.default_rng(seed)
        self.conv = r.standard_normal((int(self.cols[3]), taps)).astype(np.float32)
        self.a_log, self.dt = (0.7 * r.standard_normal(heads) - 1).astype(np.float32), r.standard_normal(heads).astype(np.float32)
        self.d = [dev(x) for x in (self.conv, self.a_log, self.dt)]

    def run(self, proj, cuts, batch=1):
        n, hv = proj.shape[1], self.shape[0] * self.shape[3]
        check(self.lib.kx_delta_restart(self.h, None))
        out = np.empty((batch, n, hv), np.float32)
        for at, c in portions(n, cuts):
            rows = np.ascontiguousarray(proj[:, at:at + c].transpose(1, 0, 2), np.float32)
            d, o = dev(rows), DevBuf(batch * c * hv * 4)
            check(self.lib.kx_delta_run(self.h, d.ptr, rows.shape[2], *map(int, self.cols[:5]), *[x.ptr for x in self.d], batch, c, o.ptr, None))
            out[:, at:at + c] = o.to_numpy(np.float32, (c, batch, hv)).transpose(1, 0, 2)
        return out

    def oracle(self, proj):
        heads, kv, dim, vdim, _ = self.shape
        n = len(proj)
        qkv, b, a = np.split(proj.astype(np.float64), self.cols[3:5], axis=1)
        qkv = K.silu(K.causal_conv(qkv, self.conv.astype(np.float64)))
        q, k, v = np.split(qkv, self.cols[1:3], axis=1)
        q, k, v = K.unit(q.reshape(n, kv, dim)) * dim ** -0.5, K.unit(k.reshape(n, kv, dim)), v.reshape(n, heads, vdim)
        beta, g = K.sigmoid(b), np.exp(-np.exp(self.a_log.astype(np.float64)) * K.softplus(a + self.dt))
        return np.stack([K.delta_rule(q[:, h // (heads // kv)], k[:, h // (heads // kv)], v[:, h], beta[:, h], g[:, h])[0] for h in range(heads)],
                        1).reshape(n, -1)

    def close(self):
        check(self.lib.kx_delta_destroy(self.h))


DELTAS = [(4, 2, 16, 24, 4), (3, 3, 8, 5, 1), (6, 1, 40, 33, 2), (2, 2, 64, 64, 3), (4, 4, 100, 70, 4), (2, 1, 128, 128, 5), (1, 1, 200, 17, 4), (2, 2, 256, 40, 3)]


@pytest.mark.parametrize("case", DELTAS, ids=lambda c: "-".join(map(str, c)))
def test_delta_rule_in_portions_of_every_kind(kxlib, case):
    n = 150
    d = Delta(kxlib, *case)
    proj = np.random.default_rng(4).standard_normal((1, n, d.cols[-1])).astype(np.float32)
    want = d.oracle(proj[0])
    for name, cuts in SCHEDULES.items():
        say(f"delta {case} {name}")
        assert rel(d.run(proj, cuts)[0], want) < 3e-5, name
    d.close()


def test_delta_state_holds_a_write_for_long_and_forgets_what_is_overwritten(kxlib):
    """No decay to speak of: a value written at the start under one key is read back hundreds of tokens later, and a second
    write under the same key replaces it (that is what the rule's subtraction is for)."""
    heads, kv, dim, vdim, taps = 1, 1, 32, 8, 1
    d = Delta(kxlib, heads, kv, dim, vdim, taps)
    d.conv[:] = 1.0
    d.d[0].upload(d.conv)
    d.d[1].upload(np.array([-20.0], np.float32))
    d.a_log[:] = -20.0
    n = 400
    proj = np.zeros((1, n, d.cols[-1]), np.float32)
    proj[..., d.cols[3]] = -30.0                                  # beta = 0 ...
    for t, val in ((3, 2.0), (200, -1.0)):
        proj[0, t, d.cols[3]] = 30.0                              # ... but at the two writes, under key 5
        proj[0, t, d.cols[1] + 5] = 20.0
        proj[0, t, d.cols[2]:d.cols[3]] = val
    proj[..., 5] = 20.0                                           # every query reads key 5
    want = d.oracle(proj[0])
    assert abs(want[199, 0] * dim ** 0.5 - K.silu(2.0)) < 1e-5 and abs(want[399, 0] * dim ** 0.5 - K.silu(-1.0)) < 1e-5
    for name, cuts in SCHEDULES.items():
        assert rel(d.run(proj, cuts)[0], want) < 1e-5, name
    d.close()


def test_delta_batch_equals_each_alone(kxlib):
    d = Delta(kxlib, 4, 2, 48, 40, 4, batch=5)
    proj = np.random.default_rng(6).standard_normal((5, 90, d.cols[-1])).astype(np.float32)
    for s in ("whole", "mixed", "decoded"):
        together = d.run(proj, SCHEDULES[s], 5)
        for b in range(5):
            assert rel(together[b], d.run(proj[b:b + 1], SCHEDULES[s])[0]) < 1e-6, (s, b)
    d.close()


# ---- products with their rows and epilogues --------------------------------------------------------------------

def _matrix(w, f32):
    ld = -(-w.shape[1] // 64) * 64
    pad = np.zeros((w.shape[0], ld), np.float32)
    pad[:, :w.shape[1]] = w
    return dev(pad if f32 else (pad.view(np.uint32) >> 16).astype(np.uint16)), ld


def _rounded(x, f32):
    return np.asarray(x, np.float64) if f32 else KC.bf16(x).astype(np.float64)


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("tokens", [1, 2, 3, 4, 5, 33, 64, 65, 200])
def test_products_build_their_rows_and_update_the_streams(kxlib, tokens, f32):
    r = np.random.default_rng(tokens)
    tol = 2e-5 if f32 else 1.5e-2
    for rows, cols, streams, groups in ((70, 96, 2, 2), (257, 120, 1, 1), (33, 1000, 4, 40), (130, 576, 3, 3)):
        say(f"product {rows}x{cols} tokens={tokens} streams={streams} groups={groups} f32={f32}")
        w = KC.bf16(r.standard_normal((rows, cols)) * cols ** -0.5)
        dw, ld = _matrix(w, f32)
        es = 4 if f32 else 2
        scratch = DevBuf(tokens * ld * es)
        base = dict(f32=f32, tokens=tokens, rows=rows, cols=cols, ld=ld, streams=streams, groups=groups, eps=1e-5, d_w=dw.ptr)

        def run(out, **kw):
            a = KxLinearArgs(**base)
            for k, v in kw.items():
                setattr(a, k, v)
            a.d_out = out.ptr
            check(kxlib.kx_linear_run(C.byref(a), scratch.ptr, None))
            check(kxlib.kx_sync(None))

        # a grouped norm of weighted streams in front, stored
        x = r.standard_normal((tokens, streams, cols)).astype(np.float32)
        win, wn = r.standard_normal(streams).astype(np.float32), (1 + 0.3 * r.standard_normal(cols)).astype(np.float32)
        dx, din, dn = dev(x), dev(win), dev(wn)
        h = _rounded(K.grouped_rms_norm(K.hyper_read(x.transpose(1, 0, 2).astype(np.float64), win), wn, groups, 1e-5), f32)
        out = dev(np.full((tokens, rows + 3), 7.0, np.float32))
        run(out, row_kind=1, epilogue=0, d_streams_in=dx.ptr, d_in=din.ptr, d_norm=dn.ptr, out_ld=rows + 3)
        got = out.to_numpy(np.float32, (tokens, rows + 3))
        assert rel(got[:, :rows], h @ w.T) < tol and (got[:, rows:] == 7.0).all()

        # a row from memory, the product written to all streams
        ld_x = ld + 64
        xr = np.zeros((tokens, ld_x), np.float32)
        xr[:, :cols] = KC.bf16(r.standard_normal((tokens, cols)))
        dxr = dev(xr if f32 else (xr.view(np.uint32) >> 16).astype(np.uint16))
        s0 = r.standard_normal((tokens, streams, rows)).astype(np.float32)
        mix, ow = r.standard_normal((streams, streams)).astype(np.float32), r.standard_normal(streams).astype(np.float32)
        ds, dm, do = dev(s0), dev(mix), dev(ow)
        run(ds, row_kind=0, epilogue=2, d_x=dxr.ptr, x_ld=ld_x, d_mix=dm.ptr, d_outw=do.ptr)
        want = K.hyper_write(s0.transpose(1, 0, 2).astype(np.float64), mix, ow, xr[:, :cols].astype(np.float64) @ w.T).transpose(1, 0, 2)
        assert rel(ds.to_numpy(np.float32, s0.shape), want) < tol
        if streams == 1:                                          # a plain residual
            ds = dev(s0)
            run(ds, row_kind=0, epilogue=2, d_x=dxr.ptr, x_ld=ld_x)
            assert rel(ds.to_numpy(np.float32, s0.shape)[:, 0], s0[:, 0] + xr[:, :cols].astype(np.float64) @ w.T) < tol

        # the delta rule's gated read-out in front
        heads, vdim = (4, cols // 4)
        o, g = r.standard_normal((tokens, cols)).astype(np.float32), r.standard_normal((tokens, cols + 5)).astype(np.float32)
        wv = (1 + 0.3 * r.standard_normal(vdim)).astype(np.float32)
        d_o, dg, dwv = dev(o), dev(g), dev(wv)
        h = K.rms(o.astype(np.float64).reshape(tokens, heads, vdim), 1e-5) * wv * K.silu(g[:, :cols].astype(np.float64)).reshape(tokens, heads, vdim)
        run(out, row_kind=2, epilogue=0, d_o=d_o.ptr, d_gate=dg.ptr, gate_ld=cols + 5, heads=heads, vdim=vdim, d_norm=dwv.ptr, out_ld=rows + 3)
        assert rel(out.to_numpy(np.float32, (tokens, rows + 3))[:, :rows], _rounded(h.reshape(tokens, cols), f32) @ w.T) < tol


@pytest.mark.parametrize("f32", [1, 0], ids=["f32", "bf16"])
@pytest.mark.parametrize("tokens", [1, 3, 9, 64, 130])
def test_clamped_gated_activation(kxlib, tokens, f32):
    r = np.random.default_rng(tokens)
    for ff, cols in ((72, 96), (32, 64), (150, 200)):
        blocks = -(-ff // 32)
        gate, up = (KC.bf16(3.0 * r.standard_normal((ff, cols)) * cols ** -0.5) for _ in range(2))
        packed = np.zeros((blocks, 2, 32, cols), np.float32)
        for half, m in ((0, gate), (1, up)):
            full = np.zeros((blocks * 32, cols), np.float32)
            full[:ff] = m
            packed[:, half] = full.reshape(blocks, 32, cols)
        dw, ld = _matrix(packed.reshape(-1, cols), f32)
        x = np.zeros((tokens, ld), np.float32)
        x[:, :cols] = KC.bf16(r.standard_normal((tokens, cols)))
        dx = dev(x if f32 else (x.view(np.uint32) >> 16).astype(np.uint16))
        out_ld = blocks * 32 + 8
        out = DevBuf(tokens * out_ld * (4 if f32 else 2))
        a = KxLinearArgs(f32=f32, tokens=tokens, rows=blocks * 64, cols=cols, ld=ld, row_kind=0, epilogue=1, streams=1, groups=1, x_ld=ld, out_ld=out_ld,
                         limit=1.5, alpha=1.702, bias=1.0, d_w=dw.ptr, d_x=dx.ptr, d_out=out.ptr)
        check(kxlib.kx_linear_run(C.byref(a), None, None))
        check(kxlib.kx_sync(None))
        got = to_f32(out.to_numpy(np.float32 if f32 else np.uint16, (tokens, out_ld)))[:, :ff]
        w = {"gate": gate.astype(np.float64), "up": up.astype(np.float64), "down": np.eye(ff)}
        want = K.clamped_glu(x[:, :cols].astype(np.float64), w, "", 1.5)
        assert np.abs(want).max() > 3.47 and rel(got, want) < (2e-5 if f32 else 1e-2)     # both clamps are reached


# ---- models -----------------------------------------------------------------------------------------------------

MODELS = {
    "mixed": KC.config([KC.attention(), KC.delta(), KC.attention(heads=6, kv_heads=3, dim=40, vdim=32, size=20, pool=5), KC.delta(heads=6, kv_heads=1, conv=2)]),
    "three streams, no feed-forward": KC.config([KC.delta(ff=0), KC.attention(ff=0, pool=1), KC.delta(kv_heads=4, conv=1, ff=50)], width=120, streams=3, groups=5),
    "one stream": KC.config([KC.attention(heads=2, kv_heads=2, dim=64, vdim=70, size=33, pool=8, scale=0.3, limit=0.7), KC.delta(heads=2, kv_heads=2, dim=72, vdim=16)],
                            width=80, streams=1, groups=1, eps=1e-3, vocab=301),
    "one head": KC.config([KC.attention(heads=1, kv_heads=1, dim=8, vdim=8, size=1, pool=2, ff=32), KC.delta(heads=1, kv_heads=1, dim=4, vdim=4, conv=3, ff=32)],
                          width=64, streams=4, groups=8, vocab=33),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            cfg = MODELS[name]
            w = KC.weights(cfg, sum(map(ord, name)))
            made[name] = cfg, w, KC.write(tmp_path_factory.mktemp("kagalorn"), cfg, w)
        return made[name]
    return get


@pytest.mark.parametrize("dtype, bar", [("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)])
@pytest.mark.parametrize("name", MODELS)
def test_model_whole_decoded_and_in_portions(kxlib, models, name, dtype, bar):
    cfg, w, path = models(name)
    if dtype == "bfloat16" and name == "one head":
        bar = 0.1          # unit vectors of 4 elements: nothing averages the rounding of a projection's input
    ids = KC.tokens(cfg, 170, 1)
    record = []
    want = K.forward(cfg, w, ids, record)
    with KC.Model(path, dtype, context=170) as m:
        check(kxlib.kx_model_set_residual_record(m.h, 1))
        for s, cuts in dict(SCHEDULES, late=[140, 1]).items():
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


@pytest.mark.parametrize("dtype, bar", [("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)])
def test_model_long_decoding_over_a_short_ring(kxlib, models, dtype, bar):
    cfg, w, path = models("mixed")
    ids = KC.tokens(cfg, 600, 2)
    want = K.forward(cfg, w, ids)
    with KC.Model(path, dtype, context=600, step_tokens=40) as m:     # a ring of two tiles per attention layer
        for cuts in ([600], [3, 1], [100, 2, 1]):
            assert KC.logit_error(m.run(ids, cuts)[:, 0], want).max() < bar, cuts


@pytest.mark.parametrize("dtype, bar", [("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)])
def test_model_batches_and_sequences_that_follow_each_other(kxlib, models, dtype, bar):
    cfg, w, path = models("mixed")
    n = 60
    ids = np.stack([KC.tokens(cfg, n, 10 + b) for b in range(6)])
    want = np.stack([K.forward(cfg, w, s) for s in ids], 1)
    with KC.Model(path, dtype, batch=6, context=80) as m:
        for batch in (6, 2, 1, 5):                                    # cache rows and state of longer-gone sequences are taken over
            for cuts in ([n], [7, 1, 1, 20, 2], [1]):
                err = KC.logit_error(m.run(ids[:batch], cuts, batch), want[:, :batch])
                assert err.max() < bar, (batch, cuts)
        short = m.run(ids[3][:9], [4])[:, 0]                          # shorter than what was there before
        assert KC.logit_error(short, want[:9, 3]).max() < bar


def test_wanted_places_and_the_sampled_position(kxlib, models):
    cfg, w, path = models("mixed")
    ids = KC.tokens(cfg, 100, 3)
    want = K.forward(cfg, w, ids)
    with KC.Model(path, "float32", context=100, step_tokens=30) as m:
        m.restart()
        got = m.extend(ids, [99, 0, 31, 31, 29, 30, 5])[:, 0]         # any order, across the steps the call is cut into
        assert KC.logit_error(got, want[[99, 0, 31, 31, 29, 30, 5]]).max() < F32_LOGITS
        last, out = np.empty((1, cfg["vocab"]), np.float32), np.zeros(1, np.uint32)
        check(kxlib.kx_model_logits(m.h, last.ctypes.data))
        check(kxlib.kx_greedy_sample(m.h, out.ctypes.data))
        assert KC.logit_error(last, want[99:]).max() < F32_LOGITS and out[0] == want[99].argmax()
        m.restart()
        assert m.extend(ids[:10], []).shape == (0, 1, cfg["vocab"])
        assert KC.logit_error(m.extend(ids[10:12])[:, 0], want[10:12]).max() < F32_LOGITS


def _prompt_with_gap(cfg, w, n):
    for seed in range(20):
        p = KC.tokens(cfg, 25, 100 + seed)
        ids, gap = KC.greedy(cfg, w, p, n)
        if gap > 0.02:
            return p, ids
    raise AssertionError("no prompt without a near-tie")


def test_greedy_generation_by_library_command_line_and_host_api(kxlib, models):
    cfg, w, path = models("three streams, no feed-forward")
    p, ids = _prompt_with_gap(cfg, w, 12)
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
    assert (doc["layers_run"], doc["layers_in_checkpoint"]) == (2, 3) and doc["token_ids"] != ids
    assert runtime.generate_ids(model_dir=path, prompt_ids=list(map(int, p)), max_tokens=12, max_time=100, dtype="float32") == ids


def test_weights_in_32_bit_files_and_random_weights(kxlib, models, tmp_path):
    cfg, w, path = models("one stream")
    ids = KC.tokens(cfg, 30, 4)
    mixed = KC.write(tmp_path / "m", cfg, w, f32=[n for i, n in enumerate(w) if i % 2])
    with KC.Model(path, "float32") as a, KC.Model(mixed, "float32") as b:
        assert (a.run(ids, [30]) == b.run(ids, [30])).all()
    os.unlink(tmp_path / "m" / "model.safetensors")
    with KC.Model(tmp_path / "m", "bfloat16", random_init=1, seed=7) as a:
        x = a.run(ids, [30])
        assert np.isfinite(x).all() and x.std() > 0.01 and a.shape.weight_bytes > 0


def test_what_the_design_does_not_have_is_refused(kxlib, models):
    cfg, _, path = models("one head")
    with KC.Model(path, "bfloat16", context=32) as m:
        m.run(KC.tokens(cfg, 5, 1), [5])
        for rc, word in ((kxlib.kx_model_rewind(m.h, 1), b"recurrent"), (kxlib.kx_model_set_fusion(m.h, 0), b"not available"),
                         (kxlib.kx_model_latent(m.h, 0, 0, 0, 1, None), b"not available"), (kxlib.kx_model_set_prefill_chunk(m.h, 33), b"32")):
            assert rc != 0
        assert b"outside" in kxlib.kx_last_error()
        assert kxlib.kx_model_rewind(m.h, 0) == 0
        ids = np.zeros(30, np.uint32)
        assert kxlib.kx_extend(m.h, ids.ctypes.data, 28, None, 0, None) != 0 and b"27" in kxlib.kx_last_error()
        ids[0] = cfg["vocab"]
        assert kxlib.kx_extend(m.h, ids.ctypes.data, 1, None, 0, None) != 0 and b"vocabulary" in kxlib.kx_last_error()
        assert kxlib.kx_restart(m.h, 2) != 0


def test_trace_replay(kxlib, models, tmp_path):
    cfg, w, path = models("mixed")
    a, b = KC.tokens(cfg, 50, 20), KC.tokens(cfg, 20, 21)
    steps = [("x", a[:30], [29, 3], []), ("x", a[30:32], [], []), ("x", a[32:], [0, 17], ["x"]), ("y", b, [19], ["y"]), ("x", b[:4], [3], ["x"])]
    lines = "".join(json.dumps({"step": i, "entries": [{"id": r, "tokens": list(map(int, t)), "want": q}], "end": e}) + "\n" for i, (r, t, q, e) in enumerate(steps))
    fa, fb = K.forward(cfg, w, a), K.forward(cfg, w, b)
    want = {0: fa[[29, 3]], 2: fa[[32, 49]], 3: fb[[19]], 4: fb[[3]]}
    for dtype, bar in (("float32", F32_LOGITS), ("bfloat16", BF16_LOGITS)):
        out = tmp_path / dtype
        out.mkdir()
        cmd = [os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out), "--max-tokens", "64"]
        r = subprocess.run(cmd, input=lines, capture_output=True, text=True, timeout=400)
        assert r.returncode == 0 and r.stdout.split("\n")[:-1] == [f"done {i}" for i in range(5)], r
        assert sorted(os.listdir(out)) == [f"{i}.f32" for i in want]
        for i, ref in want.items():
            assert KC.logit_error(np.fromfile(out / f"{i}.f32", np.float32).reshape(ref.shape), ref).max() < bar, (dtype, i)
    two = json.dumps({"step": 0, "entries": [{"id": "a", "tokens": [1], "want": []}, {"id": "b", "tokens": [1], "want": []}], "end": []})
    r = subprocess.run(cmd, input=two + "\n", capture_output=True, text=True, timeout=400)
    assert r.returncode == 1 and "one request at a time" in r.stderr
