"""Small Kagalorn models for tests: configurations, random weights, the files, and a handle on the opened model."""
import ctypes as C
import json
import os
import struct

import numpy as np

import kagalorn_oracle as K
from blok_amd.lib import DTYPES, KxModelShape, KxOpenOptions, check, kx


def bf16(x):
    """x rounded to bf16 (nearest, ties to even), as float32."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def attention(heads=4, kv_heads=2, dim=24, vdim=20, size=12, pool=4, scale=None, ff=72, limit=1.5):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                           "mask": {"size": size, "pool": pool}, "scale": dim ** -0.5 if scale is None else scale},
            "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def delta(heads=4, kv_heads=2, dim=16, vdim=24, conv=4, ff=72, limit=1.5):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def config(layers, vocab=150, width=96, streams=2, groups=2, eps=1e-5):
    return {"architecture": "Kagalorn", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps, "groups": groups},
            "layers": layers}


def shapes(cfg):
    """name -> shape of every tensor."""
    w, s = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h, g, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        t = {"norm1": (w,), "mix.o": (w, h * v), "mix.g": (h * v, w), "mix.k": (g * d, w)}
        if layer["type"] == "attention":
            t.update({"mix.q": (h * d, w), "mix.v": (g * v, w), "mix.q.norm": (h * d,), "mix.k.norm": (g * d,)})
        else:
            t.update({"mix.q": (g * d, w), "mix.v": (h * v, w), "mix.b": (h, w), "mix.a": (h, w), "mix.A_log": (h,), "mix.dt_bias": (h,),
                      "mix.norm": (v,), "mix.q.conv": (g * d, m["conv"]), "mix.k.conv": (g * d, m["conv"]), "mix.v.conv": (h * v, m["conv"])})
        if layer["mlp"]:
            f = layer["mlp"]["ff"]
            t.update({"norm2": (w,), "mlp.gate": (f, w), "mlp.up": (f, w), "mlp.down": (w, f)})
        for q in (1, 2) if layer["mlp"] else (1,):
            t.update({f"hc{q}.in": (s,), f"hc{q}.out": (s,), f"hc{q}.mix": (s, s)})
        out.update({p + k: x for k, x in t.items()})
    return out


def weights(cfg, seed):
    """Random weights with bf16 values, large enough that every mechanism matters in the logits."""
    r = np.random.default_rng(seed)
    w = {}
    for name, shape in shapes(cfg).items():
        leaf = name.split(".", 1)[-1]
        z = r.standard_normal(shape)
        if leaf.startswith("hc"):
            z = {"in": 0.6 + 0.3 * z, "out": 1.0 + 0.3 * z, "mix": np.eye(shape[0], *shape[1:]) + 0.2 * z}[leaf[4:]]
        elif leaf.endswith("conv"):
            z = 0.4 * z + (np.arange(shape[1]) == shape[1] - 1)
        elif leaf.endswith("A_log"):
            z = 0.7 * z - 1.0
        elif leaf.endswith("dt_bias"):
            z = 0.5 * z - 1.5
        elif len(shape) == 1:
            z = 1.0 + 0.3 * z
        elif name != "embed":
            z = z * shape[1] ** -0.5 * (2.0 if leaf.endswith((".q", ".k", ".a", ".b")) else 1.0)
        w[name] = bf16(z).astype(np.float64)
    return w


def write(path, cfg, w, f32=()):
    """config.json and model.safetensors; tensors named in `f32` are stored as F32."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {"__metadata__": {"format": "pt"}}, [], 0
    for name, x in w.items():
        a = np.asarray(x, np.float32)
        blob = a.tobytes() if name in f32 else (a.view(np.uint32) >> 16).astype(np.uint16).tobytes()
        head[name] = {"dtype": "F32" if name in f32 else "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(blob)]}
        blobs.append(blob)
        at += len(blob)
    text = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text + b"".join(blobs))
    return str(path)


class Model:
    """kx_model_open with the calls the tests make."""

    def __init__(self, path, dtype="float32", batch=1, context=512, step_tokens=2048, **opt):
        self.lib = kx()
        o = KxOpenOptions()
        check(self.lib.kx_open_options_default(C.byref(o)))
        o.dtype, o.max_batch, o.max_context, o.step_tokens = DTYPES[dtype], batch, context, step_tokens
        for k, v in opt.items():
            setattr(o, k, v)
        self.h = C.c_void_p()
        check(self.lib.kx_model_open(str(path).encode(), C.byref(o), C.byref(self.h)))
        self.shape = KxModelShape()
        check(self.lib.kx_model_info(self.h, C.byref(self.shape)))

    def restart(self, batch=1):
        self.batch = batch
        check(self.lib.kx_restart(self.h, batch))

    def extend(self, tokens, want=None):
        """tokens [n] or [batch][n]; logits [n][batch][vocab] (or of the places in `want`)."""
        ids = np.ascontiguousarray(np.asarray(tokens, np.uint32).reshape(self.batch, -1))
        n = ids.shape[1]
        want = np.arange(n, dtype=np.int32) if want is None else np.asarray(want, np.int32)
        out = np.empty((len(want), self.batch, self.shape.vocab), np.float32)
        check(self.lib.kx_extend(self.h, ids.ctypes.data, n, want.ctypes.data, len(want), out.ctypes.data))
        return out

    def run(self, tokens, cuts, batch=1):
        """A new sequence (or batch of them) in portions of the given sizes, the last one repeated to the end."""
        self.restart(batch)
        ids = np.asarray(tokens, np.uint32).reshape(batch, -1)
        out, at, k = [], 0, 0
        while at < ids.shape[1]:
            n = min(cuts[min(k, len(cuts) - 1)], ids.shape[1] - at)
            out.append(self.extend(ids[:, at:at + n]))
            at, k = at + n, k + 1
        return np.concatenate(out)

    def generate(self, prompt, n, ignore_eos=1, batch=1):
        p = np.ascontiguousarray(np.asarray(prompt, np.uint32).reshape(batch, -1))
        out, counts = np.zeros((batch, n), np.uint32), np.zeros(batch, np.int32)
        check(self.lib.kx_generate(self.h, p.ctypes.data, batch, p.shape[1], n, ignore_eos, out.ctypes.data, counts.ctypes.data))
        return [list(map(int, out[b, :counts[b]])) for b in range(batch)]

    def close(self):
        if self.h:
            check(self.lib.kx_model_destroy(self.h))
            self.h = None

    def __enter__(self):
        return self

    def __exit__(self, *_):
        self.close()


def logit_error(got, want):
    """Per position: root mean square of the difference (mean taken off), over the root mean square of the logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt(np.mean((want - want.mean(-1, keepdims=True)) ** 2))


def tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n)


def greedy(cfg, w, prompt, n, forward=K.forward):
    """Greedy continuation by the plain forward pass, whole sequence every time, and the smallest top-2 gap met."""
    ids, gap = list(map(int, prompt)), np.inf
    for _ in range(n):
        row = forward(cfg, w, ids)[-1]
        top = np.sort(row)[-2:]
        gap = min(gap, (top[1] - top[0]) / np.std(row))
        ids.append(int(np.argmax(row)))
    return ids[len(prompt):], gap
