"""Small Rapitar models for tests: configurations and random weights (files and opened models: kagalorn_case.py)."""
import numpy as np

from kagalorn_case import bf16

RANK = 12   # of the time mixing's decay projection, which only the tensors' shapes tell


def mamba2(heads=6, vdim=20, state=24, groups=2, norm_groups=3, conv=4, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}, "mlp": mlp}


def wkv(heads=3, dim=24, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": mlp}


def latent(heads=3, dim=20, rot_dim=12, vdim=28, q_rank=40, kv_rank=36, scale=None, base=1000.0, dims=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"dims": rot_dim if dims is None else dims, "base": base}}}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def moe(ff=24, experts=7, top=2):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers, vocab=150, width=96, eps=1e-5):
    return {"architecture": "Rapitar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def shapes(cfg):
    """name -> shape of every tensor."""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        m, mlp = layer["mixer"], layer["mlp"]
        h = m["heads"]
        t = {"norm1": (w,)}
        if layer["type"] == "mamba2":
            inner, bc = h * m["vdim"], 2 * m["groups"] * m["state"]
            t.update({"mix.in": (2 * inner + bc + h, w), "mix.conv": (inner + bc, m["conv"]), "mix.conv.b": (inner + bc,), "mix.dt_bias": (h,),
                      "mix.A_log": (h,), "mix.D": (h,), "mix.norm": (inner,), "mix.o": (w, inner)})
        elif layer["type"] == "wkv":
            hd = h * m["dim"]
            t.update({"mix.mu." + c: (w,) for c in "rkvgw"})
            t.update({"mix." + c: (hd, w) for c in "rkvg"})
            t.update({"mix.w1": (RANK, w), "mix.w2": (hd, RANK), "mix.w0": (hd,), "mix.u": (h, m["dim"]), "mix.norm": (hd,), "mix.o": (w, hd)})
        else:
            t.update({"mix.dq": (m["q_rank"], w), "mix.dq.norm": (m["q_rank"],), "mix.uq": (h * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                      "mix.dkv": (m["kv_rank"] + m["rot_dim"], w), "mix.dkv.norm": (m["kv_rank"],), "mix.uk": (h * m["dim"], m["kv_rank"]),
                      "mix.uv": (h * m["vdim"], m["kv_rank"]), "mix.sink": (h,), "mix.g": (h * m["vdim"], w), "mix.o": (w, h * m["vdim"])})
        if mlp and mlp["kind"] == "dense":
            t.update({"mlp.up": (mlp["ff"], w), "mlp.down": (w, mlp["ff"])})
        elif mlp:
            e, f = mlp["router"]["experts"], mlp["expert"]["ff"]
            t.update({"mlp.router": (e, w), "mlp.router.b": (e,)})
            for j in range(e):
                t.update({f"mlp.e{j}.gate": (f, w), f"mlp.e{j}.up": (f, w), f"mlp.e{j}.down": (w, f)})
        out.update({f"l{i}.{k}": x for k, x in t.items()})
    return out


def weights(cfg, seed):
    """Random weights with bf16 values, large enough that every mechanism matters in the logits.

    The first channels, as many as the most experts of a layer, are the routers': every token's embedding holds evenly
    spaced levels there in an order of its own, no layer writes to them, and the routers read nothing else.  So no
    rounding changes which experts are chosen."""
    r = np.random.default_rng(seed)
    w = {}
    for name, shape in shapes(cfg).items():
        leaf = name.split(".", 1)[-1]
        z = r.standard_normal(shape)
        if name == "embed":
            pass
        elif leaf == "mix.conv":
            z = 0.4 * z + (np.arange(shape[1]) == shape[1] - 1)
        elif leaf == "mix.A_log":
            z = 0.9 * z - 1.0
        elif leaf == "mix.dt_bias":
            z = 0.5 * z - 1.5
        elif leaf == "mix.w0":
            z = 1.2 * z - 1.5
        elif leaf in ("mix.u", "mix.sink"):
            z = 0.8 * z
        elif leaf.startswith("mix.mu"):
            z = 0.5 + 0.4 * z
        elif leaf in ("mix.conv.b", "mlp.router.b"):
            z = 0.02 * z if leaf.endswith("router.b") else 0.3 * z
        elif leaf == "norm1" or name == "final.norm":
            z = 0.3 * z
        elif len(shape) == 1:
            z = 1.0 + 0.3 * z
        else:
            z = z * shape[1] ** -0.5 * (2.0 if leaf in ("mix.uq", "mix.uk", "mix.w1", "mix.w2") else 1.0)
        w[name] = z
    most = max([x["mlp"]["router"]["experts"] for x in cfg["layers"] if x["mlp"] and x["mlp"]["kind"] == "moe"], default=0)
    if most:
        w["embed"][:, :most] = np.stack([r.permutation(np.linspace(-2.0, 2.0, most)) for _ in range(cfg["vocab"])])
    for name, x in w.items():
        leaf = name.split(".", 1)[-1]
        if leaf in ("mix.o", "mlp.down") or leaf.endswith(".down"):
            x[:most] = 0.0
        elif leaf == "norm1":
            x[:most] = 0.0
        elif leaf == "mlp.router":
            x[:] = 0.0
            x[np.arange(len(x)), r.permutation(most)[:len(x)]] = 3.0
    return {name: bf16(x).astype(np.float64) for name, x in w.items()}
