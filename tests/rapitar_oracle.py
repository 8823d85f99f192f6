"""A plain float64 forward pass of the Rapitar design, for tests: one function per mechanism, whole sequences, no cache.

It shares no code with the library.  `w` is a dict name -> float64 array (Linear weights [out, in]), `cfg` the parsed
config.json.  Every function takes and returns arrays with time along the first axis.
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_about_one(x, weight, eps):
    """The model's norm: its weight is stored as the difference from one."""
    return rms(x, eps) * (1.0 + weight)


def grouped_rms(x, groups, eps):
    return rms(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape)


def causal_conv(x, kernel, bias):
    """Per-channel convolution over time, zeros before the start; kernel [channels, taps], its last column meets the
    current token."""
    taps = kernel.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return bias + sum(padded[j:j + len(x)] * kernel[:, j] for j in range(taps))


def ssd(x, b, c, dt, decay, skip, state=None):
    """The state-space recurrence of one head: x [T, vdim], b, c [T, N], dt, decay [T].  Returns (y [T, vdim], state [N, vdim])."""
    s = np.zeros((b.shape[1], x.shape[1])) if state is None else state.copy()
    out = np.empty_like(x)
    for t in range(len(x)):
        s = decay[t] * s + dt[t] * np.outer(b[t], x[t])
        out[t] = s.T @ c[t] + skip * x[t]
    return out, s


def gated_then_normed(y, z, weight, groups, eps):
    return grouped_rms(y * silu(z), groups, eps) * weight


def mamba2_mixer(h, w, p, m, eps):
    heads, vdim, n, g = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, t = heads * vdim, len(h)
    z, xbc, dt = np.split(h @ w[p + "in"].T, [inner, 2 * inner + 2 * g * n], axis=1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, b, c = np.split(xbc, [inner, inner + g * n], axis=1)
    x, b, c = x.reshape(t, heads, vdim), b.reshape(t, g, n), c.reshape(t, g, n)
    dt = softplus(dt + w[p + "dt_bias"])
    decay = np.exp(-np.exp(w[p + "A_log"]) * dt)
    y = np.empty_like(x)
    for a in range(heads):
        q = a // (heads // g)
        y[:, a] = ssd(x[:, a], b[:, q], c[:, q], dt[:, a], decay[:, a], w[p + "D"][a])[0]
    return gated_then_normed(y.reshape(t, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


def shifted_mix(h, mu):
    """Every token's h moved towards the token before it by mu per channel; a zero row stands before the first."""
    before = np.concatenate([np.zeros((1, h.shape[1])), h[:-1]])
    return h + (before - h) * mu


def wkv(r, k, v, decay, bonus, state=None):
    """One head: r, k, decay [T, dim], v [T, vdim], bonus [dim].  Returns (o [T, vdim], state [dim, vdim])."""
    s = np.zeros((k.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.empty_like(v)
    for t in range(len(r)):
        kv = np.outer(k[t], v[t])
        out[t] = (s + bonus[:, None] * kv).T @ r[t]
        s = decay[t][:, None] * s + kv
    return out, s


def wkv_decay(mix, w, p):
    return np.exp(-np.exp(np.tanh(mix @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def wkv_mixer(h, w, p, m, eps):
    heads, dim, t = m["heads"], m["dim"], len(h)
    mix = {c: shifted_mix(h, w[p + "mu." + c]) for c in "rkvgw"}
    r, k, v = (np.reshape(mix[c] @ w[p + c].T, (t, heads, dim)) for c in "rkv")
    gate = silu(mix["g"] @ w[p + "g"].T)
    decay = wkv_decay(mix["w"], w, p).reshape(t, heads, dim)
    o = np.stack([wkv(r[:, a], k[:, a], v[:, a], decay[:, a], w[p + "u"][a])[0] for a in range(heads)], 1)
    return (rms(o, eps).reshape(t, -1) * w[p + "norm"] * gate) @ w[p + "o"].T


def rotate_half(x, positions, dims, base):
    """Rotary positions on the first `dims` of the last axis, dimension i paired with i + dims/2; x [T, ..., d]."""
    half = dims // 2
    a = positions.reshape(-1, *[1] * (x.ndim - 1)) * base ** (-2.0 * np.arange(half) / dims)
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., dims:]], -1)


def sink_attention(q, k, v, scale, sink):
    """One head, causal: q, k [T, d], v [T, vdim]; the denominator has exp(sink) more."""
    out = np.empty((len(q), v.shape[1]))
    for i in range(len(q)):
        s = k[:i + 1] @ q[i] * scale
        top = max(s.max(), sink)
        e = np.exp(s - top)
        out[i] = e @ v[:i + 1] / (e.sum() + np.exp(sink - top))
    return out


def latent_mixer(h, w, p, m, eps):
    heads, dim, rot, vdim, rank, t = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], len(h)
    pos = np.arange(t, dtype=np.float64)
    turn = lambda x: rotate_half(x, pos, m["rot"]["dims"], m["rot"]["base"])
    q = (rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"] @ w[p + "uq"].T).reshape(t, heads, dim + rot)
    q = np.concatenate([q[..., :dim], turn(q[..., dim:])], -1)
    c, shared = np.split(h @ w[p + "dkv"].T, [rank], axis=1)
    c, shared = rms(c, eps) * w[p + "dkv.norm"], turn(shared)
    k = (c @ w[p + "uk"].T).reshape(t, heads, dim)
    v = (c @ w[p + "uv"].T).reshape(t, heads, vdim)
    o = np.stack([sink_attention(q[:, a], np.concatenate([k[:, a], shared], 1), v[:, a], m["scale"], w[p + "sink"][a]) for a in range(heads)], 1)
    return (o.reshape(t, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_ff(h, w, p):
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


def route(logits, top):
    """Chosen experts per token (largest logit first, the lower index of a tie first) and the softmax over their logits."""
    ids = np.argsort(-logits, axis=1, kind="stable")[:, :top]
    z = np.take_along_axis(logits, ids, 1)
    e = np.exp(z - z[:, :1])
    return ids, e / e.sum(1, keepdims=True)


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def moe_ff(h, w, p, m):
    ids, weight = route(h @ w[p + "router"].T + w[p + "router.b"], m["router"]["top"])
    out = np.zeros_like(h)
    for e in range(m["router"]["experts"]):
        tok, slot = np.nonzero(ids == e)
        if len(tok):
            out[tok] += weight[tok, slot][:, None] * expert(h[tok], w, f"{p}e{e}.")
    return out


MIXERS = {"mamba2": mamba2_mixer, "wkv": wkv_mixer, "latent_attention": latent_mixer}


def forward(cfg, w, tokens, record=None):
    """Logits [T, vocab]; `record`, if a list, receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm_about_one(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        mlp = layer.get("mlp")
        if mlp:
            y = y + (dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(h, w, p + "mlp.", mlp))
        x = x + y
        if record is not None:
            record.append(x)
    return norm_about_one(x, w["final.norm"], eps) @ w["head"].T
