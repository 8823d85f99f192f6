"""A plain float64 forward pass of the Kagalorn design, for tests: one function per mechanism, whole sequences, no cache.

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


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def grouped_rms_norm(x, weight, groups, eps):
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape) * weight


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def causal_conv(x, kernel):
    """Per-channel convolution over time, zeros before the start; kernel [channels, taps], its last column meets the
    current token."""
    taps = kernel.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(padded[j:j + len(x)] * kernel[:, j] for j in range(taps))


def delta_rule(q, k, v, beta, decay, state=None):
    """The gated delta rule of one head: q, k [T, dim], v [T, vdim], beta, decay [T].  Returns (o [T, vdim], state)."""
    s = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    out = np.empty_like(v)
    for t in range(len(q)):
        s *= decay[t]
        u = beta[t] * (v[t] - s.T @ k[t])
        s += np.outer(k[t], u)
        out[t] = s.T @ q[t]
    return out, s


def delta_mixer(h, w, p, m, eps):
    heads, kvh, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    n = len(h)
    q, k, v = (silu(causal_conv(h @ w[p + c].T, w[p + c + ".conv"])) for c in "qkv")
    q = unit(q.reshape(n, kvh, dim)) * dim ** -0.5
    k = unit(k.reshape(n, kvh, dim))
    v = v.reshape(n, heads, vdim)
    beta = sigmoid(h @ w[p + "b"].T)
    decay = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = np.empty_like(v)
    for a in range(heads):
        g = a // (heads // kvh)
        o[:, a] = delta_rule(q[:, g], k[:, g], v[:, a], beta[:, a], decay[:, a])[0]
    gate = silu(h @ w[p + "g"].T).reshape(n, heads, vdim)
    return (rms(o, eps) * w[p + "norm"] * gate).reshape(n, -1) @ w[p + "o"].T


def visible(i, size, pool):
    """What position i attends to: (its window's positions, its pooled blocks)."""
    lo = max(0, i - size + 1)
    blocks = [b for b in range(i // pool + 1) if b * pool + pool - 1 <= i - size]
    return list(range(lo, i + 1)), blocks


def sink_softmax(scores):
    """Softmax with a 1 more in the denominator."""
    top = max(0.0, float(scores.max()))
    e = np.exp(scores - top)
    return e / (np.exp(-top) + e.sum())


def pooled_window_attention(q, k, v, scale, size, pool):
    """One query head: q, k [T, dim], v [T, vdim]."""
    out = np.empty((len(q), v.shape[1]))
    for i in range(len(q)):
        toks, blocks = visible(i, size, pool)
        ks = [k[j] for j in toks] + [k[b * pool:(b + 1) * pool].mean(0) for b in blocks]
        vs = [v[j] for j in toks] + [v[b * pool:(b + 1) * pool].mean(0) for b in blocks]
        out[i] = sink_softmax(np.array(ks) @ q[i] * scale) @ np.array(vs)
    return out


def attention_mixer(h, w, p, m, eps):
    heads, kvh, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    n = len(h)
    q = (rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]).reshape(n, heads, dim)
    k = (rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]).reshape(n, kvh, dim)
    v = (h @ w[p + "v"].T).reshape(n, kvh, vdim)
    o = np.empty((n, heads, vdim))
    for a in range(heads):
        g = a // (heads // kvh)
        o[:, a] = pooled_window_attention(q[:, a], k[:, g], v[:, g], m["scale"], m["mask"]["size"], m["mask"]["pool"])
    return (o.reshape(n, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def clamped_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def hyper_read(streams, weights):
    """The sublayer's input: streams [S, T, width], weights [S]."""
    return np.tensordot(weights, streams, 1)


def hyper_write(streams, mix, out, y):
    """mix [from, to]; every stream from the old ones."""
    return np.stack([np.tensordot(mix[:, t], streams, 1) + out[t] * y for t in range(len(streams))])


MIXERS = {"attention": attention_mixer, "delta": delta_mixer}


def forward(cfg, w, tokens, record=None):
    """Logits [T, vocab]; `record`, if a list, receives the sum of the streams after every layer."""
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = np.stack([w["embed"][np.asarray(tokens)]] * cfg["streams"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."

        def sublayer(x, q, f):
            h = grouped_rms_norm(hyper_read(x, w[f"{p}hc{q}.in"]), w[f"{p}norm{q}"], groups, eps)
            return hyper_write(x, w[f"{p}hc{q}.mix"], w[f"{p}hc{q}.out"], f(h))

        x = sublayer(x, 1, lambda h: MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps))
        if layer.get("mlp"):
            x = sublayer(x, 2, lambda h: clamped_glu(h, w, p + "mlp.", layer["mlp"]["limit"]))
        if record is not None:
            record.append(x.sum(0))
    return grouped_rms_norm(x.sum(0), w["final.norm"], groups, eps) @ w["head"].T
