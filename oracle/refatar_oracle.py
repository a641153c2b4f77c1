"""Plain, slow restatement of the Refatar decoder in numpy, one function per mechanism.

Everything runs token by token or with full score matrices, in the dtype of its inputs (float64 in the tests); nothing
here is shared with the package.  Weights are a flat dict of arrays under the checkpoint's tensor names, the
configuration is the checkpoint's config dict.
"""

import math

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z)))).astype(z.dtype)


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_rms_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def causal_conv(x, w):
    """x [T, C], w [C, taps]: y[t] = sum_j w[:, j] x[t - taps + 1 + j], nothing before the first token."""
    t, c = x.shape
    taps = w.shape[1]
    y = np.zeros_like(x)
    for i in range(t):
        for j in range(taps):
            s = i - taps + 1 + j
            if s >= 0:
                y[i] += w[:, j] * x[s]
    return y


def canon(h, w):
    return h + causal_conv(h, w)


def window_visible(i, j, size, keep_first):
    return j <= i and (i - j < size or j < keep_first)


def window_attention(q, k, v, scale, size, keep_first):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]; softmax over the window and the kept first tokens."""
    t, h, _ = q.shape
    g = k.shape[1]
    out = np.zeros((t, h, v.shape[2]), dtype=q.dtype)
    for i in range(t):
        js = np.array([j for j in range(i + 1) if window_visible(i, j, size, keep_first)])
        for a in range(h):
            kv = a // (h // g)
            s = (k[js, kv] @ q[i, a]) * scale
            p = np.exp(s - s.max())
            out[i, a] = (p / p.sum()) @ v[js, kv]
    return out


def hgrn2_recurrence(q, f, v, state=None):
    """q, f [T, H, D], v [T, H, Dv]: S = diag(f) S + (1 - f) v^T, o = S^T q.  Returns (o [T, H, Dv], S [H, D, Dv])."""
    t, h, d = q.shape
    s = np.zeros((h, d, v.shape[2]), dtype=q.dtype) if state is None else state.copy()
    o = np.zeros((t, h, v.shape[2]), dtype=q.dtype)
    for i in range(t):
        s = f[i][:, :, None] * s + (1.0 - f[i])[:, :, None] * v[i][:, None, :]
        o[i] = np.einsum("hdv,hd->hv", s, q[i])
    return o, s


def delta_recurrence(q, k, v, decay, beta, state=None):
    """Gated delta rule, q, k [T, H, D] (already per value head), v [T, H, Dv], decay, beta [T, H]."""
    t, h, d = q.shape
    s = np.zeros((h, d, v.shape[2]), dtype=q.dtype) if state is None else state.copy()
    o = np.zeros((t, h, v.shape[2]), dtype=q.dtype)
    for i in range(t):
        s = decay[i][:, None, None] * s
        u = beta[i][:, None] * (v[i] - np.einsum("hdv,hd->hv", s, k[i]))
        s = s + k[i][:, :, None] * u[:, None, :]
        o[i] = np.einsum("hdv,hd->hv", s, q[i])
    return o, s


def left_mixer(h, w, p, m):
    t = h.shape[0]
    heads, kvh = m["heads"], m["kv_heads"]
    q = (h @ w[p + ".q"].T + w[p + ".q.b"]).reshape(t, heads, m["dim"])
    k = (h @ w[p + ".k"].T + w[p + ".k.b"]).reshape(t, kvh, m["dim"])
    v = (h @ w[p + ".v"].T + w[p + ".v.b"]).reshape(t, kvh, m["vdim"])
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"], m["mask"]["keep_first"]).reshape(t, -1)
    return (o * sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def right_mixer(h, w, p, m, eps):
    t = h.shape[0]
    heads, d, dv = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + ".q"].T).reshape(t, heads, d)
    low = w[p + ".lower"]
    f = (low + (1.0 - low) * sigmoid(h @ w[p + ".f"].T + w[p + ".f.b"])).reshape(t, heads, d)
    v = (h @ w[p + ".v"].T).reshape(t, heads, dv)
    o, _ = hgrn2_recurrence(q, f, v)
    return (rms(o, eps) * w[p + ".norm"]).reshape(t, -1) @ w[p + ".o"].T


def parallel_mixer(h, w, p, m, eps):
    return m["left_scale"] * left_mixer(h, w, p + ".left", m["left"]) + m["right_scale"] * right_mixer(h, w, p + ".right", m["right"], eps)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_mixer(h, w, p, m, eps):
    t = h.shape[0]
    heads, kvh, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[f"{p}.{n}"].T, w[f"{p}.{n}.conv"])) for n in "qkv")
    q = unit(q.reshape(t, kvh, d)) * d ** -0.5
    k = unit(k.reshape(t, kvh, d))
    of = np.arange(heads) // (heads // kvh)
    beta = sigmoid(h @ w[p + ".b"].T)
    decay = np.exp(-np.exp(w[p + ".A_log"]) * softplus(h @ w[p + ".a"].T + w[p + ".dt_bias"]))
    o, _ = delta_recurrence(q[:, of], k[:, of], v.reshape(t, heads, dv), decay, beta)
    o = rms(o, eps) * w[p + ".norm"]
    return (o.reshape(t, -1) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def dense_mlp(h, w, p):
    return np.square(np.maximum(h @ w[p + ".up"].T, 0)) @ w[p + ".down"].T


def token_side(x, e, w, p, eps):
    y = (gelu_tanh(x @ w[p + ".side.gate"].T) * e) @ w[p + ".side.proj"].T
    return x + rms(y, eps) * w[p + ".side.norm"]


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def forward(config, weights, tokens, dtype=np.float64):
    """tokens [T] -> (logits [T, vocab], residual stream after every layer [layers, T, width])."""
    w = {n: np.asarray(a, dtype=dtype) for n, a in weights.items()}
    eps = config["norm"]["eps"]
    tokens = np.asarray(tokens)
    x = w["embed"][tokens]
    side = w["side.embed"][tokens]
    sd = config["token_side"]["dim"]
    after = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}"
        h = canon(zero_centred_rms_norm(x, w[p + ".norm1"], eps), w[p + ".canon1"])
        mixer = {"parallel": parallel_mixer, "delta": delta_mixer}[layer["type"]]
        x = x + zero_centred_rms_norm(mixer(h, w, p + ".mix", layer["mixer"], eps), w[p + ".norm1b"], eps)
        if layer["mlp"] is not None:
            h = canon(zero_centred_rms_norm(x, w[p + ".norm2"], eps), w[p + ".canon2"])
            x = x + zero_centred_rms_norm(dense_mlp(h, w, p + ".mlp"), w[p + ".norm2b"], eps)
        x = token_side(x, side[:, i * sd:(i + 1) * sd], w, p, eps)
        after.append(x)
    logits = zero_centred_rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return softcap(logits, config["logit_softcap"]), np.stack(after)
