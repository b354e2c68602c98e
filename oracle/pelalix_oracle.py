"""Plain CPU statement of the Pelalix decoder, one function per mechanism, in NumPy float64 (or float32).

Written from the design's equations and independent of the product: it reads a config dict and a {name: array} table and
recomputes the whole sequence for every call -- no cache, no batch, no fused step.  Tests compare the framework with it.
A test that wants to see a fault plants it here (the keyword arguments `faults`), never on the GPU.
"""
import numpy as np


def dyt(x, alpha, w, b):
    """Dynamic tanh in place of a norm: tanh(alpha x) w + b, no statistics."""
    return np.tanh(x * alpha) * w + b


def rms_rows(x, w, eps):
    """Root-mean-square norm over the last axis, plain weight."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def token_shift(h, mu):
    """h_t + (h_{t-1} - h_t) mu with h_{-1} = 0; the shift reads the unshifted neighbour."""
    prev = np.concatenate([np.zeros_like(h[:1]), h[:-1]], axis=0)
    return h + (prev - h) * mu


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def mix_heads(s, talk):
    """s [H, T, T] -> out[h] = sum_g talk[h, g] s[g]."""
    return np.tensordot(talk, s, axes=(1, 0))


def causal(s):
    T = s.shape[-1]
    return np.where(np.tril(np.ones((T, T), dtype=bool))[None], s, -np.inf)


def softmax_sink(s, sink):
    """softmax over the last axis whose denominator also holds exp(sink_h), once."""
    m = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - m))


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention(h, w, p, m, eps, v_first, no_sink=False, no_talk=False):
    """One attention mixer on h [T, width].  p: tensor prefix ("l0.mix."), m: the mixer's sizes.  Returns (out, own values)."""
    T = h.shape[0]
    H, G, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_rows(h @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(T, H, dim)
    k = rms_rows(h @ w[p + "k"].T, w[p + "k.norm"], eps).reshape(T, G, dim)
    own = h @ w[p + "v"].T
    v = (own if v_first is None else mix_values(own, v_first, w[p + "vmix"])).reshape(T, G, vdim)
    per = H // G
    kk, vv = np.repeat(k, per, axis=1), np.repeat(v, per, axis=1)
    s = np.einsum("ihd,jhd->hij", q, kk, optimize=True) * m["scale"]
    if not no_talk:
        s = mix_heads(s, w[p + "talk"])
    a = softmax_sink(causal(s), np.full(H, -1e30) if no_sink else w[p + "sink"])
    o = np.einsum("hij,jhd->ihd", a, vv, optimize=True)
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * vdim) @ w[p + "o"].T, own


def feed_forward(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def norm(x, w, name):
    return dyt(x, w[name + ".alpha"], w[name], w[name + ".b"])


def forward(cfg, weights, tokens, dtype=np.float64, layers_out=None, no_shift=False, **faults):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer."""
    w = {k: np.asarray(v, dtype=dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)] * dtype(cfg["embedding"]["scale"])
    v_first = None
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = norm(x, w, p + "norm1")
        if not no_shift:
            h = token_shift(h, w[p + "shift"])
        y, own = attention(h, w, p + "mix.", m, eps, v_first if m["v_mix"] else None, **faults)
        if m["v_mix"] and v_first is None:
            v_first = own
        x = x + y * w[p + "ls1"]
        if layer["mlp"] is not None:
            x = x + feed_forward(norm(x, w, p + "norm2"), w, p + "mlp.") * w[p + "ls2"]
        if layers_out is not None:
            layers_out.append(x)
    return norm(x, w, "final.norm") @ w["head"].T
