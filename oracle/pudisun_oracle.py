"""Plain CPU statement of the Pudisun decoder, one function per mechanism, in NumPy float64 (or float32).

Written from the design's equations and independent of the product: it reads a config dict and a {name: array} table and recomputes the
whole sequence for every call -- no cache, no chunks, no batch, no fused step.  Tests compare the framework with it.  A test that wants
to see a fault plants it here (the keyword arguments `faults`), never on the GPU.
"""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, w, eps):
    """Root-mean-square norm over the last axis, plain weight."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


# ---------------------------------------------------------------- rotary positions
def yarn_bounds(dims, base, s):
    """(lo, hi): the pairs whose rotation over the original length lies between `fast` and `slow` turns."""
    def at(turns):
        return dims * math.log(s["original"] / (turns * 2.0 * math.pi)) / (2.0 * math.log(base))
    return max(math.floor(at(s["fast"])), 0), min(math.ceil(at(s["slow"])), dims - 1)


def frequencies(rot):
    """(angle per position of each pair, factor on cos and sin)."""
    dims, s = rot["dims"], rot.get("scaling")
    f = float(rot["base"]) ** (-2.0 * np.arange(dims // 2) / dims)
    if not s:
        return f, 1.0
    lo, hi = yarn_bounds(dims, rot["base"], s)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, pos, rot, no_mscale=False):
    """x [T, ..., n]: the first rot.dims of the last axis turn with the position, dimension i paired with i + dims / 2."""
    f, mult = frequencies(rot)
    mult = 1.0 if no_mscale else mult
    h = rot["dims"] // 2
    a = np.asarray(pos, dtype=np.float64)[:, None] * f
    a = a.reshape(a.shape[:1] + (1,) * (x.ndim - 2) + a.shape[1:])
    c, s = (np.cos(a) * mult).astype(x.dtype), (np.sin(a) * mult).astype(x.dtype)
    u, v = x[..., :h], x[..., h:2 * h]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * h:]], axis=-1)


# ---------------------------------------------------------------- attention
def softmax_sink(s, sink):
    """softmax over the last axis of s [H, T, T] whose denominator also holds exp(sink_h), once."""
    m = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    e = np.exp(s - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - m))


def latent_qk(h, w, p, m, eps, pos, **faults):
    """Queries [T, H, dim + rot], latents [T, rank], the shared rotated keys [T, rot]."""
    H, dim, rd, R = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    rot = dict(m["rot"], dims=rd)
    q = (h @ w[p + "q"].T).reshape(len(h), H, dim + rd)
    d = h @ w[p + "dkv"].T
    c, kr = rms(d[:, :R], w[p + "dkv.norm"], eps), d[:, R:]
    return np.concatenate([q[..., :dim], rotate(q[..., dim:], pos, rot, **faults)], axis=-1), c, rotate(kr, pos, rot, **faults)


def latent_core(q, c, kr, uk, uv, sink, m, no_sink=False, window=None, hide=None):
    """Attention rows [T, H, vdim] of queries at the last positions over all latents.  uk [H dim, rank], uv [H vdim, rank]."""
    H, dim = m["heads"], m["dim"]
    T, S = len(q), len(c)
    k, v = (c @ uk.T).reshape(S, H, dim), (c @ uv.T).reshape(S, H, m["vdim"])
    s = (np.einsum("ihd,jhd->hij", q[..., :dim], k, optimize=True) + np.einsum("ihd,jd->hij", q[..., dim:], kr, optimize=True)) * m["scale"]
    see = np.arange(S)[None, :] <= np.arange(S - T, S)[:, None]
    if hide is not None:
        see = see & (np.arange(S) != hide)[None, :]
    a = softmax_sink(np.where(see[None], s, -np.inf), np.full(H, -1e30) if no_sink else sink)
    return np.einsum("hij,jhd->ihd", a, v, optimize=True)


def latent_attention(h, w, p, m, eps, no_sink=False, no_mscale=False, no_gate=False, pos0=0, **_):
    q, c, kr = latent_qk(h, w, p, m, eps, pos0 + np.arange(len(h)), no_mscale=no_mscale)
    o = latent_core(q, c, kr, w[p + "uk"], w[p + "uv"], w[p + "sink"], m, no_sink=no_sink).reshape(len(h), -1)
    if not no_gate:
        o = o * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ---------------------------------------------------------------- gated linear attention
def gla_decay(a1, w_a2, b, tau):
    """log of the decay of every key channel: log(sigmoid(W_a2 a1 + b)) / tau."""
    return log_sigmoid(a1 @ w_a2.T + b) / tau


def gla_scan(q, k, v, loga, s0=None):
    """S_t = diag(exp(loga_t)) S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t per head; [T, H, dim | vdim].  Returns (o, S)."""
    T, H, dim = q.shape
    s = np.zeros((H, dim, v.shape[2]), dtype=q.dtype) if s0 is None else s0.copy()
    o = np.empty((T, H, v.shape[2]), dtype=q.dtype)
    for t in range(T):
        s = np.exp(loga[t])[:, :, None] * s + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", s, q[t])
    return o, s


def gla(h, w, p, m, eps, forget_state=False, no_decay=False, **_):
    T, H, dim, vdim = len(h), m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dim) * h.dtype.type(dim ** -0.5)
    k, v = (h @ w[p + "k"].T).reshape(T, H, dim), (h @ w[p + "v"].T).reshape(T, H, vdim)
    loga = gla_decay(h @ w[p + "a1"].T, w[p + "a2"], w[p + "a2.b"], m["tau"]).reshape(T, H, dim)
    if no_decay:
        loga = loga * 0
    if forget_state:
        loga = loga - 1e3
    o = rms(gla_scan(q, k, v, loga)[0], w[p + "norm"], eps).reshape(T, H * vdim)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------------- the model
def feed_forward(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"latent_attention": latent_attention, "gla": gla}


def forward(cfg, weights, tokens, dtype=np.float64, layers_out=None, **faults):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer."""
    w = {k: np.asarray(v, dtype=dtype) for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], dtype(cfg["residual_mult"])
    x = w["embed"][np.asarray(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        j = i
        while cfg["layers"][j].get("weights_of") is not None:
            j = cfg["layers"][j]["weights_of"]
        p = f"l{j}."
        x = x + m * MIXERS[layer["type"]](rms(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps, **faults)
        if layer["mlp"] is not None:
            x = x + m * feed_forward(rms(x, w[p + "norm2"], eps), w, p + "mlp.")
        if layers_out is not None:
            layers_out.append(x)
    return (rms(x, w["final.norm"], eps) @ w["embed"].T) * dtype(cfg["logit_scale"])
