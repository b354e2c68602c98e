"""Layered text decoders on the GPU against the plain float64 statement (oracle/pelalix_oracle.py): each mechanism alone, then the model
through the framework's own entry points.  Configurations and weights are made here; sizes vary per layer where that can hide a fault."""
import numpy as np
import pytest
import torch

import pelalix_oracle as orc

pytestmark = pytest.mark.gpu

BF16, F32, I32 = torch.bfloat16, torch.float32, torch.int32
DEV = "cuda:0"


def bf(a):
    """numpy -> the values a bf16 tensor holds, as float64."""
    return torch.as_tensor(np.asarray(a, dtype=np.float32)).to(BF16).double().numpy()


def dev(a, dt=BF16):
    return torch.as_tensor(np.asarray(a, dtype=np.float32)).to(DEV, dt).contiguous()


def host(t):
    return t.detach().double().cpu().numpy()


# ---------------------------------------------------------------- configurations and weights
def attn(H, G, dim, vdim, scale=None, v_mix=True, ff=None):
    return {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "v_mix": v_mix,
                                           "scale": dim ** -0.5 if scale is None else scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


CONFIGS = {
    # one layer kind after another: own sizes per layer, a layer without feed-forward, value mixing that starts late, uneven sizes
    "uneven": dict(width=136, vocab=301, eps=3e-4, escale=5.0, layers=[
        attn(6, 3, 40, 24, v_mix=False, ff=200), attn(5, 1, 24, 36, scale=0.11, ff=None), attn(2, 2, 96, 18, ff=72), attn(4, 4, 32, 9, v_mix=False, ff=136)]),
    "grouped": dict(width=192, vocab=512, eps=1e-5, escale=9.0, layers=[attn(8, 2, 64, 32, ff=320), attn(8, 2, 64, 32, scale=0.2, ff=320), attn(8, 2, 64, 32, ff=320)]),
    "wide": dict(width=128, vocab=320, eps=1e-6, escale=1.0, layers=[attn(16, 4, 96, 64, ff=192), attn(12, 4, 128, 64, ff=128)]),
    "streamed": dict(width=1024, vocab=330, eps=1e-5, escale=8.0, layers=[attn(4, 2, 64, 64, ff=1024), attn(8, 4, 32, 256 // 8, ff=2048)]),
    "many": dict(width=256, vocab=384, eps=1e-5, escale=12.0, layers=[attn(32, 8, 96, 96, ff=256), attn(20, 4, 64, 128, v_mix=False, ff=256), attn(32, 32, 32, 24, ff=64)]),
}


def config_dict(c):
    return {"architecture": "Pelalix", "width": c["width"], "vocab": c["vocab"], "norm": {"eps": c["eps"]}, "embedding": {"scale": c["escale"]},
            "layers": c["layers"]}


def make_weights(cfg, seed=0):
    """Weights under which every mechanism shows in the logits: sharp attention, unlike heads, a talk matrix far from the identity."""
    r = np.random.default_rng(seed)
    D, w = cfg["width"], {}

    def nrm(name):
        w[name], w[name + ".b"], w[name + ".alpha"] = r.normal(1, 0.3, D), r.normal(0, 0.2, D), np.asarray(r.uniform(0.4, 0.9))
    w["embed"] = r.normal(0, 1 / cfg["embedding"]["scale"], (cfg["vocab"], D))
    for i, ly in enumerate(cfg["layers"]):
        p, m = f"l{i}.", ly["mixer"]
        H, G = m["heads"], m["kv_heads"]
        nrm(p + "norm1")
        for n, rows in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"]), ("g", H)):
            w[p + "mix." + n] = r.normal(0, 1.2 * D ** -0.5, (rows, D))
        w[p + "mix.q.norm"], w[p + "mix.k.norm"] = r.normal(1.6, 0.4, H * m["dim"]), r.normal(1.6, 0.4, G * m["dim"])
        w[p + "mix.talk"] = np.eye(H) + r.normal(0, 0.5 * H ** -0.5, (H, H))
        w[p + "mix.sink"], w[p + "mix.vmix"] = r.normal(2, 1, H), np.asarray(r.uniform(0.2, 0.7))
        w[p + "mix.o"] = r.normal(0, 1.5 * (H * m["vdim"]) ** -0.5, (D, H * m["vdim"]))
        w[p + "ls1"], w[p + "ls2"], w[p + "shift"] = r.normal(0.7, 0.3, D), r.normal(0.7, 0.3, D), r.uniform(0, 0.9, D)
        if ly["mlp"]:
            ff = ly["mlp"]["ff"]
            nrm(p + "norm2")
            w[p + "mlp.gate"], w[p + "mlp.up"] = r.normal(0, 1.5 * D ** -0.5, (ff, D)), r.normal(0, 1.5 * D ** -0.5, (ff, D))
            w[p + "mlp.down"] = r.normal(0, 1.5 * ff ** -0.5, (D, ff))
    nrm("final.norm")
    w["head"] = r.normal(0, D ** -0.5, (cfg["vocab"], D))
    return {k: bf(v) for k, v in w.items()}


_built = {}


def build(name, dtype):
    """(model, oracle weights, config dict) of a named configuration; kept for the session."""
    if (name, dtype) not in _built:
        from phi_3_vision_mlx_amd.config import make_config
        from phi_3_vision_mlx_amd.registry import family
        d = config_dict(CONFIGS[name])
        w = make_weights(d, seed=len(name))
        cfg = make_config(d, dtype=dtype)
        _built[name, dtype] = family(cfg).model_cls(cfg, {k: torch.as_tensor(v).float() for k, v in w.items()}, device=DEV), w, d
    return _built[name, dtype]


def tokens(d, n, seed):
    return np.random.default_rng(seed).integers(0, d["vocab"], n)


def rel(got, want):
    """Worst row error: rms over the vocabulary of the difference / rms of the logits."""
    d = np.asarray(got, dtype=np.float64) - want
    return float(np.sqrt((d ** 2).mean(-1)).max() / np.sqrt((want ** 2).mean()))


def close(got, want, dt, what=""):
    """Worst row and worst element of got - want, both against the rms of want: rounding of a bf16 (or fp32) result and its inputs."""
    d, s = np.asarray(got, dtype=np.float64) - want, np.sqrt((want ** 2).mean())
    row, worst = float(np.sqrt((d ** 2).mean(-1)).max() / s), float(np.abs(d).max() / s)
    assert row < (1e-5 if dt == F32 else 0.04) and worst < (1e-4 if dt == F32 else 0.15), (what, row, worst)


TOL = {"float32": 2e-5, "bfloat16": 0.035}
DTYPES = ["float32", "bfloat16"]


# ---------------------------------------------------------------- mechanisms
def test_embedding_scale():
    from phi_3_vision_mlx_amd import ops
    t = bf(np.random.default_rng(0).normal(0, 1, (50, 72)))
    ids = np.array([0, 49, 7, -3, 60])
    x = ops.embed_scale(torch.as_tensor(ids, dtype=I32, device=DEV), dev(t), 3.7)
    assert np.abs(host(x) - t[np.clip(ids, 0, 49)] * np.float32(3.7)).max() < 1e-6


@pytest.mark.parametrize("R", [2, 5, 64])
@pytest.mark.parametrize("parts", [[37], [1] * 9, [2, 3, 2, 17, 1, 8], [8, 16, 7], [20, 5, 20]])
def test_dynamic_tanh_and_token_shift(R, parts):
    """Any cut of a sequence gives what the whole gives, also where a portion is longer than the history (it wraps onto its own
    first token's predecessor) and for rows whose sequence starts inside the batch."""
    from phi_3_vision_mlx_amd import ops
    B, H, T = 2, 300, sum(parts)
    r = np.random.default_rng(R)
    x, w, b, mu = r.normal(0, 2, (B, T, H)), bf(r.normal(1, 0.3, H)), bf(r.normal(0, 0.3, H)), bf(r.uniform(0, 1, H))
    pads = [0, min(4, T - 1)]
    xd = dev(x, F32)
    want = np.stack([np.concatenate([np.zeros((p, H)), orc.token_shift(orc.dyt(host(xd)[i, p:], 0.75, w, b), mu)]) for i, p in enumerate(pads)])
    hist = torch.full((B, R, H), float("nan"), dtype=F32, device=DEV)
    pad = torch.tensor(pads, dtype=I32, device=DEV)
    past = 0
    for k, n in enumerate(parts):
        out = torch.empty((B * n, H), dtype=F32, device=DEV)
        kw = dict(d_past=torch.tensor([past], dtype=I32, device=DEV), past=0) if k % 2 else dict(past=past)   # both ways to pass the position
        ops.dyt(xd[:, past:past + n].contiguous().view(-1, H), (0.75, dev(w), dev(b)), out, B, n, shift=dev(mu), hist=hist, pad_len=pad, **kw)
        got = host(out).reshape(B, n, H)
        for i, p in enumerate(pads):
            lo = max(p - past, 0)
            assert not n > lo or np.abs(got[i, lo:] - want[i, past + lo:past + n]).max() < 3e-6, (i, past, n)
        past += n
    plain = torch.empty((B * T, H), dtype=BF16, device=DEV)
    ops.dyt(xd.view(-1, H), (0.75, dev(w), dev(b)), plain, B * T, 1)
    assert np.abs(host(plain).reshape(B, T, H) - orc.dyt(host(xd), 0.75, w, b)).max() < 0.02


@pytest.mark.parametrize("M,N,K", [(1, 64, 128), (1, 320, 1024), (1, 128, 3072), (1, 64, 8192), (2, 50, 136), (5, 96, 2048), (8, 64, 3072), (8, 40, 12288), (12, 128, 3072), (16, 192, 512),
                                   (16, 64, 8192), (60, 128, 1024), (300, 3072, 512), (1100, 512, 256), (1100, 256, 192)])
def test_scaled_residual_epilogue(M, N, K):
    """x + col_scale * (W a) in fp32 from every projection kernel that serves bf16 rows."""
    from phi_3_vision_mlx_amd import ops
    r = np.random.default_rng(M + N)
    a, w, res, ls = dev(r.normal(0, 1, (M, K))), bf(r.normal(0, K ** -0.5, (N, K))), r.normal(0, 1, (M, N)), bf(r.normal(1, 0.5, N))
    x = dev(res, F32)
    want = host(x) + (host(a) @ w.T) * ls
    ops.project(a, dev(w), ops.EPI_SCALE_RESID_F32, resid=x, col_scale=dev(ls), out=x)
    close(host(x), want, F32)


@pytest.mark.parametrize("K", [1024, 2048, 3072, 4096, 8192, 640])
@pytest.mark.parametrize("silu", [False, True])
def test_dynamic_tanh_in_the_projection_prologue(K, silu):
    """One row: the fused launch (the last width: the two launches) = dyt with token shift, then the projection; the history as well."""
    from phi_3_vision_mlx_amd import ops
    r, N, R = np.random.default_rng(K), 96, 4
    x, w = r.normal(0, 2, (6, K)), bf(r.normal(0, K ** -0.5, (2 * N if silu else N, K)))
    nw, nb, mu = bf(r.normal(1, 0.3, K)), bf(r.normal(0, 0.3, K)), bf(r.uniform(0, 1, K))
    xd, hist = dev(x, F32), torch.full((1, R, K), float("nan"), dtype=F32, device=DEV)
    h = orc.dyt(host(xd), 0.7, nw, nb)
    y = orc.token_shift(h, mu) @ w.T
    want = orc.silu(y[:, :N]) * y[:, N:] if silu else y
    scratch = torch.empty((1, K), dtype=BF16, device=DEV)
    for t in range(6):
        out = torch.full((1, N), float("nan"), dtype=BF16, device=DEV)
        kw = dict(d_past=torch.tensor([t], dtype=I32, device=DEV)) if t % 2 else dict(past=t)
        ops.project_dyt(xd[t:t + 1].contiguous(), (0.7, dev(nw), dev(nb)), dev(w), scratch, ops.EPI_SILU_MUL if silu else ops.EPI_NONE, out=out,
                        shift=dev(mu), hist=hist, **kw)
        close(host(out), want[t:t + 1], BF16, t)
        assert np.abs(host(hist)[0, t % R] - h[t]).max() < 3e-6
    out = torch.empty((1, N), dtype=BF16, device=DEV)
    ops.project_dyt(xd[:1].contiguous(), (0.7, dev(nw), dev(nb)), dev(w), scratch, ops.EPI_SILU_MUL if silu else ops.EPI_NONE, out=out)
    y = h[:1] @ w.T
    close(host(out), orc.silu(y[:, :N]) * y[:, N:] if silu else y, BF16)


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("M,N,K", [(1, 64, 128), (3, 50, 136), (7, 301, 72), (16, 192, 512), (40, 128, 192), (130, 100, 100), (300, 320, 256)])
def test_projection_of_any_size(M, N, K, dt):
    from phi_3_vision_mlx_amd import ops
    r = np.random.default_rng(M)
    a, w, res, ls = r.normal(0, 1, (M, K)), bf(r.normal(0, K ** -0.5, (N, K))), r.normal(0, 1, (M, N)), bf(r.normal(1, 0.5, N))
    ad = dev(a, dt)
    y = host(ad) @ w.T
    close(host(ops.project(ad, dev(w))), y, dt)
    x = dev(res, F32)
    ops.project(ad, dev(w), ops.EPI_SCALE_RESID_F32, resid=x, col_scale=dev(ls), out=x)
    assert np.abs(host(x) - (host(dev(res, F32)) + y * ls)).max() < 2e-5        # (fp32 sums whatever the activations' type)
    if N % 2 == 0:
        n = N // 2
        got = host(ops.project(ad, dev(w), ops.EPI_SILU_MUL))
        close(got, orc.silu(y[:, :n]) * y[:, n:], dt)


class Mix:
    """One attention mixer on the device and in the plain statement, from the packed projection's outputs on."""

    def __init__(self, H, G, dim, vdim, B, Tp, dt, seed=0, scale=None):
        from phi_3_vision_mlx_amd.cache import round_up
        self.H, self.G, self.dim, self.vdim, self.B, self.Tp, self.dt = H, G, dim, vdim, B, Tp, dt
        self.r = np.random.default_rng(seed)
        self.scale = dim ** -0.5 if scale is None else scale
        self.ld = round_up(H * dim + G * (dim + vdim) + H, 64)
        self.qn, self.kn = bf(self.r.normal(1.0, 0.3, H * dim)), bf(self.r.normal(1.0, 0.3, G * dim))
        self.talk, self.sink = bf(np.eye(H) + self.r.normal(0, 0.8 * H ** -0.5, (H, H))), bf(self.r.normal(1, 1, H))
        self.k = torch.zeros((B, G, Tp, round_up(dim, 32)), dtype=dt, device=DEV)
        self.v = torch.zeros((B, G, Tp // 16, round_up(vdim, 32), 16), dtype=dt, device=DEV)
        self.vmix, self.eps = 0.0, 1e-5

    def run(self, qkv, L, past, pads=None, first=None, plan=None, d_past=False):
        from phi_3_vision_mlx_amd import ops
        B, H, G = self.B, self.H, self.G
        n = ops.mix_plan(B, L, H, G, self.dim, self.vdim, self.Tp if L == 1 else past + L, self.dt) if plan is None else plan
        ws = torch.full((max(1, ops.mix_ws_bytes(B, L, H, self.vdim, max(n, 1)) // 4),), float("nan"), dtype=F32, device=DEV)
        q = torch.zeros(B * H * L * self.k.shape[3], dtype=self.dt, device=DEV)
        out = torch.full((B * L, H * self.vdim), float("nan"), dtype=self.dt, device=DEV)
        ops.attention_mixed(qkv, q, self.k, self.v, out, (dev(self.qn), dev(self.kn)), dev(self.talk), dev(self.sink), B, L, H, G, self.dim, self.vdim,
                            self.eps, self.scale, 0 if d_past else past, v_first=first, vmix=self.vmix,
                            pad_len=None if pads is None else torch.tensor(pads, dtype=I32, device=DEV),
                            d_past=torch.tensor([past], dtype=I32, device=DEV) if d_past else None, ws=ws, n_split=n)
        return host(out).reshape(B, L, H, self.vdim)

    def oracle(self, qkv, pad=0, first=None, no_sink=False, far_off=None, scores=False):
        """Output rows of one sequence [T, H, vdim] from its packed rows [T, ld]."""
        H, G, dim, vdim = self.H, self.G, self.dim, self.vdim
        x = qkv[pad:]
        T = x.shape[0]
        q = orc.rms_rows(x[:, :H * dim], self.qn, self.eps).reshape(T, H, dim)
        k = orc.rms_rows(x[:, H * dim:(H + G) * dim], self.kn, self.eps).reshape(T, G, dim)
        v = x[:, (H + G) * dim:(H + G) * dim + G * vdim]
        if first is not None:
            v = orc.mix_values(v, first[pad:], self.vmix)
        v = v.reshape(T, G, vdim)
        kk, vv = np.repeat(k, H // G, axis=1), np.repeat(v, H // G, axis=1)
        s = orc.causal(orc.mix_heads(np.einsum("ihd,jhd->hij", q, kk) * self.scale, self.talk))
        if scores:
            return s
        if far_off is not None:
            s[:, :, far_off] = -np.inf
        a = orc.softmax_sink(s, np.full(H, -1e30) if no_sink else self.sink)
        n = H * dim + G * (dim + vdim)
        return np.concatenate([np.zeros((pad, H, vdim)), np.einsum("hij,jhd->ihd", a, vv) * orc.sigmoid(x[:, n:n + H])[:, :, None]])


SIZES = [(4, 2, 96, 48), (6, 3, 40, 24), (8, 8, 64, 128), (5, 1, 24, 36), (16, 4, 96, 64), (12, 4, 128, 96), (32, 8, 96, 96), (32, 32, 32, 16), (20, 5, 64, 128), (3, 3, 128, 7)]


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("H,G,dim,vdim", SIZES)
def test_mixed_attention_prompt_portions_and_decode(H, G, dim, vdim, dt):
    """A prompt, a portion behind it, then single tokens (positions as host value and from the device), rows of unequal padding."""
    B, parts, pads = 3, [45, 2, 17] + [1] * 5, [0, 7, 40]
    T = sum(parts)
    m = Mix(H, G, dim, vdim, B, 96, dt, seed=H)
    m.vmix = 0.4
    raw = dev(m.r.normal(0, 1, (B, T, m.ld)), dt)
    first = dev(m.r.normal(0, 1, (B, T, G * vdim)), dt)
    want = np.stack([m.oracle(host(raw)[b], pads[b], host(first)[b]) for b in range(B)])
    past = 0
    for k, L in enumerate(parts):
        got = m.run(raw[:, past:past + L].contiguous().view(B * L, -1), L, past, pads, first[:, past:past + L].contiguous().view(B * L, -1),
                    d_past=k % 2 == 1)
        assert np.isfinite(got).all()
        for b in range(B):
            lo = max(0, pads[b] - past)
            if lo < L:
                close(got[b, lo:], want[b, past + lo:past + L], dt, (b, past, L))
        past += L


@pytest.mark.parametrize("n_split", [0, 1, 2, 3, 5, 16])
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 96, 48), (16, 4, 96, 64), (32, 8, 96, 96)])
def test_mixed_attention_key_splits(H, G, dim, vdim, n_split):
    """Every number of key splits (more than there are key tiles included) and the any-size kernel give the same rows."""
    B, L, past = 2, 33, 64
    m = Mix(H, G, dim, vdim, B, 128, BF16, seed=n_split)
    raw = dev(m.r.normal(0, 1, (B, past + L, m.ld)), BF16)
    pads = [0, 70]
    want = np.stack([m.oracle(host(raw)[b], pads[b]) for b in range(B)])
    m.run(raw[:, :past].contiguous().view(B * past, -1), past, 0, pads)
    got = m.run(raw[:, past:].contiguous().view(B * L, -1), L, past, pads, plan=n_split)
    close(got[0], want[0, past:], BF16)
    close(got[1, 6:], want[1, 70:], BF16)
    if n_split:
        one = dev(m.r.normal(0, 1, (B, 1, m.ld)), BF16)
        full = torch.cat([raw, one], dim=1)
        got = m.run(one.view(B, -1), 1, past + L, pads, plan=n_split)
        want = [m.oracle(host(full)[b], pads[b])[-1] for b in range(B)]
        close(got[:, 0], np.stack(want), BF16)


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("far", [0, 1, 15, 16, 31, 32, 255, 256, 399])
def test_one_far_key_decides(far, dt):
    """One key among hundreds carries almost all of the weight; the key's place is at tile and block borders, in prompts and in decode.
    The same comparison without that key, or without the sink, is far off: the test can see both."""
    H, G, dim, vdim, T = 8, 4, 64, 32, 401
    m = Mix(H, G, dim, vdim, 1, 512, dt, seed=far)
    x = m.r.normal(0, 1, (1, T, m.ld)) * 0.3
    m.talk, m.scale = bf(np.eye(H) + m.r.normal(0, 0.05, (H, H))), 0.25
    x[0, -1, :H * dim] = 4.0 * np.tile(x[0, far, H * dim:(H + G) * dim].reshape(G, 1, dim), (1, H // G, 1)).reshape(-1)
    raw = dev(x, dt)
    m.sink = bf(m.oracle(host(raw)[0], scores=True)[:, -1, far])           # the sink takes half of the weight
    want = m.oracle(host(raw)[0])
    got = m.run(raw.view(T, -1), T, 0)
    tol = 3e-5 if dt == F32 else 0.03
    assert np.abs(got[0, -1] - want[-1]).max() < tol
    m.run(raw[:, :-1].contiguous().view(T - 1, -1), T - 1, 0)
    assert np.abs(m.run(raw[:, -1].contiguous(), 1, T - 1)[0, 0] - want[-1]).max() < tol
    assert np.abs(m.oracle(host(raw)[0], far_off=far)[-1] - want[-1]).max() > 3 * tol
    assert np.abs(m.oracle(host(raw)[0], no_sink=True)[-1] - want[-1]).max() > 3 * tol


# ---------------------------------------------------------------- the model
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_prompt_logits(name, dtype):
    m, w, d = build(name, dtype)
    for n in (1, 2, 16, 17, 90):
        t = tokens(d, n, n)
        want = orc.forward(d, w, t)
        got, _ = m(input_ids=t[None], max_tokens=1, full_logits=True)
        assert got.dtype == (F32 if dtype == "float32" else BF16)
        assert rel(host(got)[0], want) < TOL[dtype], n
        last, _ = m(input_ids=t[None], max_tokens=1)
        assert last.shape[1] == 1 and rel(host(last)[0], want[-1:]) < TOL[dtype]


@pytest.mark.parametrize("fault", ["no_shift", "no_sink", "no_talk", "vmix", "eps", "scale"])
def test_the_comparison_sees_each_mechanism(fault):
    """The same comparison against an oracle with one mistake in it: out of tolerance by a wide margin (bf16 tolerance)."""
    m, w, d = build("grouped", "bfloat16")
    t = tokens(d, 60, 3)
    got = host(m(input_ids=t[None], max_tokens=1, full_logits=True)[0])[0]
    kw = {fault: True} if fault.startswith("no_") else {}
    w2, d2 = dict(w), {**d, "layers": [dict(x, mixer=dict(x["mixer"])) for x in d["layers"]], "norm": dict(d["norm"])}
    if fault == "vmix":
        w2["l1.mix.vmix"] = w["l1.mix.vmix"] * 0
    if fault == "eps":
        d2["norm"]["eps"] = 0.3
    if fault == "scale":
        d2["layers"][1]["mixer"]["scale"] = 0.125
    assert rel(got, orc.forward(d, w, t)) < TOL["bfloat16"] < 2 * TOL["bfloat16"] < rel(got, orc.forward(d2, w2, t, **kw))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cut", [2, 3, 16, 31])
def test_portions_of_a_prompt(cut, dtype):
    """A prompt fed in portions through the cache gives the whole prompt's logits."""
    m, w, d = build("uneven", dtype)
    t = tokens(d, 75, cut)
    want = orc.forward(d, w, t)
    got, cache = m(input_ids=t[None, :cut], max_tokens=80, full_logits=True)
    rows = [host(got)[0]]
    while cache[0].offset < len(t):
        o = cache[0].offset
        got, cache = m(input_ids=t[None, o:o + cut], cache=cache)
        rows.append(host(got)[0])
    assert rel(np.concatenate(rows), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_decode_token_by_token(name, dtype):
    """Eager one-token calls and the captured greedy step (teacher-forced), over tile and block borders; eager work between replays."""
    m, w, d = build(name, dtype)
    t = tokens(d, 70, 1)
    want = orc.forward(d, w, t)
    for start in (1, 13):
        got, cache = m(input_ids=t[None, :start], max_tokens=70, full_logits=True)
        rows = [host(got)[0]]
        for i in range(start, len(t)):
            if i % 3 == 0:
                lg, cache = m(input_ids=t[None, i:i + 1], cache=cache)
            else:
                lg, _ = m.greedy_step(torch.tensor([[int(t[i])]], dtype=I32, device=DEV), cache)
            rows.append(host(lg)[0])
        assert rel(np.concatenate(rows), want) < TOL[dtype], start


def test_long_decode_wraps_the_shift_history():
    m, w, d = build("grouped", "float32")
    t = tokens(d, 420, 9)
    want = orc.forward(d, w, t)
    _, cache = m(input_ids=t[None, :3], max_tokens=430, full_logits=True)
    for i in range(3, len(t)):
        lg, _ = m.greedy_step(torch.tensor([[int(t[i])]], dtype=I32, device=DEV), cache)
        if i % 40 == 0 or i > 410:
            assert rel(host(lg)[0], want[i:i + 1]) < TOL["float32"], i


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["uneven", "many"])
def test_batches_of_unequal_requests(name, dtype):
    """Left-padded batches, prompt and decode, against each request alone in the oracle."""
    from phi_3_vision_mlx_amd.processor import collate_requests
    m, w, d = build(name, dtype)
    full = [tokens(d, n + 20, n) for n in (1, 2, 33, 64, 5)]
    want = [orc.forward(d, w, t) for t in full]
    cut = [len(t) - 20 for t in full]
    inputs = collate_requests([{"input_ids": t[None, :c]} for t, c in zip(full, cut)])
    got, cache = m(**inputs, max_tokens=24, full_logits=True)
    W = max(cut)
    for b, c in enumerate(cut):
        assert rel(host(got)[b, W - c:], want[b][:c]) < TOL[dtype], b
    for s in range(20):
        tok = torch.tensor([[int(t[c + s])] for t, c in zip(full, cut)], dtype=I32, device=DEV)
        lg, _ = m.greedy_step(tok, cache)
        for b, c in enumerate(cut):
            assert rel(host(lg)[b], want[b][c + s:c + s + 1]) < TOL[dtype], (b, s)


def test_rewind_and_read_only_beams():
    """advance_offset rewinds keys AND the token shift's input; a beam call leaves the cache as it was; too long a rewind is an error."""
    m, w, d = build("grouped", "float32")
    t = tokens(d, 40, 2)
    _, cache = m(input_ids=t[None, :20], max_tokens=200, full_logits=True)
    side = tokens(d, 7, 5)
    want_side = orc.forward(d, w, np.concatenate([t[:20], side]))[20:]
    for adv in (0, 0):
        got, _ = m(input_ids=side[None], cache=cache, advance_offset=adv)
        assert rel(host(got)[0], want_side) < TOL["float32"] and cache[0].offset == 20
    beams = np.stack([tokens(d, 4, s) for s in range(3)])
    got, _ = m(input_ids=beams, cache=cache, n_beam=3, advance_offset=0)
    for b in range(3):
        assert rel(host(got)[b], orc.forward(d, w, np.concatenate([t[:20], beams[b]]))[20:]) < TOL["float32"]
    got, _ = m(input_ids=side[None, :3], cache=cache, advance_offset=1)          # keeps one of the three
    t2 = np.concatenate([t[:20], side[:1], t[20:]])
    want = orc.forward(d, w, t2)
    got, _ = m(input_ids=t[None, 20:], cache=cache)
    assert rel(host(got)[0], want[21:]) < TOL["float32"]
    more = tokens(d, 150, 8)
    m(input_ids=more[None], cache=cache)
    cache[0].offset = 30
    with pytest.raises(ValueError, match="history"):
        m(input_ids=t[None, :2], cache=cache)


def test_captured_prefill_is_the_eager_one():
    """A prompt length seen twice is captured; later prompts of that length replay, with eager work in between, and each keeps its own
    cache while it is alive."""
    m, w, d = build("grouped", "bfloat16")
    L, keep = 40, []
    for s in range(5):
        t = tokens(d, L + 6, 100 + s)
        lg, cache = m(input_ids=t[None, :L], max_tokens=9)
        want = orc.forward(d, w, t)
        assert rel(host(lg)[0], want[L - 1:L]) < TOL["bfloat16"], s
        for i in range(L, L + 6):
            lg, _ = m.greedy_step(torch.tensor([[int(t[i])]], dtype=I32, device=DEV), cache)
            assert rel(host(lg)[0], want[i:i + 1]) < TOL["bfloat16"], (s, i)
        m(input_ids=tokens(d, 11, s)[None], max_tokens=2)
        if s % 2:
            keep.append(cache)
        else:
            del cache
    assert any(k[0] == L for k in m._prefill_graphs)


def greedy(d, w, prompt, n):
    t, margins = list(prompt), []
    for _ in range(n):
        z = orc.forward(d, w, t)[-1]
        o = np.sort(z)
        margins.append(o[-1] - o[-2])
        t.append(int(z.argmax()))
    return t[len(prompt):], min(margins)


def text_processor(d):
    from phi_3_vision_mlx_amd.processor import TextProcessor
    return TextProcessor(None, vocab_size=d["vocab"])


def test_greedy_generation_through_the_api():
    """api._generate on text: the tokens are the oracle's greedy tokens (fp32 model), one prompt and a padded batch."""
    from phi_3_vision_mlx_amd import api
    m, w, d = build("grouped", "float32")
    proc = text_processor(d)
    n = 12
    prompts, want = [], []
    for k in range(40):                                         # one short and one long prompt whose greedy choices are clear
        p = f"prompt {k}" if not prompts else f"a much longer prompt of a few dozen characters, number {k}"
        toks, margin = greedy(d, w, proc(p)["input_ids"][0], n)
        if margin > 1e-3:
            prompts.append(p), want.append(toks)
        if len(prompts) == 2:
            break
    assert len(prompts) == 2
    out = api._generate(m, proc, prompts[0], max_tokens=n, verbose=False, mute=True)
    assert out[0] == proc.tokenizer.decode(want[0]) if isinstance(out, list) else out == proc.tokenizer.decode(want[0])
    out = api._generate(m, proc, prompts, max_tokens=n, verbose=False, mute=True)
    assert out == [proc.tokenizer.decode(t) for t in want]
    picked = api._choose_from(m, proc, prompts[0], choices="ABC", mute=True)
    opts = [proc([f" {c}"])["input_ids"][0, -1] for c in "ABC"]
    z = orc.forward(d, w, proc(prompts[0])["input_ids"][0])[-1]
    assert picked == "ABC"[int(np.argmax(z[opts]))]


@pytest.mark.parametrize("use_beam", [False, True])
def test_constrain_runs_on_the_rewound_cache(use_beam):
    """The constrained decoder's calls (rewinds, beams) on a bf16 and an fp32 model agree on the text."""
    from phi_3_vision_mlx_amd import api
    m, w, d = build("grouped", "float32")
    proc = text_processor(d)
    a = api._constrain(m, proc, ["hello"], [(3, " so")], mute=True, use_beam=use_beam, verbose=False)
    assert len(a) == 1 and a[0]
    t = np.asarray(proc("hello")["input_ids"][0])
    lg, _ = m(input_ids=t[None], max_tokens=1)
    assert rel(host(lg)[0], orc.forward(d, w, t)[-1:]) < TOL["float32"]


@pytest.mark.parametrize("slots", [2, 3])
def test_engine_reuses_slots(slots):
    """Continuous batching: more requests than slots, unequal prompts and budgets, rows freed and taken again mid-flight; every request's
    tokens are what the oracle alone generates."""
    from phi_3_vision_mlx_amd.engine import ContinuousEngine
    m, w, d = build("grouped", "float32")
    eng = ContinuousEngine(m, text_processor(d), slots=slots, window=256)
    jobs = [(tokens(d, n, 40 + n), k) for n, k in ((9, 6), (30, 3), (4, 9), (17, 1), (2, 7), (25, 5))]
    reqs = [eng.submit({"input_ids": t[None]}, k) for t, k in jobs]
    eng.run_until_idle()
    checked = 0
    for (t, k), r in zip(jobs, reqs):
        assert r.error is None and len(r.tokens) == k
        want, margin = greedy(d, w, t, k)
        if margin > 1e-3:
            assert r.tokens == want
            checked += 1
    assert checked >= 4 and eng.joined_mid_flight > 0
    m.serving = False


def test_mixed_length_requests_as_one_decode_batch():
    from phi_3_vision_mlx_amd.dist import generate_requests
    m, w, d = build("grouped", "float32")
    reqs = [tokens(d, n, n) for n in (50, 3, 21)]
    got = generate_requests(m, text_processor(d), [{"input_ids": t[None]} for t in reqs], 6, return_tokens=True)
    for t, g in zip(reqs, got):
        want, margin = greedy(d, w, t, 6)
        assert margin < 1e-3 or g == want


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(tmp_path, dtype):
    """A directory written with this family's names, replayed by trace.Replay: batches that end row by row, wanted places in order."""
    from phi_3_vision_mlx_amd.api import load
    from phi_3_vision_mlx_amd.trace import Replay
    from phi_3_vision_mlx_amd.weights import save_safetensors_dir
    d = config_dict(CONFIGS["uneven"])
    w = make_weights(d, seed=3)
    save_safetensors_dir({k: torch.as_tensor(v).to(BF16) for k, v in w.items()}, d, str(tmp_path))
    m, _ = load(model_path=str(tmp_path), dtype=dtype)
    full = {"a": tokens(d, 30, 1), "b": tokens(d, 9, 2), "c": tokens(d, 50, 3)}
    want = {k: orc.forward(d, w, t) for k, t in full.items()}
    rp, at = Replay(m, 200), {"a": 20, "b": 4, "c": 44}
    rows = rp.step([{"id": k, "tokens": full[k][:n].tolist(), "want": [n - 1, 0]} for k, n in at.items()])
    for i, (k, n) in enumerate(at.items()):
        assert rel(np.stack([host(r) for r in rows[2 * i:2 * i + 2]]), want[k][[n - 1, 0]]) < TOL[dtype]
    while at:
        es = [{"id": k, "tokens": [int(full[k][n])], "want": [0]} for k, n in at.items()]
        rows = rp.step(es)
        for e, r in zip(es, rows):
            assert rel(host(r)[None], want[e["id"]][at[e["id"]]][None]) < TOL[dtype], e
        at = {k: n + 1 for k, n in at.items()}
        done = [k for k, n in at.items() if n == len(full[k])]
        rp.end(done)
        at = {k: n for k, n in at.items() if k not in done}
    assert not rp.of
