"""The Pudisun decoder on the GPU against the plain float64 statement (oracle/pudisun_oracle.py): each mechanism alone, then the model through
the framework's own entry points.  Configurations and weights are made here; sizes vary per layer where that can hide a fault."""
import numpy as np
import pytest
import torch

import pudisun_oracle as orc

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


def i32(*v):
    return torch.tensor(v, dtype=I32, device=DEV)


def close(got, want, dt, what="", tight=1e-5):
    """Worst row and worst element of got - want, both against the rms of want: rounding of a bf16 (or fp32) result and its inputs."""
    d, s = np.asarray(got, dtype=np.float64) - want, np.sqrt((want ** 2).mean()) + 1e-30
    assert np.isfinite(d).all(), what
    row, worst = float(np.sqrt((d ** 2).mean(-1)).max() / s), float(np.abs(d).max() / s)
    assert row < (tight if dt == F32 else 0.04) and worst < (10 * tight if dt == F32 else 0.15), (what, row, worst)


DTYPES = ["float32", "bfloat16"]
TOL = {"float32": 3e-5, "bfloat16": 0.05}


# ---------------------------------------------------------------- row kernels and projections
@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("rows,H", [(1, 64), (5, 137), (9, 1024), (3, 1536), (70, 2048), (2, 3072), (2, 4096), (3, 5120)])
def test_rms_norm_of_fp32_rows(rows, H, dt):
    from phi_3_vision_mlx_amd import ops
    r = np.random.default_rng(H)
    x, w = r.normal(0, 2, (rows, H)) * 10.0 ** r.uniform(-4, 2, (rows, 1)), bf(r.normal(1, 0.4, H))
    xd = dev(x, F32)
    for eps, gain in ((1e-5, 1.0), (0.3, -0.37)):
        out = torch.full((rows, H), float("nan"), dtype=dt, device=DEV)
        ops.rms_rows(xd, (dev(w), eps, gain), out)
        want = orc.rms(host(xd), w, eps) * gain
        assert np.abs(host(out) - want).max() < (5e-6 if dt == F32 else 0.02) * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("K", [1024, 2048, 3072, 4096, 8192, 640])
@pytest.mark.parametrize("gelu", [False, True])
def test_rms_norm_in_the_projection_prologue(K, gelu):
    """One row: the fused launch (the last width: the two launches) = norm, then the projection."""
    from phi_3_vision_mlx_amd import ops
    r, N = np.random.default_rng(K), 96
    x, w, nw = r.normal(0, 3, (1, K)), bf(r.normal(0, K ** -0.5, (2 * N if gelu else N, K))), bf(r.normal(1, 0.3, K))
    xd, scratch, out = dev(x, F32), torch.empty((1, K), dtype=BF16, device=DEV), torch.full((1, N), float("nan"), dtype=BF16, device=DEV)
    y = orc.rms(host(xd), nw, 0.2) * -0.7 @ w.T
    ops.project_rms(xd, (dev(nw), 0.2, -0.7), dev(w), scratch, ops.EPI_GELU_MUL if gelu else ops.EPI_NONE, out=out)
    close(host(out), orc.gelu_tanh(y[:, :N]) * y[:, N:] if gelu else y, BF16)


@pytest.mark.parametrize("M,N,K", [(1, 64, 128), (1, 96, 3072), (2, 50, 136), (3, 40, 1024), (5, 96, 2048), (8, 64, 3072), (8, 40, 8192), (12, 128, 3072),
                                   (16, 192, 512), (20, 256, 3072), (60, 128, 1024), (100, 256, 1024), (300, 3072, 512), (1100, 512, 256), (7, 33, 72)])
@pytest.mark.parametrize("dt", [F32, BF16])
def test_gelu_gated_projection(M, N, K, dt):
    """gelu_tanh(gate) * up from every projection kernel, large gates of either sign included."""
    from phi_3_vision_mlx_amd import ops
    r = np.random.default_rng(M + N)
    a, w = r.normal(0, 1, (M, K)), bf(r.normal(0, 3 * K ** -0.5, (2 * N, K)))
    ad = dev(a, dt)
    y = host(ad) @ w.T
    close(host(ops.project(ad, dev(w), ops.EPI_GELU_MUL)), orc.gelu_tanh(y[:, :N]) * y[:, N:], dt)


# ---------------------------------------------------------------- latent attention
class Latent:
    """One mixer on the device and in the plain statement, from the packed projection's outputs on."""

    def __init__(self, H, dim, rot, vdim, rank, B, Tp, dt, seed=0, scale=None, scaling=None, base=10000.0):
        from phi_3_vision_mlx_amd import cache, config, mixers
        from phi_3_vision_mlx_amd.layered import LayeredModel
        self.r, self.B, self.Tp, self.dt = np.random.default_rng(seed), B, Tp, dt
        self.scale = (dim + rot) ** -0.5 if scale is None else scale
        self.d = {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": self.scale,
                  "rot": {"base": base, "dims": rot, "scaling": scaling}}
        self.m = config._latent_attention(0, self.d)
        r, W = self.r, 24
        self.w = {k: bf(v) for k, v in dict(q=np.zeros((H * (dim + rot), W)), dkv=np.zeros((rank + rot, W)), g=np.zeros((H * vdim, W)), o=np.zeros((W, H * vdim)),
                                            uk=r.normal(0, rank ** -0.5, (H * dim, rank)), uv=r.normal(0, rank ** -0.5, (H * vdim, rank)),
                                            sink=r.normal(1, 1, H)).items()}
        self.w["dkv.norm"] = bf(r.normal(1, 0.3, rank))
        self.eps = 1e-2
        cfg = type("C", (), {"norm_eps": self.eps, "dtype": "float32" if dt == F32 else "bfloat16"})
        self.mx = mixers.LatentHeads(self.m, {k: torch.as_tensor(v) for k, v in self.w.items()}, "", DEV, cfg)
        self.rows = cache.LatentRows(self.m, B, Tp, 2, dt, DEV)
        holder = type("H", (), {"_tables": {}, "device": torch.device(DEV)})()
        self.rows.cos, self.rows.sin = LayeredModel._rot_tables(holder, self.m.rot, Tp + 512)
        self.ld, self.n_out = self.mx.w_in.shape[0], H * vdim

    def y(self, T, spread=1.0):
        return dev(self.r.normal(0, spread, (self.B, T, self.ld)), self.dt)

    def run(self, y, past, pads=None, plan=None, d_past=False):
        """y [B, L, ld] -> [B, L, H, vdim]."""
        from phi_3_vision_mlx_amd import mixers
        L = y.shape[1]
        n_keys = self.Tp if L == 1 else past + L
        plan = self.mx.plan(self.B, L, n_keys) if plan is None else plan
        self.mx.plan, kept = lambda *a: plan, self.mx.plan
        bufs = {k: torch.full((n,), float("nan") if k != "q" else 0.0, dtype=dt, device=DEV) for k, (n, dt) in self.mx.buffers(self.B, L, n_keys).items()}
        self.mx.plan = kept
        out = torch.full((self.B * L, self.n_out), float("nan"), dtype=self.dt, device=DEV)
        call = mixers.Call(self.B, L, 0 if d_past else past, L, i32(past) if d_past else None, None if pads is None else i32(*pads))
        self.mx.run(y.clone().view(self.B * L, self.ld), out, self.rows, bufs, call, plan)
        return host(out).reshape(self.B, L, self.m.heads, self.m.vdim)

    def oracle(self, y, pad=0, **faults):
        """Rows [T, H, vdim] of one sequence of packed rows [T, ld]; rows of padding are zero."""
        m, d = self.m, self.d
        x, H, W = y[pad:], m.heads, m.dim + m.rot.dims
        pos = np.arange(len(x))
        q = x[:, :H * W].reshape(-1, H, W)
        q = np.concatenate([q[..., :m.dim], orc.rotate(q[..., m.dim:], pos, d["rot"], faults.pop("no_mscale", False))], axis=-1)
        lat = x[:, H * W:H * W + m.rank + m.rot.dims]
        o = orc.latent_core(q, orc.rms(lat[:, :m.rank], self.w["dkv.norm"], self.eps), orc.rotate(lat[:, m.rank:], pos, d["rot"]), self.w["uk"], self.w["uv"],
                            self.w["sink"], d, **faults)
        g0 = H * W + m.rank + m.rot.dims
        o = o * orc.sigmoid(x[:, g0:g0 + self.n_out]).reshape(o.shape)
        return np.concatenate([np.zeros((pad,) + o.shape[1:]), o])


YARN = {"factor": 3.0, "original": 96, "fast": 20.0, "slow": 1.5}
LATENT_SIZES = [(4, 32, 16, 48, 72), (16, 64, 32, 96, 512), (24, 128, 64, 128, 512), (3, 8, 8, 8, 8), (20, 40, 24, 72, 136), (17, 96, 64, 256, 320),
                (5, 20, 6, 18, 40), (2, 64, 96, 64, 640), (6, 24, 2, 40, 56)]


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("H,dim,rot,vdim,rank", LATENT_SIZES)
def test_latent_attention_prompt_portions_and_decode(H, dim, rot, vdim, rank, dt):
    """A prompt, portions behind it, then single tokens (positions as host value and from the device), rows of unequal padding."""
    B, parts, pads = 3, [45, 2, 17, 16, 40] + [1] * 5, [0, 7, 40]
    m = Latent(H, dim, rot, vdim, rank, B, 192, dt, seed=H, scaling=YARN if H % 2 else None, scale=-0.2 if H == 17 else None)
    y = m.y(sum(parts))
    want = np.stack([m.oracle(host(y)[b], pads[b]) for b in range(B)])
    past = 0
    for k, L in enumerate(parts):
        got = m.run(y[:, past:past + L].contiguous(), past, pads, d_past=L == 1 and k % 2 == 1)
        for b in range(B):
            lo = max(0, pads[b] - past)
            if lo < L:
                close(got[b, lo:], want[b, past + lo:past + L], dt, (b, past, L))
        past += L


@pytest.mark.parametrize("H,dim,rot,vdim,rank", [(4, 32, 16, 48, 72), (18, 64, 32, 96, 512)])
def test_latent_attention_forms_agree(H, dim, rot, vdim, rank):
    """In the latent space with any number of key splits (more than tiles included), over expanded keys, and the any-size kernel: the same rows."""
    B, L, past, pads = 2, 12, 150, [0, 155]
    m = Latent(H, dim, rot, vdim, rank, B, 192, BF16, seed=3, scaling=YARN)
    y = m.y(past + L)
    want = np.stack([m.oracle(host(y)[b], pads[b]) for b in range(B)])
    m.run(y[:, :past].contiguous(), 0, pads)
    for plan in (1, 2, 3, 7, 128, -1, 0):
        got = m.run(y[:, past:].contiguous(), past, pads, plan=plan)
        close(got[0], want[0, past:], BF16, plan), close(got[1, 5:], want[1, 155:], BF16, plan)
    one = m.y(1)
    full = torch.cat([y, one], dim=1)
    want = np.stack([m.oracle(host(full)[b], pads[b])[-1] for b in range(B)])
    for plan in (1, 2, 3, 128, 0):
        close(m.run(one, past + L, pads, plan=plan, d_past=plan == 2)[:, 0], want, BF16, plan)


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("far", [0, 1, 15, 63, 64, 127, 128, 255, 256, 399])
def test_one_far_key_decides(far, dt):
    """One key among hundreds carries almost all of the weight next to the sink; its place is at tile borders, in prompts and in decode.  The same
    comparison without that key, or without the sink, is far off: the test can see both."""
    H, dim, rot, vdim, rank, T = 8, 32, 16, 32, 64, 401
    m = Latent(H, dim, rot, vdim, rank, 1, 448, dt, seed=far, scale=0.3)
    x = m.r.normal(0, 0.3, (1, T, m.ld))
    c = orc.rms(x[0, far, H * (dim + rot):H * (dim + rot) + rank], m.w["dkv.norm"], m.eps)
    key = (c @ m.w["uk"].T).reshape(H, dim)
    q = np.zeros((H, dim + rot))
    q[:, :dim] = key / np.linalg.norm(key, axis=1, keepdims=True) ** 2 * 40
    x[0, -1, :H * (dim + rot)] = q.reshape(-1)
    y = dev(x, dt)
    m.w["sink"] = bf(np.full(H, 12.0))                           # (the score is 40 * 0.3: the sink takes about half)
    m.mx.sink = dev(m.w["sink"])
    want = m.oracle(host(y)[0])
    tol = 5e-5 if dt == F32 else 0.06
    assert np.abs(m.run(y, 0)[0, -1] - want[-1]).max() < tol
    m.run(y[:, :-1].contiguous(), 0)
    for plan in (None, 0) if dt == F32 else (None, 1, 0):
        assert np.abs(m.run(y[:, -1:].contiguous(), T - 1, plan=plan)[0, 0] - want[-1]).max() < tol
    assert np.abs(m.oracle(host(y)[0], hide=far)[-1] - want[-1]).max() > 3 * tol
    assert np.abs(m.oracle(host(y)[0], no_sink=True)[-1] - want[-1]).max() > 3 * tol


def test_rotation_reaches_far_positions():
    """Scores that live in the rotated part alone, at positions of some thousands: angles in 32 bits, YaRN's factor, both ends of its ramp."""
    m = Latent(2, 8, 32, 16, 16, 1, 4096, F32, seed=5, scaling={"factor": 8.0, "original": 512, "fast": 32.0, "slow": 1.0}, scale=0.4, base=50.0)
    y = m.y(3000)
    y[:, :, 8:40] *= 2
    want = m.oracle(host(y)[0])
    got = m.run(y, 0)[0]
    assert np.abs(got - want).max() < 2e-3 * np.abs(want).max()
    assert np.abs(m.oracle(host(y)[0], no_mscale=True) - want).max() > 0.05 * np.abs(want).max()


# ---------------------------------------------------------------- gated linear attention
class Gla:
    def __init__(self, H, dim, vdim, rank, B, dt, seed=0, tau=12.0, bias=(2.0, 1.5), R=2):
        from phi_3_vision_mlx_amd import config, mixers
        self.r, self.B, self.dt, self.R, self.tau = np.random.default_rng(seed), B, dt, R, tau
        self.m = config.GlaMixer(H, dim, vdim, tau)
        r, W = self.r, 16
        self.w = {k: bf(v) for k, v in dict(q=np.zeros((H * dim, W)), k=np.zeros((H * dim, W)), v=np.zeros((H * vdim, W)), g=np.zeros((H * vdim, W)),
                                            a1=np.zeros((rank, W)), o=np.zeros((W, H * vdim)), a2=r.normal(0, rank ** -0.5, (H * dim, rank)),
                                            norm=r.normal(1, 0.4, vdim)).items()}
        self.w["a2.b"] = bf(r.normal(*bias, H * dim))
        self.eps = 1e-3
        cfg = type("C", (), {"norm_eps": self.eps, "dtype": "float32" if dt == F32 else "bfloat16"})
        self.mx = mixers.LinearState(self.m, {k: torch.as_tensor(v) for k, v in self.w.items()}, "", DEV, cfg)
        self.s = torch.full((B, R, H, dim, vdim), float("nan"), dtype=F32, device=DEV)
        self.ld = self.mx.w_in.shape[0]

    def y(self, T):
        return dev(self.r.normal(0, 1, (self.B, T, self.ld)), self.dt)

    def run(self, y, past, pads=None, keep=None, plan=None, d_past=False):
        from phi_3_vision_mlx_amd import mixers, ops
        L = y.shape[1]
        plan = self.mx.plan(self.B, L, 0) if plan is None else plan
        ws = torch.full((ops.gla_ws_bytes(self.m, self.B, L, plan) // 4 + 4,), float("nan"), dtype=F32, device=DEV)
        out = torch.full((self.B * L, self.m.heads * self.m.vdim), float("nan"), dtype=self.dt, device=DEV)
        call = mixers.Call(self.B, L, 0 if d_past else past, L if keep is None else keep, i32(past) if d_past else None, None if pads is None else i32(*pads))
        ops.gated_linear_attention(self.mx, y.view(self.B * L, self.ld), out, self.s, ws, call, plan)
        return host(out).reshape(self.B, L, -1)

    def parts(self, x):
        m = self.m
        n, nv = m.heads * m.dim, m.heads * m.vdim
        q, k, v = (x[:, a:b].reshape(len(x), m.heads, -1) for a, b in ((0, n), (n, 2 * n), (2 * n, 2 * n + nv)))
        loga = orc.gla_decay(x[:, 2 * (n + nv):2 * (n + nv) + self.mx.rank], self.w["a2"], self.w["a2.b"], self.tau).reshape(len(x), m.heads, m.dim)
        return q * m.dim ** -0.5, k, v, loga, x[:, 2 * n + nv:2 * (n + nv)]

    def oracle(self, y, pad=0):
        """Output rows [T, H vdim] (padding: zero) and the last state of one sequence of packed rows."""
        q, k, v, loga, g = self.parts(y[pad:])
        o, s = orc.gla_scan(q, k, v, loga)
        o = orc.rms(o, self.w["norm"], self.eps).reshape(len(g), -1) * orc.silu(g)
        return np.concatenate([np.zeros((pad, o.shape[1])), o]), s


GLA_SIZES = [(6, 56, 72, 12), (2, 96, 192, 16), (3, 128, 256, 40), (5, 8, 8, 4), (2, 64, 24, 33), (3, 24, 96, 8), (2, 20, 36, 16), (1, 7, 10, 3), (2, 160, 64, 16)]


@pytest.mark.parametrize("dt", [F32, BF16])
@pytest.mark.parametrize("H,dim,vdim,rank", GLA_SIZES)
def test_gla_prompt_portions_and_decode(H, dim, vdim, rank, dt):
    """Portions at and off the chunk length, single tokens, both ways to pass the position, rows of unequal padding; the state itself as well."""
    B, parts, pads = 3, [70, 2, 64, 9, 1, 1, 130, 1, 3], [0, 7, 69]
    m = Gla(H, dim, vdim, rank, B, dt, seed=dim, R=2 + H % 2)
    y = m.y(sum(parts))
    past = 0
    want = [m.oracle(host(y)[b], pads[b])[0] for b in range(B)]
    for k, L in enumerate(parts):
        got = m.run(y[:, past:past + L].contiguous(), past, pads, d_past=k % 2 == 1)
        past += L
        for b in range(B):
            lo = max(0, pads[b] - (past - L))
            close(got[b, lo:], want[b][past - L + lo:past], dt, (b, past, L), tight=2e-5)
            s = m.oracle(host(y)[b, :past], pads[b])[1]
            assert np.abs(host(m.s[b, past % m.R]) - s).max() < 2e-5 * np.abs(s).max()       # (fp32 from the same inputs, whatever the activations)


@pytest.mark.parametrize("L,keeps", [(5, (0, 2, 5, 1)), (40, (0, 1, 17, 39)), (150, (0, 1, 64, 100, 128))])
def test_gla_keeps_the_state_of_the_tokens_that_stay(L, keeps):
    m = Gla(3, 40, 24, 16, 2, F32, seed=L)
    y0 = m.y(30)
    m.run(y0, 0)
    seq, past = [host(y0)[b] for b in range(2)], 30
    for keep in keeps:
        y = m.y(L)
        got = m.run(y, past, keep=keep)
        for b in range(2):
            close(got[b], m.oracle(np.concatenate([seq[b], host(y)[b]]))[0][past:], F32, (keep, b), tight=2e-5)
            seq[b] = np.concatenate([seq[b], host(y)[b, :keep]])
        past += keep


@pytest.mark.parametrize("tau,bias", [(1.0, (-30.0, 12.0)), (2.0, (-3.0, 4.0)), (16.0, (12.0, 3.0)), (0.25, (0.0, 60.0))])
def test_gla_decays_of_every_strength(tau, bias):
    """Channels that forget within a token next to channels that keep everything: pairs inside a block, across blocks and across chunks."""
    for dt in (F32, BF16):
        m = Gla(2, 32, 40, 16, 2, dt, seed=1, tau=tau, bias=bias)
        y = m.y(200)
        want = [m.oracle(host(y)[b])[0] for b in range(2)]
        a, b = m.run(y, 0), m.run(y, 0, plan=0)
        for i in range(2):
            close(a[i], want[i], dt, tight=5e-5), close(b[i], want[i], dt, tight=5e-5)


@pytest.mark.parametrize("far", [0, 1, 15, 16, 63, 64, 65, 127, 128, 190])
def test_gla_one_far_token_is_remembered(far):
    """One token writes, much later one asks for it, nothing else is in the state: a chunk or block that loses or doubles a token shows."""
    m = Gla(2, 16, 24, 8, 1, F32, seed=far, bias=(9.0, 0.5))
    n, T = 2 * 16, 193
    x = np.zeros((1, T, m.ld))
    x[0, far, n:2 * n], x[0, far, 2 * n:2 * n + 48] = m.r.normal(0, 1, n), m.r.normal(0, 1, 48)
    x[0, far:, :n], x[0, :, 2 * n + 48:2 * n + 96] = x[0, far, n:2 * n], 2.0
    y = dev(x, F32)
    want = m.oracle(host(y)[0])[0]
    for cut in (T, 64, 100, 7, 1):
        got = np.concatenate([m.run(y[:, t:t + cut].contiguous(), t)[0] for t in range(0, T, cut)])
        assert np.abs(got - want).max() < 3e-5 * np.abs(want).max() and np.abs(want[-1]).max() > 0.1, cut


# ---------------------------------------------------------------- configurations and weights
def latent(H, dim, rot, vdim, rank, scale=None, ff=None, scaling=YARN, base=700.0, **kw):
    return {"type": "latent_attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff}, **kw,
            "mixer": {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": (dim + rot) ** -0.5 if scale is None else scale,
                      "rot": {"base": base, "dims": rot, **({"scaling": scaling} if scaling else {})}}}


def gla(H, dim, vdim, tau=4.0, ff=None, **kw):
    return {"type": "gla", "mlp": None if ff is None else {"kind": "dense", "ff": ff}, "mixer": {"heads": H, "dim": dim, "vdim": vdim, "tau": tau}, **kw}


CONFIGS = {
    # one layer kind after another: own sizes per layer, layers without feed-forward, uneven sizes
    "uneven": dict(width=136, vocab=301, eps=3e-3, mult=0.6, lscale=1.7, layers=[
        gla(3, 20, 36, ff=200), latent(5, 24, 6, 18, 40, scale=0.31), latent(4, 40, 8, 24, 72, ff=72, scaling=None), gla(2, 40, 24, tau=1.0), gla(1, 7, 9, ff=40)]),
    # layers that use others' weights, with states of their own, out of order
    "shared": dict(width=192, vocab=512, eps=1e-5, mult=1.0, lscale=0.5, layers=[
        latent(8, 32, 16, 32, 64, ff=320), gla(4, 24, 32, ff=192), gla(4, 24, 32, ff=192, weights_of=1), latent(8, 32, 16, 32, 64, ff=320, weights_of=0),
        latent(6, 48, 32, 40, 96, ff=64), gla(4, 24, 32, ff=192, weights_of=2)]),
    "streamed": dict(width=1024, vocab=330, eps=1e-5, mult=0.8, lscale=0.4, layers=[latent(16, 64, 32, 64, 256, ff=1024), gla(8, 64, 128, tau=16.0, ff=2048)]),
    "many": dict(width=256, vocab=384, eps=1e-6, mult=-0.5, lscale=3.0, layers=[latent(32, 128, 64, 128, 512, ff=256), latent(20, 16, 32, 96, 136, ff=64), gla(16, 96, 160, ff=128)]),
}


def config_dict(c):
    return {"architecture": "Pudisun", "width": c["width"], "vocab": c["vocab"], "norm": {"eps": c["eps"]}, "residual_mult": c["mult"],
            "logit_scale": c["lscale"], "layers": c["layers"]}


def make_weights(cfg, seed=0):
    """Weights under which every mechanism shows in the logits: sharp attention, sinks that matter, decays of all strengths."""
    r = np.random.default_rng(seed)
    D, w = cfg["width"], {}
    w["embed"] = r.normal(0, 1, (cfg["vocab"], D))
    for i, ly in enumerate(cfg["layers"]):
        if ly.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", ly["mixer"]
        H, x = m["heads"], p + "mix."
        w[p + "norm1"] = r.normal(1, 0.3, D)
        if ly["type"] == "gla":
            n, nv, rank = H * m["dim"], H * m["vdim"], 5 + 3 * i
            for k, rows in (("q", n), ("k", n), ("v", nv), ("g", nv)):
                w[x + k] = r.normal(0, D ** -0.5, (rows, D))
            w[x + "a1"], w[x + "a2"], w[x + "a2.b"] = r.normal(0, D ** -0.5, (rank, D)), r.normal(0, rank ** -0.5, (n, rank)), r.normal(3, 2, n)
            w[x + "norm"], w[x + "o"] = r.normal(1, 0.3, m["vdim"]), r.normal(0, 1.5 * nv ** -0.5, (D, nv))
        else:
            R, rot, nv = m["kv_rank"], m["rot_dim"], H * m["vdim"]
            w[x + "q"], w[x + "dkv"], w[x + "dkv.norm"] = r.normal(0, 1.5 * D ** -0.5, (H * (m["dim"] + rot), D)), r.normal(0, 1.5 * D ** -0.5, (R + rot, D)), r.normal(1, 0.3, R)
            w[x + "uk"], w[x + "uv"] = r.normal(0, 1.5 * R ** -0.5, (H * m["dim"], R)), r.normal(0, 1.5 * R ** -0.5, (nv, R))
            w[x + "sink"], w[x + "g"], w[x + "o"] = r.normal(2, 1, H), r.normal(0, D ** -0.5, (nv, D)), r.normal(0, 2 * nv ** -0.5, (D, nv))
        if ly["mlp"]:
            ff = ly["mlp"]["ff"]
            w[p + "norm2"] = r.normal(1, 0.3, D)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = r.normal(0, 1.5 * D ** -0.5, (ff, D)), r.normal(0, 1.5 * D ** -0.5, (ff, D)), r.normal(0, 1.5 * ff ** -0.5, (D, ff))
    w["final.norm"] = r.normal(1, 0.3, D)
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


def rows_off(got, want):
    """Row errors: rms over the vocabulary of the difference / rms of the logits."""
    d = np.asarray(got, dtype=np.float64) - want
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((want ** 2).mean())


def rel(got, want):
    return float(rows_off(got, want).max())


def agree(got, want, dtype):
    """fp32: every row.  bf16: most rows tightly; a few may be far -- the norm behind a recurrence turns a state that is nearly orthogonal to
    its query (a sequence's first tokens) into a unit vector, and the rounding of q and k with it."""
    e = rows_off(got, want)
    if dtype == "float32":
        return bool(e.max() < TOL[dtype])
    return bool(np.median(e) < TOL[dtype] and np.quantile(e, 0.9) < 2.5 * TOL[dtype] and e.max() < 0.6)


# ---------------------------------------------------------------- the model
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_prompt_logits(name, dtype):
    m, w, d = build(name, dtype)
    for n in (1, 2, 16, 17, 90, 200):
        t = tokens(d, n, n)
        want = orc.forward(d, w, t)
        got, _ = m(input_ids=t[None], max_tokens=1, full_logits=True)
        assert got.dtype == (F32 if dtype == "float32" else BF16)
        assert agree(host(got)[0], want, dtype), n
        last, _ = m(input_ids=t[None], max_tokens=1)
        assert last.shape[1] == 1 and rel(host(last)[0], host(got)[0, -1:]) < 1e-6 + (0 if dtype == "float32" else 0.02)


def test_residual_stream_after_every_layer():
    m, w, d = build("shared", "float32")
    t, seen, want = tokens(d, 40, 4), [], []
    m.hidden_hook = lambda i, x, B, L: seen.append(host(x))
    try:
        m(input_ids=t[None], max_tokens=1, full_logits=True)
    finally:
        m.hidden_hook = None
    orc.forward(d, w, t, layers_out=want)
    assert len(seen) == len(want) and all(rel(a, b) < TOL["float32"] for a, b in zip(seen, want))


@pytest.mark.parametrize("fault", ["no_sink", "no_mscale", "no_gate", "no_decay", "forget_state", "eps", "scale", "tau", "residual_mult", "logit_scale", "weights_of"])
def test_the_comparison_sees_each_mechanism(fault):
    """The same comparison against an oracle with one mistake in it: out of tolerance by a wide margin (bf16 tolerance)."""
    m, w, d = build("shared", "bfloat16")
    t = tokens(d, 60, 3)
    got = host(m(input_ids=t[None], max_tokens=1, full_logits=True)[0])[0]
    kw = {fault: True} if fault.startswith(("no_", "forget")) else {}
    d2 = {**d, "layers": [dict(x, mixer=dict(x["mixer"])) for x in d["layers"]], "norm": dict(d["norm"])}
    if fault == "eps":
        d2["norm"]["eps"] = 0.5
    if fault == "scale":
        d2["layers"][4]["mixer"]["scale"] = 0.3
    if fault == "tau":
        d2["layers"][1]["mixer"]["tau"] = 1.0
    if fault in ("residual_mult", "logit_scale"):
        d2[fault] = 0.8 * d[fault]
    w2 = dict(w)
    if fault == "weights_of":                                    # (the layer has weights of its own)
        del d2["layers"][3]["weights_of"]
        w2.update({k.replace("l0.", "l3.", 1): np.roll(v, 1, axis=0) for k, v in w.items() if k.startswith("l0.")})
    off = np.median(rows_off(got, orc.forward(d2, w2, t, **kw)))
    assert agree(got, orc.forward(d, w, t), "bfloat16") and off > 1.5 * TOL["bfloat16"], off


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,cut", [("uneven", 2), ("uneven", 3), ("shared", 16), ("shared", 31), ("uneven", 64), ("many", 50)])
def test_portions_of_a_prompt(name, cut, dtype):
    """A prompt fed in portions through the cache gives the whole prompt's logits."""
    m, w, d = build(name, dtype)
    t = tokens(d, 140, cut)
    want = orc.forward(d, w, t)
    got, cache = m(input_ids=t[None, :cut], max_tokens=150, full_logits=True)
    rows = [host(got)[0]]
    while cache[0].offset < len(t):
        o = cache[0].offset
        got, cache = m(input_ids=t[None, o:o + cut], cache=cache)
        rows.append(host(got)[0])
    assert agree(np.concatenate(rows), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", CONFIGS)
def test_decode_token_by_token(name, dtype):
    """Eager one-token calls and the captured greedy step (teacher-forced), over tile and chunk borders; eager work between replays."""
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
        assert agree(np.concatenate(rows), want, dtype), start


def test_long_decode():
    m, w, d = build("shared", "float32")
    t = tokens(d, 420, 9)
    want = orc.forward(d, w, t)
    _, cache = m(input_ids=t[None, :3], max_tokens=430, full_logits=True)
    for i in range(3, len(t)):
        lg, _ = m.greedy_step(torch.tensor([[int(t[i])]], dtype=I32, device=DEV), cache)
        if i % 40 == 0 or i > 410:
            assert rel(host(lg)[0], want[i:i + 1]) < 2 * TOL["float32"], i


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["uneven", "shared", "many"])
def test_batches_of_unequal_requests(name, dtype):
    """Left-padded batches, prompt and decode, against each request alone in the oracle."""
    from phi_3_vision_mlx_amd.processor import collate_requests
    m, w, d = build(name, dtype)
    full = [tokens(d, n + 20, n) for n in (1, 2, 33, 64, 5, 130)]
    want = [orc.forward(d, w, t) for t in full]
    cut = [len(t) - 20 for t in full]
    got, cache = m(**collate_requests([{"input_ids": t[None, :c]} for t, c in zip(full, cut)]), max_tokens=24, full_logits=True)
    W = max(cut)
    rows = [[host(got)[b, W - c:]] for b, c in enumerate(cut)]
    for s in range(20):
        lg, _ = m.greedy_step(torch.tensor([[int(t[c + s])] for t, c in zip(full, cut)], dtype=I32, device=DEV), cache)
        for b in range(len(cut)):
            rows[b].append(host(lg)[b])
    for b in range(len(cut)):
        assert agree(np.concatenate(rows[b]), want[b], dtype), b


def test_rewind_and_read_only_beams():
    """advance_offset keeps the recurrent state of the columns that stay; a beam call leaves the cache as it was; one step back is exact; a
    state that is no longer held is an error, not a wrong answer."""
    m, w, d = build("shared", "float32")
    t = tokens(d, 40, 2)
    _, cache = m(input_ids=t[None, :20], max_tokens=200, full_logits=True)
    side = tokens(d, 27, 5)
    want_side = orc.forward(d, w, np.concatenate([t[:20], side]))[20:]
    for n in (27, 7, 1, 27):
        got, _ = m(input_ids=side[None, :n], cache=cache, advance_offset=0)
        assert rel(host(got)[0], want_side[:n]) < TOL["float32"] and cache[0].offset == 20
    beams = np.stack([tokens(d, 4, s) for s in range(3)])
    got, _ = m(input_ids=beams, cache=cache, n_beam=3, advance_offset=0)
    for b in range(3):
        assert rel(host(got)[b], orc.forward(d, w, np.concatenate([t[:20], beams[b]]))[20:]) < TOL["float32"]
    for keep, n in ((1, 3), (5, 27)):                            # keeps some of the columns
        t = np.concatenate([t[:cache[0].offset], side[:keep], t[20:]])
        got, _ = m(input_ids=side[None, :n], cache=cache, advance_offset=keep)
    o = cache[0].offset
    want = orc.forward(d, w, t)
    got, _ = m(input_ids=t[None, o:-2], cache=cache)
    assert rel(host(got)[0], want[o:-2]) < TOL["float32"]
    m(input_ids=side[None, :1], cache=cache)                     # one step that is taken back
    cache[0].offset -= 1
    got, _ = m(input_ids=t[None, -2:-1], cache=cache)
    assert rel(host(got)[0], want[-2:-1]) < TOL["float32"]
    m.greedy_step(i32(3).view(1, 1), cache)                      # the same of a captured step
    cache[0].offset -= 1
    got, _ = m.greedy_step(i32(int(t[-1])).view(1, 1), cache)
    assert rel(host(got)[0], want[-1:]) < TOL["float32"]
    m(input_ids=tokens(d, 50, 8)[None], cache=cache)
    cache[0].offset = 30
    with pytest.raises(ValueError, match="held"):
        m(input_ids=t[None, :2], cache=cache)


def test_captured_prefill_is_the_eager_one():
    """A prompt length seen twice is captured; later prompts of that length replay, with eager work in between, and each keeps its own
    cache while it is alive."""
    m, w, d = build("shared", "bfloat16")
    L, keep = 40, []
    for s in range(5):
        t = tokens(d, L + 6, 100 + s)
        lg, cache = m(input_ids=t[None, :L], max_tokens=9)
        want = orc.forward(d, w, t)
        rows = [host(lg)[0]]
        for i in range(L, L + 6):
            lg, _ = m.greedy_step(torch.tensor([[int(t[i])]], dtype=I32, device=DEV), cache)
            rows.append(host(lg)[0])
        assert agree(np.concatenate(rows), want[L - 1:], "bfloat16"), s
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
        margins.append((o[-1] - o[-2]) / np.abs(z).max())
        t.append(int(z.argmax()))
    return t[len(prompt):], min(margins)


def text_processor(d):
    from phi_3_vision_mlx_amd.processor import TextProcessor
    return TextProcessor(None, vocab_size=d["vocab"])


def test_greedy_generation_through_the_api():
    """api._generate on text: the tokens are the oracle's greedy tokens (fp32 model), one prompt and a padded batch."""
    from phi_3_vision_mlx_amd import api
    m, w, d = build("shared", "float32")
    proc = text_processor(d)
    n, prompts, want = 12, [], []
    for k in range(40):                                          # one short and one long prompt whose greedy choices are clear
        p = f"prompt {k}" if not prompts else f"a much longer prompt of a few dozen characters, number {k}"
        toks, margin = greedy(d, w, proc(p)["input_ids"][0], n)
        if margin > 1e-3:
            prompts.append(p), want.append(toks)
        if len(prompts) == 2:
            break
    assert len(prompts) == 2
    out = api._generate(m, proc, prompts[0], max_tokens=n, verbose=False, mute=True)
    assert (out[0] if isinstance(out, list) else out) == proc.tokenizer.decode(want[0])
    out = api._generate(m, proc, prompts, max_tokens=n, verbose=False, mute=True)
    assert out == [proc.tokenizer.decode(t) for t in want]
    picked = api._choose_from(m, proc, prompts[0], choices="ABC", mute=True)
    opts = [proc([f" {c}"])["input_ids"][0, -1] for c in "ABC"]
    z = orc.forward(d, w, proc(prompts[0])["input_ids"][0])[-1]
    assert picked == "ABC"[int(np.argmax(z[opts]))]


@pytest.mark.parametrize("use_beam", [False, True])
def test_constrained_decoding_runs_on_recurrent_states(use_beam):
    from phi_3_vision_mlx_amd import api
    m, w, d = build("shared", "float32")
    a = api._constrain(m, text_processor(d), ["hello"], [(3, " so")], mute=True, use_beam=use_beam, verbose=False)
    assert len(a) == 1 and a[0]


@pytest.mark.parametrize("slots", [2, 3])
def test_engine_reuses_slots(slots):
    """Continuous batching: more requests than slots, unequal prompts and budgets, rows freed and taken again mid-flight; every request's
    tokens are what the oracle alone generates."""
    from phi_3_vision_mlx_amd.engine import ContinuousEngine
    m, w, d = build("shared", "float32")
    eng = ContinuousEngine(m, text_processor(d), slots=slots, window=256)
    jobs = [(tokens(d, n, 40 + n), k) for n, k in ((9, 6), (70, 3), (4, 9), (17, 1), (2, 7), (25, 5), (66, 4))]
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
    m, w, d = build("shared", "float32")
    reqs = [tokens(d, n, n) for n in (50, 3, 21)]
    got = generate_requests(m, text_processor(d), [{"input_ids": t[None]} for t in reqs], 6, return_tokens=True)
    for t, g in zip(reqs, got):
        want, margin = greedy(d, w, t, 6)
        assert margin < 1e-3 or g == want


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(tmp_path, dtype):
    """A directory written with this family's names, replayed by trace.Replay: batches that end row by row, wanted places in order, a
    second batch on the memory of the first."""
    from phi_3_vision_mlx_amd.api import load
    from phi_3_vision_mlx_amd.trace import Replay
    from phi_3_vision_mlx_amd.weights import save_safetensors_dir
    d = config_dict(CONFIGS["uneven"])
    w = make_weights(d, seed=3)
    save_safetensors_dir({k: torch.as_tensor(v).to(BF16) for k, v in w.items()}, d, str(tmp_path))
    m, _ = load(model_path=str(tmp_path), dtype=dtype)
    rp = Replay(m, 200)
    for batch in range(2):
        full = {"a": tokens(d, 30, 1 + batch), "b": tokens(d, 9, 2 + batch), "c": tokens(d, 50, 3 + batch)}
        want = {k: orc.forward(d, w, t) for k, t in full.items()}
        at = {"a": 20, "b": 4, "c": 44}
        rows = rp.step([{"id": k, "tokens": full[k][:n].tolist(), "want": [n - 1, 0]} for k, n in at.items()])
        got = {k: [(n - 1, host(rows[2 * i])), (0, host(rows[2 * i + 1]))] for i, (k, n) in enumerate(at.items())}
        while at:
            es = [{"id": k, "tokens": [int(full[k][n])], "want": [0]} for k, n in at.items()]
            rows = rp.step(es)
            for e, r in zip(es, rows):
                got[e["id"]].append((at[e["id"]], host(r)))
            at = {k: n + 1 for k, n in at.items()}
            done = [k for k, n in at.items() if n == len(full[k])]
            rp.end(done)
            at = {k: n for k, n in at.items() if k not in done}
        assert not rp.of
        for k, rows in got.items():
            assert agree(np.stack([r for _, r in rows]), want[k][[i for i, _ in rows]], dtype), k
