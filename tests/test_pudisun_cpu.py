"""The Pudisun decoder without a GPU: configuration, registry, weight table and loader, rotary frequencies, cache states, host-side launch planning
and argument checks, and the plain statement (oracle/pudisun_oracle.py) against itself."""
import ctypes as C
import json
import os
import re

import numpy as np
import pytest
import torch

import pudisun_oracle as orc
from phi_3_vision_mlx_amd import _lib, cache, config, mixers, registry, weights

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
YARN = {"factor": 3.0, "original": 200, "fast": 16.0, "slow": 2.0}


def latent(H=3, dim=8, rot=4, vdim=12, rank=20, scaling=YARN, ff=40, **kw):
    return {"type": "latent_attention", "mixer": {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": 0.3,
                                                  "rot": {"base": 900.0, "dims": rot, **({"scaling": scaling} if scaling else {})}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}, **kw}


def gla(H=2, dim=12, vdim=20, tau=8.0, ff=None, **kw):
    return {"type": "gla", "mixer": {"heads": H, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}, **kw}


def cfg_dict(**kw):
    d = {"architecture": "Pudisun", "width": 48, "vocab": 280, "norm": {"eps": 2e-5}, "residual_mult": 0.6, "logit_scale": 1.5,
         "layers": [gla(), latent(), gla(H=1, ff=24), latent(weights_of=1), gla(weights_of=0), latent(H=4, scaling=None, ff=None)]}
    return {**d, **kw}


# ---------------------------------------------------------------- configuration, registry, weights
def test_config_reads_every_layer():
    c = config.make_config(cfg_dict(), dtype="float32", state_rows=3)
    assert (c.hidden_size, c.vocab_size, c.num_hidden_layers, c.norm_eps, c.residual_mult, c.logit_scale, c.embed_scale, c.dtype, c.state_rows) == \
        (48, 280, 6, 2e-5, 0.6, 1.5, 1.0, "float32", 3)
    assert [s.owner for s in c.layers] == [None, None, None, 1, 0, None]
    assert c.layers[1].mixer == config.LatentMixer(3, 8, 12, 20, config.Rotary(4, 900.0, (3.0, 200.0, 16.0, 2.0)), 0.3)
    assert c.layers[0].mixer == config.GlaMixer(2, 12, 20, 8.0) and c.layers[5].mixer.rot.yarn is None
    f = registry.family(c)
    assert f.layered and f.name == "Pudisun" and c.design.norm == "rms" and c.design.tied_head
    for u in f.units:                                            # every named unit is a source file
        assert os.path.exists(os.path.join(ROOT, "phi-3-vision-mlx_amd", "csrc", f"p3v_{u}.hip")), u


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][0].update(type="attention"), "mixer type"),
    (lambda d: d["layers"][1]["mlp"].update(kind="sparse"), "feed-forward kind"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=2), "rotary dimensions"),
    (lambda d: d["layers"][3].update(weights_of=9), "no layer has the weights"),
    (lambda d: d["layers"][3].update(weights_of=3), "no layer has the weights"),
    (lambda d: d["layers"][4].update(weights_of=2), "other sizes"),
    (lambda d: d.update(residual_mult=0), "residual_mult"),
    (lambda d: d.update(layers=[]), "without layers")])
def test_config_errors(change, match):
    d = json.loads(json.dumps(cfg_dict()))
    change(d)
    with pytest.raises(ValueError, match=match):
        config.make_config(d)


def test_options_the_family_does_not_have():
    for k in ("use_quantized_cache", "quantized_fp8", "quantized_int4"):
        with pytest.raises(ValueError, match="not available"):
            config.make_config(cfg_dict(), **{k: True})


def test_weights_of_a_chain_names_the_owner():
    c = config.make_config(cfg_dict(layers=[gla(), gla(weights_of=0), gla(weights_of=1), gla(weights_of=3 - 2)]))
    assert [s.owner for s in c.layers] == [None, 0, 0, 0]


@pytest.mark.parametrize("dims,base,s", [(16, 10000.0, None), (16, 50.0, YARN), (32, 1e6, dict(factor=40.0, original=4096, fast=32.0, slow=1.0)),
                                         (2, 10.0, YARN), (64, 500.0, dict(factor=1.0, original=64, fast=2.0, slow=2.0)), (8, 3.0, dict(factor=8.0, original=10000, fast=1e4, slow=1e-4))])
def test_rotary_frequencies(dims, base, s):
    f, mult = config.Rotary(dims, base, None if s is None else tuple(float(s[k]) for k in ("factor", "original", "fast", "slow"))).frequencies()
    want, wm = orc.frequencies({"dims": dims, "base": base, "scaling": s})
    assert np.allclose(f, want, rtol=1e-12) and mult == pytest.approx(wm) and len(f) == dims // 2


def test_weight_table_and_loader(tmp_path):
    d = cfg_dict()
    c = config.make_config(d)
    w = weights.synth_weights(c, seed=1)
    assert [n for n, _, _ in weights.weight_specs(c)] == list(w)
    assert "head" not in w and "l3.norm1" not in w and "l4.mix.q" not in w and "l0.norm2" not in w and "l2.norm2" in w and "l0.norm1.alpha" not in w
    assert tuple(w["l1.mix.dkv"].shape) == (24, 48) and tuple(w["l1.mix.uv"].shape) == (36, 20) and tuple(w["l0.mix.a2"].shape) == (24, weights.FREE_RANK)
    w["l0.mix.a1"], w["l0.mix.a2"] = w["l0.mix.a1"][:5].clone(), w["l0.mix.a2"][:, :5].clone()      # (the checkpoint decides the rank of the decay's projection)
    weights.save_safetensors_dir(w, d, str(tmp_path))
    got = weights.load_safetensors_dir(str(tmp_path), config.load_config(str(tmp_path / "config.json")))
    assert all(torch.equal(got[k], v) for k, v in w.items())
    weights.save_safetensors_dir({**w, "l0.mix.a2": w["l0.mix.a2"][:-1].contiguous()}, d, str(tmp_path))
    with pytest.raises(ValueError, match="l0.mix.a2"):
        weights.load_safetensors_dir(str(tmp_path), c)
    weights.save_safetensors_dir({k: v for k, v in w.items() if k != "l1.mix.sink"}, d, str(tmp_path))
    with pytest.raises(KeyError, match="l1.mix.sink"):
        weights.load_safetensors_dir(str(tmp_path), c)


def test_mixer_weights_are_packed_and_padded():
    c = config.make_config(cfg_dict())
    w = weights.synth_weights(c, seed=2)
    m = mixers.LatentHeads(c.layers[1].mixer, w, "l1.mix.", "cpu", c)
    assert m.w_in.shape == (128, 48) and torch.equal(m.w_in[:36], w["l1.mix.q"]) and torch.equal(m.w_in[36:60], w["l1.mix.dkv"]) and m.w_in[96:].abs().max() == 0
    assert m.uk.shape == (24, 64) and m.uk[:, 20:].abs().max() == 0 and m.ukt.shape == (3, 64, 32)
    assert torch.equal(m.ukt[2, :20, :8], w["l1.mix.uk"][16:24].T) and m.ukt[:, :, 8:].abs().max() == 0
    g = mixers.LinearState(c.layers[0].mixer, w, "l0.mix.", "cpu", c)
    assert g.rank == weights.FREE_RANK and torch.equal(g.w_in[128:128 + g.rank], w["l0.mix.a1"])
    with pytest.raises(ValueError, match="columns"):
        mixers.LinearState(c.layers[0].mixer, {**w, "l0.mix.a1": w["l0.mix.a1"][:3]}, "l0.mix.", "cpu", c)


# ---------------------------------------------------------------- state
def state(B=2, S=10, n=300, **kw):
    return cache.LayeredCacheState(config.make_config(cfg_dict(), **kw), B, S, n, "cpu")


def test_state_layout_views_beams_and_scrub():
    st = state(state_rows=3)
    assert st.recurrent and [type(m).__name__ for m in st.mix] == ["RecurrentRows", "LatentRows"] * 2 + ["RecurrentRows", "LatentRows"]
    assert tuple(st.mix[1].c.shape) == (2, st.Tp, 64 + 32) and tuple(st.mix[0].s.shape) == (2, 3, 2, 12, 20) and st.shift == [None] * 6
    assert st.mix[1].c is not st.mix[3].c and st.mix[0].s.dtype == torch.float32 and st.mix[1].c.dtype == torch.bfloat16
    st.pad_len = torch.tensor([3, 0], dtype=torch.int32)
    v = st.row_view(slice(1, 2), 5, 7, 0)
    v.mix[1].c[:] = 1
    v.mix[2].s[:] = 2
    assert v.B == 1 and v.offset == 7 and st.mix[1].c[1].min() == 1 and st.mix[1].c[0].max() == 0 and st.mix[2].s[1].min() == 2 and st.mix[2].s[0].max() == 0
    v.note_written(7, 12)                                        # (a fresh row needs no history)
    st.offset = 20
    b = st.beams(3, 6)
    assert b.B == 6 and b.Tp % 64 == 0 and b.Tp >= 26 and b.pad_len.tolist() == [3, 3, 3, 0, 0, 0]
    assert torch.equal(b.mix[1].c[4, :20], st.mix[1].c[1, :20]) and b.mix[2].s[3:].min() == 2 and b.mix[2].s.data_ptr() != st.mix[2].s.data_ptr()
    st.mix[1].c.fill_(float("nan"))
    st.scrub(5, 40)
    assert torch.isfinite(st.mix[1].c[:, 5:40]).all() and torch.isnan(st.mix[1].c[:, 40:]).all()


def test_recurrent_states_bound_a_rewind():
    st = state(state_rows=2)
    st.note_written(0, 30)
    st.note_written(30, 31)
    st.note_written(30, 31)                                      # one step back: the state behind 30 columns is still there
    st.note_written(31, 40, 31)                                  # nothing of it stays
    st.note_written(31, 40, 33)                                  # two columns stay: the slot of 31 is theirs now
    assert st.held == {30, 33}
    with pytest.raises(ValueError, match="held"):
        st.note_written(31, 32)
    with pytest.raises(ValueError, match="cannot follow"):
        st.note_written(33, 35, 36)
    st.note_written(33, 34)
    assert st.held == {33, 34}
    with pytest.raises(ValueError, match="held"):
        st.note_written(20, 21)
    st.note_written(0, 4)                                        # from the start: nothing is needed
    st.note_written(4, 5)


# ---------------------------------------------------------------- library
def test_struct_layouts_match_the_header():
    h = open(os.path.join(ROOT, "include", "p3v.h")).read()
    for cname, cls in (("p3v_gla_args_t", _lib.GlaArgs), ("p3v_latent_args_t", _lib.LatentArgs)):
        end = h.index("} " + cname)
        body = re.sub(r"/\*.*?\*/", "", h[h.rindex("typedef struct {", 0, end) + len("typedef struct {"):end], flags=re.S)
        names = []
        for stmt in filter(None, (x.strip() for x in body.split(";"))):
            names += [n.strip().lstrip("*").strip() for n in re.sub(r"^(const\s+)?(void|uint16_t|int32_t|float|int)\s*\*?\s*", "", stmt).split(",")]
        assert names == [f for f, _ in cls._fields_], cname


def test_launch_planning():
    l = _lib.lib()
    plan = lambda B, L, H=32, dim=64, rot=32, vdim=96, rank=512, n=2176, f32=0: l.p3v_latent_plan(B, L, H, dim, rot, vdim, rank, n, f32)   # noqa: E731
    assert plan(1, 1) == 34 and plan(1, 1, n=64) == 1 and 1 <= plan(64, 1) <= 34 and plan(1, 1, n=64 * 1000) <= 128 and plan(2, 16) > 0
    assert plan(1, 17) == -1 and plan(1, 300, rank=1024) == -1                                    # (the latent itself is only the small form's matter)
    for bad in (dict(f32=1), dict(dim=20), dict(rot=6), dict(vdim=18), dict(rank=1024), dict(rank=20), dict(rot=96)):
        assert plan(1, 1, **bad) == 0, bad
    for bad in (dict(f32=1), dict(dim=20), dict(dim=256), dict(vdim=264)):
        assert plan(1, 100, **bad) == 0, bad
    assert l.p3v_latent_ws_bytes(2, 3, 5, 100, 4) == 2 * 3 * 4 * 5 * (128 + 2) * 4
    assert l.p3v_gla_plan(1, 1, 4, 64, 96, 0) == 0 and l.p3v_gla_plan(2, 200, 4, 64, 96, 0) == 4 and l.p3v_gla_plan(2, 8, 4, 64, 96, 0) == 0
    for bad in ((1, 100, 4, 20, 96, 0), (1, 100, 4, 64, 36, 0), (1, 100, 4, 136, 96, 0), (1, 100, 4, 64, 264, 0)):
        assert l.p3v_gla_plan(*bad) == 0, bad
    assert l.p3v_gla_ws_bytes(2, 1, 4, 8, 8, 0) == 0 and l.p3v_gla_ws_bytes(2, 5, 4, 8, 8, 0) == 2 * 4 * 64 * 4
    assert l.p3v_gla_ws_bytes(2, 130, 4, 8, 16, 3) == (3 * 8 * (128 + 8) + 2 * 130 * 4 * 8) * 4


def test_launchers_reject_what_their_kernels_do_not_take():
    """Argument checks come before any launch: they run without a GPU."""
    l, P = _lib.lib(), 1 << 20
    ok = dict(y=P, c_norm=P, uk=P, ukt=P, uv=P, sink=P, cos_t=P, sin_t=P, c=P, q=P, kx=P, vx=P, out=P, ws=P, eps=1e-5, scale=1.0, B=1, L=4, H=4, dim=32, rot=16,
              vdim=32, rank=64, rankp=64, rotp=32, dimp=32, ld=512, past=0, Tp=128, tab_n=4096, n_keys=64, n_split=1)
    call = lambda fn, **kw: getattr(l, fn)(C.byref(_lib.LatentArgs(**{**ok, **kw})), None)   # noqa: E731
    for fn in ("p3v_latent_append", "p3v_latent_any", "p3v_latent_rows", "p3v_latent_prompt"):
        for bad in (dict(y=0), dict(c=0), dict(sink=0), dict(L=0), dict(rot=15), dict(rankp=96), dict(rankp=0), dict(rotp=8), dict(Tp=100), dict(past=125), dict(ld=300),
                    dict(tab_n=0), dict(past=-1)):
            assert call(fn, **bad) == -22, (fn, bad)
    for bad in (dict(n_split=0), dict(n_split=129), dict(ws=0), dict(q=0), dict(dimp=16), dict(rankp=128), dict(y=P + 2)):
        assert call("p3v_latent_rows", **bad) == -22, bad
    for bad in (dict(f32=1), dict(dim=20), dict(rank=576, rankp=576, ld=1024)):
        assert call("p3v_latent_rows", **bad) == _lib.ERR_UNSUPPORTED, bad
    for bad in (dict(n_keys=60), dict(n_keys=192), dict(kx=0), dict(past=61)):
        assert call("p3v_latent_prompt", **bad) == -22, bad
    for bad in (dict(f32=1), dict(vdim=264, ld=2048)):
        assert call("p3v_latent_prompt", **bad) == _lib.ERR_UNSUPPORTED, bad
    g = dict(y=P, a2=P, a2_b=P, norm=P, s=P, out=P, ws=P, eps=1e-5, tau=4.0, q_scale=0.1, B=1, L=20, H=2, dim=16, vdim=16, rank=4, ld=192, past=0, R=2, keep=20, n_chunk=1)
    for bad in (dict(s=0), dict(R=1), dict(keep=21), dict(keep=-1), dict(ld=100), dict(n_chunk=2), dict(n_chunk=-1), dict(ws=0), dict(n_chunk=0, ws=0), dict(past=-1), dict(rank=0)):
        assert l.p3v_gla(C.byref(_lib.GlaArgs(**{**g, **bad})), None) == -22, bad
    assert l.p3v_rms_rows(0, P, P, 0, 1, 8, 1e-5, 1.0, None) == -22
    a = _lib.GemvArgs(W=P, out=P, norm_w=P, M=1, N=64, K=3072, epilogue=_lib.EPI_RESID_BF16)
    assert l.p3v_gemv_rms(C.byref(a), P, 1.0, None) == _lib.ERR_UNSUPPORTED
    a.norm_w = 0
    assert l.p3v_gemv_rms(C.byref(a), P, 1.0, None) == -22


# ---------------------------------------------------------------- the plain statement against itself
def small_weights(d, seed=0):
    c = config.make_config(d)
    return {k: v.float().numpy() * (8 if k.endswith(("mix.q", "mix.k", "mix.v", "mix.o", "mix.g", "dkv", "uk", "uv", "a1", "a2", "gate", "up", "down", "embed")) else 1)
            for k, v in weights.synth_weights(c, seed=seed).items()}


def test_oracle_is_causal_and_sees_every_mechanism():
    d = cfg_dict()
    w = small_weights(d)
    t = np.random.default_rng(0).integers(0, d["vocab"], 24)
    full = orc.forward(d, w, t)
    for n in (1, 2, 13):
        assert np.allclose(orc.forward(d, w, t[:n]), full[:n], atol=1e-9)
    for fault in ("no_sink", "no_mscale", "no_gate", "no_decay", "forget_state"):
        assert np.abs(orc.forward(d, w, t, **{fault: True}) - full).max() > 1e-4 * np.abs(full).max(), fault
    for change in (dict(residual_mult=0.5), dict(logit_scale=1.0)):
        assert np.abs(orc.forward({**d, **change}, w, t) - full).max() > 1e-2 * np.abs(full).max()


def test_oracle_mechanisms_by_hand():
    assert np.allclose(orc.rms(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), 0.5), np.array([[3.0, 8.0]]) / np.sqrt(13.0))
    assert np.allclose(orc.softmax_sink(np.zeros((1, 1, 3)), np.array([0.0])), 0.25)              # three keys and the sink
    assert np.allclose(orc.gelu_tanh(np.array([0.0, 30.0, -30.0])), [0.0, 30.0, 0.0])
    r = orc.rotate(np.array([[1.0, 0.0, 7.0], [1.0, 0.0, 7.0]]), [0, 1], {"dims": 2, "base": 5.0})
    assert np.allclose(r, [[1, 0, 7], [np.cos(1), np.sin(1), 7]])
    r = orc.rotate(np.eye(4)[None, 0], [3], {"dims": 4, "base": 100.0})                           # (dimension 0 is paired with 2)
    assert np.allclose(r, [[np.cos(3), 0, np.sin(3), 0]])
    q = k = v = np.ones((3, 1, 1))
    o, s = orc.gla_scan(q, k, v, np.log(0.5) * np.ones((3, 1, 1)))
    assert np.allclose(o.ravel(), [1, 1.5, 1.75]) and np.allclose(s, 1.75)
    assert np.allclose(orc.gla_decay(np.zeros((1, 2)), np.zeros((3, 2)), np.zeros(3), 4.0), np.log(0.5) / 4)
    m = {"heads": 1, "dim": 1, "vdim": 1, "scale": 1.0}
    o = orc.latent_core(np.array([[[np.log(3.0), 0.0]]]), np.array([[0.0], [1.0]]), np.zeros((2, 1)), np.eye(1), np.eye(1), np.array([0.0]), m)
    assert np.allclose(o, 3 / 5)                                 # weights 1 : 3 next to the sink's 1
