"""Layered text decoders without a GPU: configuration, registry, weight table and loader, tokenizer, cache state, trace replay logic, host-side
launch planning, and the plain statement (oracle/pelalix_oracle.py) against itself."""
import json
import os
import re

import numpy as np
import pytest
import torch

import pelalix_oracle as orc
from phi_3_vision_mlx_amd import _lib, cache, config, registry, trace, weights
from phi_3_vision_mlx_amd.engine import ContinuousEngine
from phi_3_vision_mlx_amd.processor import ByteTokenizer, TextProcessor

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def cfg_dict(**kw):
    def layer(H, G, dim, vdim, mix, ff):
        return {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "scale": 0.2, "v_mix": mix},
                "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    d = {"architecture": "Pelalix", "width": 48, "vocab": 280, "norm": {"eps": 2e-5}, "embedding": {"scale": 3.0},
         "layers": [layer(3, 1, 16, 8, False, 40), layer(4, 2, 8, 12, True, None), layer(2, 2, 24, 12, True, 24)]}
    return {**d, **kw}


# ---------------------------------------------------------------- configuration, registry, weights
def test_config_reads_every_layer():
    c = config.make_config(cfg_dict(), dtype="float32", shift_rows=16)
    assert (c.hidden_size, c.vocab_size, c.num_hidden_layers, c.embed_scale, c.norm_eps, c.dtype, c.shift_rows) == (48, 280, 3, 3.0, 2e-5, "float32", 16)
    assert [(s.mixer.heads, s.mixer.dim, s.mixer.v_mix, s.mlp and s.mlp.ff) for s in c.layers] == [(3, 16, False, 40), (4, 8, True, None), (2, 24, True, 24)]
    assert registry.family(c).layered and registry.family(c).name == "Pelalix"


@pytest.mark.parametrize("change,match", [
    (lambda d: d["layers"][0].update(type="conv"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "feed-forward kind"),
    (lambda d: d["layers"][0]["mixer"].update(kv_heads=2), "query heads over"),
    (lambda d: d["layers"][2]["mixer"].update(vdim=20), "value widths"),
    (lambda d: d.update(layers=[]), "without layers")])
def test_config_errors(change, match):
    d = json.loads(json.dumps(cfg_dict()))
    change(d)
    with pytest.raises(ValueError, match=match):
        config.make_config(d)


def test_options_a_family_does_not_have():
    for k in ("use_quantized_cache", "quantized_fp8", "quantized_int4"):
        with pytest.raises(ValueError, match="not available"):
            config.make_config(cfg_dict(), **{k: True})
    with pytest.raises(ValueError, match="dtype"):
        config.make_config(cfg_dict(), dtype="float16")
    with pytest.raises(ValueError, match="bfloat16"):
        config.make_config(config.tiny_config_dict(), dtype="float32")


def test_registry_names():
    for arch, name in (("Phi3VForCausalLM", "Phi3V"), ("Phi3ForCausalLM", "Phi3F"), ("Pelalix", "Pelalix")):
        assert registry.family_of_name(arch).name == name
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.family_of_name("Other")
    for f in registry.FAMILIES:                                  # every named unit is a source file
        for u in f.units or ():
            assert os.path.exists(os.path.join(ROOT, "phi-3-vision-mlx_amd", "csrc", f"p3v_{u}.hip")), u


def test_weight_table_and_loader(tmp_path):
    d = cfg_dict()
    c = config.make_config(d)
    w = weights.synth_weights(c, seed=1)
    assert [n for n, _, _ in weights.weight_specs(c)] == list(w)
    assert w["l0.mix.talk"].shape == (3, 3) and abs(float(w["l0.mix.talk"].float().diagonal().mean()) - 1) < 0.5
    assert "l1.mlp.gate" not in w and "l1.norm2" not in w        # a layer without a feed-forward
    assert "l0.mix.vmix" not in w and "l1.mix.vmix" not in w and "l2.mix.vmix" in w      # (read where something is blended in)
    weights.save_safetensors_dir(w, d, str(tmp_path))
    got = weights.load_safetensors_dir(str(tmp_path), config.load_config(str(tmp_path / "config.json")))
    assert all(torch.equal(got[k], v) for k, v in w.items())
    weights.save_safetensors_dir({**w, "l2.mix.o": w["l2.mix.o"][:, :-1].contiguous()}, d, str(tmp_path))
    with pytest.raises(ValueError, match="l2.mix.o"):
        weights.load_safetensors_dir(str(tmp_path), c)
    weights.save_safetensors_dir({k: v for k, v in w.items() if k != "l1.shift"}, d, str(tmp_path))
    with pytest.raises(KeyError, match="l1.shift"):
        weights.load_safetensors_dir(str(tmp_path), c)


def test_byte_tokenizer_of_a_small_vocabulary():
    t = ByteTokenizer(280)
    ids = t.encode("<|end|>é")
    assert max(ids) < 280 and t.decode(ids) == "<|end|>é"
    assert t.encode("ab", add_special_tokens=False)[1:] == [3 + ord("a"), 3 + ord("b")]
    with pytest.raises(ValueError, match="vocabulary of 64"):
        ByteTokenizer(64).encode("z")
    assert ByteTokenizer(40000).encode("<|end|>")[-1] == 32007
    out = TextProcessor(None, vocab_size=280)(["abc", "d"])
    assert out["mask"].tolist()[1][:2] == [0, 0] and out["input_ids"].shape == (2, 5)
    with pytest.raises(ValueError, match="no images"):
        TextProcessor(None, vocab_size=280)("a", images=[1])


# ---------------------------------------------------------------- state
def state(B=2, S=10, n=300, **kw):
    return cache.LayeredCacheState(config.make_config(cfg_dict(), **kw), B, S, n, "cpu")


def test_state_layout_views_and_scrub():
    st = state()
    assert [tuple(t.shape) for t in st.k] == [(2, 1, st.Tp, 32), (2, 2, st.Tp, 32), (2, 2, st.Tp, 32)]
    assert [tuple(t.shape) for t in st.v] == [(2, 1, st.Tp // 16, 32, 16), (2, 2, st.Tp // 16, 32, 16), (2, 2, st.Tp // 16, 32, 16)]
    assert st.Tp % 128 == 0 and st.Tp >= 310 and st.k[0].dtype == torch.bfloat16 and state(dtype="float32").k[0].dtype == torch.float32
    st.pad_len = torch.tensor([3, 0], dtype=torch.int32)
    v = st.row_view(slice(1, 2), 5, 7, 0)
    v.k[1][:] = 1
    v.shift[2][:] = 2
    assert v.B == 1 and v.offset == 7 and st.k[1][1].min() == 1 and st.k[1][0].max() == 0 and st.shift[2][1].min() == 2
    for t in st.k + st.v + st.shift:
        t.fill_(float("nan"))
    st.scrub(5, 40)
    assert torch.isfinite(st.k[0][:, :, 5:40]).all() and torch.isnan(st.k[0][:, :, 40:]).all()
    assert torch.isfinite(st.v[0][:, :, 1]).all() and torch.isnan(st.v[0][:, :, 0, :, :5]).all() and torch.isfinite(st.v[0][:, :, 0, :, 5:]).all()


def test_beams_repeat_rows():
    st = state()
    st.offset, st.pad_len = 20, torch.tensor([1, 4], dtype=torch.int32)
    for t in st.k + st.v + st.shift:
        t.normal_()
    b = st.beams(3, 6)
    assert b.B == 6 and b.Tp >= 26 and b.Tp % 32 == 0 and b.pad_len.tolist() == [1, 1, 1, 4, 4, 4]
    assert torch.equal(b.k[1][4, :, :20], st.k[1][1, :, :20]) and torch.equal(b.v[2][2, :, :1], st.v[2][0, :, :1]) and torch.equal(b.shift[0][5], st.shift[0][1])


def test_history_bounds_a_rewind():
    st = state(shift_rows=8)
    st.note_written(0, 30)
    st.note_written(30, 31)
    st.note_written(24, 26)                                      # the token before column 24 is still in the ring
    with pytest.raises(ValueError, match="history"):
        st.note_written(23, 24)
    st.note_written(0, 4)                                        # from the start: nothing is needed
    st.note_written(4, 5)


# ---------------------------------------------------------------- trace replay on a stand-in model
class EchoModel:
    """Logits row = [position in the request, token, batch row]; rows are told apart by the padding."""
    device = "cpu"

    def __call__(self, input_ids, max_tokens, full_logits, pids=None, mask=None):
        ids = np.asarray(input_ids)
        m = np.ones_like(ids) if mask is None else np.asarray(mask)
        self.room = max_tokens
        st = type("S", (), {"B": ids.shape[0], "Tp": 64, "graphs": {}, "pad_len": torch.as_tensor((m == 0).sum(1)).int(), "n": m.sum(1)})()
        pos = m.cumsum(1) - 1
        return torch.as_tensor(np.stack([pos, ids, np.broadcast_to(np.arange(len(ids))[:, None], ids.shape)], -1)), [type("L", (), {"state": st})()]

    def greedy_step(self, tok, cache):
        st = cache[0].state
        out = torch.stack([torch.as_tensor(st.n), tok[:, 0].long(), torch.arange(st.B)], -1)[:, None]
        st.n = st.n + 1
        return out, None


def test_trace_replay_order_and_ends():
    m = EchoModel()
    rp = trace.Replay(m, 50)
    rows = rp.step([{"id": "x", "tokens": [7, 8, 9], "want": [2, 0]}, {"id": "y", "tokens": [5], "want": [0]}, {"id": "z", "tokens": [4, 4], "want": []}])
    assert [r.tolist() for r in rows] == [[2, 9, 0], [0, 7, 0], [0, 5, 1]] and m.room == 49
    rp.end(["y"])
    st = rp.of["x"].cache[0].state
    assert st.pad_len.tolist() == [0, 64, 1]
    rows = rp.step([{"id": "z", "tokens": [3], "want": [0]}, {"id": "x", "tokens": [2], "want": [0]}])     # (the step's order, not the batch's)
    assert [r.tolist() for r in rows] == [[2, 3, 2], [3, 2, 0]]
    with pytest.raises(ValueError, match="advances by one"):
        rp.step([{"id": "z", "tokens": [3, 3], "want": []}, {"id": "x", "tokens": [2], "want": []}])
    with pytest.raises(ValueError, match="together"):
        rp.step([{"id": "z", "tokens": [3], "want": []}])
    rp.end(["x", "z"])
    assert not rp.of
    assert [r.tolist() for r in rp.step([{"id": "x", "tokens": [1], "want": [0]}])] == [[0, 1, 0]]          # a name used again


def test_trace_command_refuses_bad_arguments():
    with pytest.raises(SystemExit) as e:
        trace.main(["--model", "m", "--dtype", "int8", "--out", "o", "--max-tokens", "4"])
    assert e.value.code == 2
    assert os.access(os.path.join(ROOT, "bin", "trace_run"), os.X_OK)


def test_engine_without_position_regimes_takes_any_window():
    class M:
        rope_regimes, device = False, "cpu"

        def new_slot_state(self, slots, window):
            return type("S", (), {"offset": 0, "T": window, "graphs": {}})()
    e = ContinuousEngine(M(), None, slots=2, window=9000)
    assert e.accepts(10, 20) and e.accepts(8000, 1000) and not e.accepts(8000, 1001)


# ---------------------------------------------------------------- library
def test_launch_planning_and_struct_layouts():
    l = _lib.lib()
    assert l.p3v_attn_mix_plan(1, 1, 32, 8, 96, 96, 2176, 0) == 136 and l.p3v_attn_mix_plan(1, 1, 32, 8, 96, 96, 8320, 0) <= 260
    assert l.p3v_attn_mix_plan(8, 1, 32, 8, 96, 96, 2176, 0) <= 32 and l.p3v_attn_mix_plan(1, 4096, 32, 8, 96, 96, 4096, 0) in range(1, 17)
    for bad in ((1, 1, 33, 11, 96, 96, 100, 0), (1, 1, 8, 8, 160, 96, 100, 0), (1, 1, 8, 8, 96, 96, 100, 1), (0, 1, 8, 8, 96, 96, 100, 0)):
        assert l.p3v_attn_mix_plan(*bad) == 0                    # the any-size kernel
    assert l.p3v_attn_mix_ws_bytes(2, 3, 4, 10, 5) == 2 * 3 * 5 * 4 * 12 * 4
    h = open(os.path.join(ROOT, "include", "p3v.h")).read()
    for cname, cls in (("p3v_dyt_args_t", _lib.DytArgs), ("p3v_mix_args_t", _lib.MixArgs)):
        end = h.index("} " + cname)
        body = re.sub(r"/\*.*?\*/", "", h[h.rindex("typedef struct {", 0, end) + len("typedef struct {"):end], flags=re.S)
        names = []
        for stmt in filter(None, (x.strip() for x in body.split(";"))):
            names += [n.strip().lstrip("*").strip() for n in re.sub(r"^(const\s+)?(void|uint16_t|int32_t|float|int)\s*\*?\s*", "", stmt).split(",")]
        assert names == [f for f, _ in cls._fields_], cname


def test_launchers_reject_what_their_kernels_do_not_take():
    """Argument checks come before any launch: they run without a GPU."""
    import ctypes as C
    l = _lib.lib()
    P = 1 << 20
    ok = dict(qkv=P, q_norm=P, k_norm=P, q=P, k=P, v=P, talk=P, sink=P, gate=P, out=P, ws=P, eps=1e-5, scale=1.0, B=1, L=4, H=4, G=2, dim=32, vdim=32,
              dimp=32, vdimp=32, ld=300, Tp=64, past=0, n_split=1)
    for bad in (dict(k=0), dict(G=3), dict(dimp=48), dict(dimp=16), dict(vdimp=40), dict(Tp=60), dict(past=61), dict(L=0), dict(talk=0), dict(n_split=-1),
                dict(n_split=2, ws=0), dict(n_split=17)):
        assert l.p3v_attn_mix(C.byref(_lib.MixArgs(**{**ok, **bad})), None) == -22, bad
    assert l.p3v_attn_mix_decode(C.byref(_lib.MixArgs(**ok)), None) == _lib.ERR_UNSUPPORTED           # more than one token
    assert l.p3v_qkv_heads(C.byref(_lib.MixArgs(**{**ok, "q_norm": 0})), None) == -22
    d = dict(x=P, w=P, b=P, alpha=1.0, B=1, L=1, H=3072)
    assert l.p3v_dyt(C.byref(_lib.DytArgs(**{**d, "mu": P})), P, 0, None) == -22                       # a shift without a history
    assert l.p3v_dyt(C.byref(_lib.DytArgs(**{**d, "mu": P, "hist": P, "hist_rows": 1})), P, 0, None) == -22
    g = _lib.GemvArgs(W=P, out=P, M=1, N=64, K=3000)
    assert l.p3v_gemv_dyt(C.byref(g), C.byref(_lib.DytArgs(**d)), None) == -22                         # widths differ
    g.K = 3072
    g.epilogue = _lib.EPI_RESID_BF16
    assert l.p3v_gemv_dyt(C.byref(g), C.byref(_lib.DytArgs(**d)), None) == _lib.ERR_UNSUPPORTED


def test_partial_library_names_what_it_lacks():
    class Half:
        p3v_version = staticmethod(lambda: 1)
    p = _lib._Partial(Half())
    assert p.p3v_version() == 1
    with pytest.raises(RuntimeError, match="p3v_gemm_fp8 is not part"):
        p.p3v_gemm_fp8(None, None)


# ---------------------------------------------------------------- the plain statement against itself
def small_weights(d, seed=0):
    c = config.make_config(d)
    return {k: v.float().numpy() * (6 if k.endswith(("mix.q", "mix.k", "mix.v", "mix.o", "gate", "up", "down", "head")) else 1)
            for k, v in weights.synth_weights(c, seed=seed).items()}


def test_oracle_is_causal_and_sees_every_mechanism():
    d = cfg_dict()
    w = small_weights(d)
    t = np.random.default_rng(0).integers(0, d["vocab"], 24)
    full = orc.forward(d, w, t)
    for n in (1, 2, 13):
        assert np.allclose(orc.forward(d, w, t[:n]), full[:n], atol=1e-12)
    for fault in ("no_shift", "no_sink", "no_talk"):
        assert np.abs(orc.forward(d, w, t, **{fault: True}) - full).max() > 1e-4 * np.abs(full).max(), fault
    other = dict(w, **{"l2.mix.vmix": w["l2.mix.vmix"] * 0})
    assert np.abs(orc.forward(d, other, t) - full).max() > 1e-4 * np.abs(full).max()


def test_oracle_mechanisms_by_hand():
    assert np.allclose(orc.token_shift(np.array([[1.0], [3.0]]), np.array([0.25])), [[0.75], [2.5]])
    a = orc.softmax_sink(np.zeros((1, 1, 3)), np.array([0.0]))
    assert np.allclose(a, 0.25)                                  # three keys and the sink
    assert np.allclose(orc.mix_heads(np.array([[[1.0]], [[10.0]]]), np.array([[1.0, 2.0], [0.0, -1.0]])).ravel(), [21, -10])
    assert np.allclose(orc.rms_rows(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), 0.5), np.array([[3.0, 8.0]]) / np.sqrt(13.0))
    assert np.allclose(orc.dyt(np.array([0.0, 1e9]), 0.5, np.array([2.0, 2.0]), np.array([1.0, 1.0])), [1.0, 3.0])
    assert np.allclose(orc.mix_values(np.array([2.0]), np.array([4.0]), 0.25), [2.5])
