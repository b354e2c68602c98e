"""Layered text decoders on MI355X: a decoder whose layers are described one by one in its config (config.LayerSpec), built from
mechanisms that take their constants as parameters (mixers.py).  Served through the same contract as the other models
(decoder.DecoderModel): `model(...)`, the captured greedy step, slot states of the engine.

Per layer, on a fp32 residual stream x (what a design has of it: config.Design):

    h  = token_shift(norm(x))                     dynamic tanh or RMS norm
    y  = W h                                      one projection for all that reads h, weights packed at load
    o  = mixer(y)                                 mixed-head attention | latent attention | gated linear attention
    x += ls1 * (W_o o)                            projection epilogue
    a  = act(W_gate h2) * (W_up h2), h2 = norm(x) norm + projection epilogue
    x += ls2 * (W_down a)                         projection epilogue

A multiplier m on every branch is taken out of the sum: the stream is kept divided by m, x / m = embed / m + sum of the branches, which
the norms undo (RMS norm of x with eps = sign(m) RMS norm of x / m with eps / m^2).

Activations are bf16, or fp32 throughout with dtype="float32" (weights stay bf16 data, which fp32 arithmetic reads exactly).
"""
import torch

from . import ops
from .cache import LatentRows, LayeredCacheState, MIXER_ROWS
from .decoder import DecoderModel
from .mixers import MIXERS, Call
from .ops import BF16, EPI_GELU_MUL, EPI_NONE, EPI_SCALE_RESID_F32, EPI_SILU_MUL, F32

ACTS = {"silu": EPI_SILU_MUL, "gelu_tanh": EPI_GELU_MUL}


class DynamicTanh:
    """tanh(alpha x) w + b in place of a norm."""

    def __init__(self, w, name, dev, cfg, gain=1.0):
        if cfg.residual_mult != 1.0 or gain != 1.0:
            raise ValueError("a dynamic tanh has no scale to take a multiplier into")
        self.args = (float(w[name + ".alpha"]), w[name].to(dev, BF16).contiguous(), w[name + ".b"].to(dev, BF16).contiguous())

    def project(self, x, w, h, epilogue=EPI_NONE, out=None, B=1, Lq=1, **shift):
        return ops.project_dyt(x, self.args, w, h, epilogue, out=out, B=B, Lq=Lq, **shift)


class RmsNorm:
    """RMS norm with a plain weight, of the stream kept divided by the branches' multiplier; gain: a factor on the result."""

    def __init__(self, w, name, dev, cfg, gain=1.0):
        m = cfg.residual_mult
        self.args = (w[name].to(dev, BF16).contiguous(), cfg.norm_eps / (m * m), gain if m > 0 else -gain)

    def project(self, x, w, h, epilogue=EPI_NONE, out=None, B=1, Lq=1):
        return ops.project_rms(x, self.args, w, h, epilogue, out=out)


NORMS = {"dyt": DynamicTanh, "rms": RmsNorm}


class _Layer:
    """Device weights of one layer: projections that read the same input are one matrix."""

    def __init__(self, spec, w, p, dev, cfg):
        def t(name):
            return w[p + name].to(dev, BF16).contiguous()
        ds, ones = cfg.design, torch.ones(cfg.hidden_size, dtype=BF16, device=dev)
        self.spec, self.act = spec, ACTS[ds.act]
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, w, p + "mix.", dev, cfg)
        self.norm1 = NORMS[ds.norm](w, p + "norm1", dev, cfg)
        self.shift, self.ls1 = t("shift") if ds.token_shift else None, t("ls1") if ds.layer_scale else ones
        self.mlp = spec.mlp is not None
        if self.mlp:
            self.norm2, self.ls2 = NORMS[ds.norm](w, p + "norm2", dev, cfg), t("ls2") if ds.layer_scale else ones
            self.gate_up, self.down = torch.cat([t("mlp.gate"), t("mlp.up")]).contiguous(), t("mlp.down")


class LayeredModel(DecoderModel):
    x_dtype = F32

    def __init__(self, cfg, weights, device="cuda:0"):
        self._init_decoder(cfg, device)
        self.act_dtype = F32 if cfg.dtype == "float32" else BF16
        dev, ds = self.device, cfg.design
        if cfg.state_rows < 2 or cfg.shift_rows < 2:
            raise ValueError("a step reads the row behind the last column and writes the next: at least two rows of history")
        self.embed = weights["embed"].to(dev, BF16).contiguous()
        self.head = self.embed if ds.tied_head else weights["head"].to(dev, BF16).contiguous()
        self.final_norm = NORMS[ds.norm](weights, "final.norm", dev, cfg, gain=cfg.logit_scale)
        own = {i: _Layer(s, weights, f"l{i}.", dev, cfg) for i, s in enumerate(cfg.layers) if s.owner is None}
        self.stack = [own[i if s.owner is None else s.owner] for i, s in enumerate(cfg.layers)]
        mixing = [i for i, s in enumerate(cfg.layers) if getattr(s.mixer, "v_mix", False)]
        self.first_v = mixing[0] if mixing else None             # the layer whose own values the later v_mix layers blend in
        self._tables = {}

    # ------------------------------------------------------------------ state and buffers
    def _rot_tables(self, rot, n):
        """cos and sin [>= n, dims / 2] fp32 of positions 0, 1, ..: angles in float64, rounded once."""
        got = self._tables.get(rot)
        if got is None or got[0].shape[0] < n:
            n = max(4096, 1 << (n - 1).bit_length())
            f, mult = rot.frequencies()
            a = torch.arange(n, dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
            got = self._tables[rot] = ((a.cos() * mult).to(self.device, F32).contiguous(), (a.sin() * mult).to(self.device, F32).contiguous())
        return got

    def _new_state(self, B, S, max_tokens, pids, mask, shared_tables=True):
        st = LayeredCacheState(self.cfg, B, S, max_tokens, self.device)
        for s, rows in zip(self.cfg.layers, st.mix):
            if isinstance(rows, LatentRows):
                rows.cos, rows.sin = self._rot_tables(s.mixer.rot, st.Tp + 512)
        self._states.add(st)
        if mask is not None:
            m = torch.as_tensor(mask)
            st.pad_len = (m == 0).sum(dim=1).to(torch.int32).to(self.device)
        return st

    def _cache_token_bytes(self):
        e = 4 if self.act_dtype == F32 else 2
        return sum(MIXER_ROWS[type(s.mixer)].token_bytes(s.mixer, e) for s in self.cfg.layers)

    def _alloc_bufs(self, B, L, n_keys=None):
        """n_keys: what the attention's key splits are planned for (one-token calls: the cache capacity, so that eager and captured steps
        split alike; prompts: past + L)."""
        M, dev, T, cfg = B * L, self.device, self.act_dtype, self.cfg
        n_keys = L if n_keys is None else n_keys
        mixers = [ly.mixer for ly in self.stack]
        ff = max((s.mlp.ff for s in cfg.layers if s.mlp is not None), default=0)
        need = {"h": (M * cfg.hidden_size, T), "y": (M * max(m.w_in.shape[0] for m in mixers), T), "o": (M * max(m.n_out for m in mixers), T), "a": (M * ff, T)}
        if self.first_v is not None:                             # its values stay readable through the stack
            need["y_first"] = (M * mixers[self.first_v].w_in.shape[0], T)
        for m in {id(m): m for m in mixers}.values():
            for k, (n, dt) in m.buffers(B, L, n_keys).items():
                need[k] = (max(n, need.get(k, (0, dt))[0]), dt)
        bufs = {k: torch.zeros(n, dtype=dt, device=dev) if k == "q" else torch.empty(n, dtype=dt, device=dev) for k, (n, dt) in need.items()}
        bufs["plans"] = [m.plan(B, L, n_keys) for m in mixers]
        return bufs

    # ------------------------------------------------------------------ layers
    def _embed(self, ids, out=None):
        return ops.embed_scale(ids, self.embed, self.cfg.embed_scale / self.cfg.residual_mult, out=out)

    def _head(self, x, out=None, bufs=None):
        n = x.shape[0]
        h = torch.empty(x.shape, dtype=self.act_dtype, device=x.device) if bufs is None else bufs["h"][:x.numel()].view(x.shape)
        if out is None:
            out = torch.empty((n, self.cfg.vocab_size), dtype=self.act_dtype, device=x.device)
        return self.final_norm.project(x, self.head, h, EPI_NONE, out=out, B=n)

    def _layers(self, x, st, B, L, past, n_beam, bufs=None, d_past=None, last_only=False, keep=None):
        """The stack on x fp32 [B*L, width], in place.  last_only: the last layer's residual branches run on the B last rows alone;
        returns those rows then."""
        if n_beam > 1:                                           # beams read the cache and leave it as it is
            st = st.beams(n_beam, L)
        if bufs is None:
            bufs = self._alloc_bufs(B, L, st.Tp if L == 1 else past + L)
        M, D = B * L, self.cfg.hidden_size
        call = Call(B, L, past, L if keep is None else keep, d_past, st.pad_len)
        for i, ly in enumerate(self.stack):
            mx = ly.mixer
            h, o = bufs["h"].view(M, D), bufs["o"][:M * mx.n_out].view(M, mx.n_out)
            y = bufs["y_first" if i == self.first_v else "y"][:M * mx.w_in.shape[0]].view(M, -1)
            shift = {} if ly.shift is None else dict(shift=ly.shift, hist=st.shift[i], past=past, d_past=d_past, pad_len=st.pad_len)
            ly.norm1.project(x, mx.w_in, h, out=y, B=B, Lq=L, **shift)
            mx.run(y, o, st.mix[i], bufs, call, bufs["plans"][i])
            if i == self.first_v:
                call.v_first = mx.values(y)
            rows = M
            if last_only and L > 1 and i == len(self.stack) - 1:
                o, x, rows = o.view(B, L, -1)[:, -1].contiguous(), x.view(B, L, -1)[:, -1].contiguous(), B
            ops.project(o, mx.o, EPI_SCALE_RESID_F32, resid=x, col_scale=ly.ls1, out=x)
            if ly.mlp:
                ff = ly.spec.mlp.ff
                h, a = h[:rows], bufs["a"][:rows * ff].view(rows, ff)
                ly.norm2.project(x, ly.gate_up, h, ly.act, out=a, B=rows)
                ops.project(a, ly.down, EPI_SCALE_RESID_F32, resid=x, col_scale=ly.ls2, out=x)
            if self.hidden_hook is not None:
                self.hidden_hook(i, x * self.cfg.residual_mult, B, rows // B)
        return x

    # ------------------------------------------------------------------ captured greedy step, captured prefill
    def _step_bufs(self, st):
        return self._alloc_bufs(st.B, 1, st.Tp)

    def _step(self, g, st):
        bufs = g["bufs"]
        self._embed(g["tok"], out=g["x"])
        self._layers(g["x"], st, st.B, 1, 0, 1, bufs=bufs, d_past=g["d_past"])
        self._head(g["x"], out=g["logits"], bufs=bufs)
        ops.step_end(g["logits"], g["next_tok"], g["tok"], g["history"], g["d_step"], g["d_past"], g["ticket"])

    def _prefill_key(self, S, max_tokens):
        return (S, max_tokens)
