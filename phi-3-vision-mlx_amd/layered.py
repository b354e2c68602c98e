"""Layered text decoders on MI355X: a decoder whose layers are described one by one in its config (config.LayerSpec), built from
mechanisms that take their constants as parameters.  Served through the same contract as the other models (decoder.DecoderModel):
`model(...)`, the captured greedy step, slot states of the engine.

Per layer, on a fp32 residual stream x:

    h  = token_shift(dyt(x))                      ops.dyt
    q | k | v | gate logits = W h                 one projection, weights packed at load
    o  = mixed-head attention                     ops.attention_mixed (norms, value mixing, append, sink, output gate)
    x += ls1 * (W_o o)                            projection epilogue
    a  = silu(W_gate h2) * (W_up h2), h2 = dyt(x) ops.dyt + projection epilogue
    x += ls2 * (W_down a)                         projection epilogue

Activations are bf16, or fp32 throughout with dtype="float32" (weights stay bf16 data, which fp32 arithmetic reads exactly).
"""
import torch

from . import ops
from .cache import LayeredCacheState, round_up
from .decoder import DecoderModel, on_device
from .ops import BF16, EPI_NONE, EPI_SCALE_RESID_F32, EPI_SILU_MUL, F32


class _Layer:
    """Device weights of one layer: projections that read the same input are one matrix."""

    def __init__(self, spec, w, p, dev):
        def t(name):
            return w[p + name].to(dev, BF16).contiguous()
        self.spec, m = spec, spec.mixer
        self.norm1 = (float(w[p + "norm1.alpha"]), t("norm1"), t("norm1.b"))
        self.shift, self.ls1 = t("shift"), t("ls1")
        qkvg = torch.cat([t("mix.q"), t("mix.k"), t("mix.v"), t("mix.g")])
        # whole GEMM tiles (the 256-column ones where the matrix is wide): the padding rows are zero and nobody reads their outputs
        n = round_up(qkvg.shape[0], 256 if qkvg.shape[0] >= 2048 else 64)
        self.qkvg = torch.cat([qkvg, qkvg.new_zeros((n - qkvg.shape[0], qkvg.shape[1]))]).contiguous()
        self.norms = (t("mix.q.norm"), t("mix.k.norm"))
        self.talk, self.sink, self.vmix, self.o = t("mix.talk"), t("mix.sink"), float(w[p + "mix.vmix"]) if p + "mix.vmix" in w else 0.0, t("mix.o")
        self.v_col = (m.heads + m.kv_heads) * m.dim              # first value column of the packed projection
        self.mlp = spec.mlp is not None
        if self.mlp:
            self.norm2, self.ls2 = (float(w[p + "norm2.alpha"]), t("norm2"), t("norm2.b")), t("ls2")
            self.gate_up, self.down = torch.cat([t("mlp.gate"), t("mlp.up")]).contiguous(), t("mlp.down")


class LayeredModel(DecoderModel):
    x_dtype = F32

    def __init__(self, cfg, weights, device="cuda:0"):
        self._init_decoder(cfg, device)
        self.act_dtype = F32 if cfg.dtype == "float32" else BF16
        dev = self.device
        self.embed, self.head = weights["embed"].to(dev, BF16).contiguous(), weights["head"].to(dev, BF16).contiguous()
        self.final_norm = (float(weights["final.norm.alpha"]), weights["final.norm"].to(dev, BF16).contiguous(),
                           weights["final.norm.b"].to(dev, BF16).contiguous())
        self.stack = [_Layer(s, weights, f"l{i}.", dev) for i, s in enumerate(cfg.layers)]
        mixing = [i for i, s in enumerate(cfg.layers) if s.mixer.v_mix]
        self.first_v = mixing[0] if mixing else None             # the layer whose own values the later v_mix layers blend in

    # ------------------------------------------------------------------ state and buffers
    def _new_state(self, B, S, max_tokens, pids, mask, shared_tables=True):
        st = LayeredCacheState(self.cfg, B, S, max_tokens, self.device)
        self._states.add(st)
        if mask is not None:
            m = torch.as_tensor(mask)
            st.pad_len = (m == 0).sum(dim=1).to(torch.int32).to(self.device)
        return st

    def _cache_token_bytes(self):
        e = 4 if self.act_dtype == F32 else 2
        return sum(e * s.mixer.kv_heads * (round_up(s.mixer.dim, 32) + round_up(s.mixer.vdim, 32)) for s in self.cfg.layers)

    def _alloc_bufs(self, B, L, n_keys=None):
        """n_keys: what the attention's key splits are planned for (one-token calls: the cache capacity, so that eager and captured steps
        split alike; prompts: past + L)."""
        M, dev, T, cfg = B * L, self.device, self.act_dtype, self.cfg
        n_keys = L if n_keys is None else n_keys
        ms = [s.mixer for s in cfg.layers]

        def plan(m):
            return ops.mix_plan(B, L, m.heads, m.kv_heads, m.dim, m.vdim, n_keys, T)
        ws = max(ops.mix_ws_bytes(B, L, m.heads, m.vdim, plan(m)) for m in ms)
        ff = max((s.mlp.ff for s in cfg.layers if s.mlp is not None), default=0)
        bufs = dict(h=torch.empty((M, cfg.hidden_size), dtype=T, device=dev),
                    qkv=torch.empty(M * max(ly.qkvg.shape[0] for ly in self.stack), dtype=T, device=dev),
                    q=torch.zeros(M * max(m.heads * round_up(m.dim, 32) for m in ms), dtype=T, device=dev),
                    o=torch.empty(M * max(m.heads * m.vdim for m in ms), dtype=T, device=dev), a=torch.empty(M * ff, dtype=T, device=dev),
                    mix_ws=torch.empty(ws // 4, dtype=F32, device=dev) if ws else None, n_split=[plan(m) for m in ms])
        if self.first_v is not None:                             # its values stay readable through the stack
            bufs["qkv_first"] = torch.empty((M, self.stack[self.first_v].qkvg.shape[0]), dtype=T, device=dev)
        return bufs

    # ------------------------------------------------------------------ layers
    def _embed(self, ids, out=None):
        return ops.embed_scale(ids, self.embed, self.cfg.embed_scale, out=out)

    def _head(self, x, out=None, bufs=None):
        h = bufs["h"][:x.shape[0]] if bufs is not None else torch.empty(x.shape, dtype=self.act_dtype, device=x.device)
        if out is None:
            out = torch.empty((x.shape[0], self.cfg.vocab_size), dtype=self.act_dtype, device=x.device)
        return ops.project_dyt(x, self.final_norm, self.head, h, EPI_NONE, out=out, B=x.shape[0])

    def _layers(self, x, st, B, L, past, n_beam, bufs=None, d_past=None, last_only=False):
        """The stack on x fp32 [B*L, width], in place.  last_only: the last layer's residual branches run on the B last rows alone;
        returns those rows then."""
        if n_beam > 1:                                           # beams read the cache and leave it as it is
            st = st.beams(n_beam, L)
        if bufs is None:
            bufs = self._alloc_bufs(B, L, st.Tp if L == 1 else past + L)
        M, eps = B * L, self.cfg.norm_eps
        v_first = None
        for i, ly in enumerate(self.stack):
            m = ly.spec.mixer
            n_o = m.heads * m.vdim
            h, o = bufs["h"], bufs["o"][:M * n_o].view(M, n_o)
            qkv = bufs["qkv_first"] if i == self.first_v else bufs["qkv"][:M * ly.qkvg.shape[0]].view(M, -1)
            ops.project_dyt(x, ly.norm1, ly.qkvg, h, out=qkv, B=B, Lq=L, shift=ly.shift, hist=st.shift[i], past=past, d_past=d_past,
                            pad_len=st.pad_len)
            ops.attention_mixed(qkv, bufs["q"], st.k[i], st.v[i], o, ly.norms, ly.talk, ly.sink, B, L, m.heads, m.kv_heads, m.dim, m.vdim, eps,
                                m.scale, past, v_first=v_first if m.v_mix else None, vmix=ly.vmix, pad_len=st.pad_len, d_past=d_past,
                                ws=bufs["mix_ws"], n_split=bufs["n_split"][i])
            if i == self.first_v:
                v_first = qkv[:, ly.v_col:ly.v_col + m.kv_heads * m.vdim]
            rows = M
            if last_only and L > 1 and i == len(self.stack) - 1:
                o, x, rows = o.view(B, L, -1)[:, -1].contiguous(), x.view(B, L, -1)[:, -1].contiguous(), B
            ops.project(o, ly.o, EPI_SCALE_RESID_F32, resid=x, col_scale=ly.ls1, out=x)
            if ly.mlp:
                ff = ly.spec.mlp.ff
                h, a = h[:rows], bufs["a"][:rows * ff].view(rows, ff)
                ops.project_dyt(x, ly.norm2, ly.gate_up, h, EPI_SILU_MUL, out=a, B=rows)
                ops.project(a, ly.down, EPI_SCALE_RESID_F32, resid=x, col_scale=ly.ls2, out=x)
            if self.hidden_hook is not None:
                self.hidden_hook(i, x, B, rows // B)
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
