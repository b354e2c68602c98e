"""The mixers of the layered decoders: what a layer does between its norm and its output projection.

A mixer holds the device weights of one layer that has them (another layer may use the same object) and takes the rows of ONE packed
projection of the layer's input:

    w_in                     the packed projection; its rows are padded with zeros to whole GEMM tiles
    n_out, o                 columns of the mixer's output, the output projection
    buffers(B, L, n_keys)    {name: (elements, dtype)} of scratch; layers share a buffer of the largest size
    plan(B, L, n_keys)       what a call's launches are planned for (a one-token call: the cache capacity, so that eager and captured
                             steps run alike)
    run(y, out, rows, bufs, call, plan)
"""
from dataclasses import dataclass
from typing import Any

import torch

from . import ops
from .cache import latent_width, round_up
from .config import GlaMixer, LatentMixer, Mixer
from .ops import BF16, F32


@dataclass
class Call:
    """One call of the stack: B rows of L new tokens behind `past` columns (d_past: the same from device memory), of which `keep` stay."""
    B: int
    L: int
    past: int
    keep: int
    d_past: Any = None
    pad_len: Any = None
    v_first: Any = None


def packed(mats):
    """Matrices that read the same input as one, in whole GEMM tiles (the 256-column ones where it is wide): the padding rows are zero
    and nobody reads their outputs."""
    w = torch.cat(mats)
    n = round_up(w.shape[0], 256 if w.shape[0] >= 2048 else 64)
    return torch.cat([w, w.new_zeros((n - w.shape[0], w.shape[1]))]).contiguous()


class MixedHeads:
    """Attention whose heads' scores are mixed before the softmax (config.Mixer)."""

    def __init__(self, m, w, p, dev, cfg):
        def t(name):
            return w[p + name].to(dev, BF16).contiguous()
        self.m, self.eps, self.T = m, cfg.norm_eps, F32 if cfg.dtype == "float32" else BF16
        self.w_in, self.o, self.n_out = packed([t("q"), t("k"), t("v"), t("g")]), t("o"), m.heads * m.vdim
        self.norms = (t("q.norm"), t("k.norm"))
        self.talk, self.sink, self.vmix = t("talk"), t("sink"), float(w[p + "vmix"]) if p + "vmix" in w else 0.0
        self.v_col = (m.heads + m.kv_heads) * m.dim              # first value column of the packed projection

    def plan(self, B, L, n_keys):
        m = self.m
        return ops.mix_plan(B, L, m.heads, m.kv_heads, m.dim, m.vdim, n_keys, self.T)

    def buffers(self, B, L, n_keys):
        m = self.m
        return {"q": (B * L * m.heads * round_up(m.dim, 32), self.T),
                "attn_ws": (ops.mix_ws_bytes(B, L, m.heads, m.vdim, self.plan(B, L, n_keys)) // 4, F32)}

    def run(self, y, out, rows, bufs, call, plan):
        m = self.m
        ops.attention_mixed(y, bufs["q"], rows.k, rows.v, out, self.norms, self.talk, self.sink, call.B, call.L, m.heads, m.kv_heads, m.dim, m.vdim,
                            self.eps, m.scale, call.past, v_first=call.v_first if m.v_mix else None, vmix=self.vmix, pad_len=call.pad_len,
                            d_past=call.d_past, ws=bufs["attn_ws"], n_split=plan)

    def values(self, y):
        return y[:, self.v_col:self.v_col + self.m.kv_heads * self.m.vdim]


class LatentHeads:
    """Latent attention (config.LatentMixer).  A few new tokens attend in the latent space: the up-projections of keys and values are
    applied to the query and to the attended latent.  A prompt expands keys and values of all its columns once and attends over those."""

    def __init__(self, m, w, p, dev, cfg):
        def t(name):
            return w[p + name].to(dev, BF16)
        self.m, self.eps, self.T = m, cfg.norm_eps, F32 if cfg.dtype == "float32" else BF16
        self.w_in, self.o, self.n_out = packed([t("q"), t("dkv"), t("g")]), t("o").contiguous(), m.heads * m.vdim
        self.c_norm, self.sink = t("dkv.norm").contiguous(), t("sink").contiguous()
        rankp, dimp = round_up(m.rank, 64), round_up(m.dim, 32)

        def wide(a):                                             # the latent's padding meets zeros
            return torch.nn.functional.pad(a, (0, rankp - m.rank)).contiguous()
        self.uk, self.uv = wide(t("uk")), wide(t("uv"))
        ukt = self.uk.view(m.heads, m.dim, rankp).transpose(1, 2)
        self.ukt = torch.nn.functional.pad(ukt, (0, dimp - m.dim)).contiguous()

    def plan(self, B, L, n_keys):
        return ops.latent_plan(self.m, B, L, n_keys, self.T)

    def buffers(self, B, L, n_keys):
        m, plan = self.m, self.plan(B, L, n_keys)
        if plan > 0:                                             # in the latent space, keys split `plan` ways
            hp = round_up(m.heads, 16)
            return {"q": (B * L * hp * latent_width(m), self.T), "attn_ws": (ops.latent_ws_bytes(m, B, L, plan) // 4, F32)}
        if plan < 0:                                             # expanded
            n = round_up(n_keys, 64)
            return {"kx": (B * n * m.heads * m.dim, self.T), "vx": (B * n * m.heads * m.vdim, self.T)}
        return {}

    def run(self, y, out, rows, bufs, call, plan):
        ops.attention_latent(self, y, out, rows.c, rows.cos, rows.sin, bufs, call, plan)


class LinearState:
    """Gated linear attention (config.GlaMixer)."""

    def __init__(self, m, w, p, dev, cfg):
        def t(name):
            return w[p + name].to(dev, BF16).contiguous()
        self.m, self.eps, self.T = m, cfg.norm_eps, F32 if cfg.dtype == "float32" else BF16
        self.w_in, self.o, self.n_out = packed([t("q"), t("k"), t("v"), t("g"), t("a1")]), t("o"), m.heads * m.vdim
        self.a2, self.a2_b, self.norm = t("a2"), t("a2.b"), t("norm")
        self.rank = self.a2.shape[1]
        if w[p + "a1"].shape[0] != self.rank:
            raise ValueError(f"{p}a1 has {w[p + 'a1'].shape[0]} rows, {p}a2 {self.rank} columns")

    def plan(self, B, L, n_keys):
        return ops.gla_plan(self.m, B, L, self.T)

    def buffers(self, B, L, n_keys):
        return {"gla_ws": (ops.gla_ws_bytes(self.m, B, L, self.plan(B, L, n_keys)) // 4, F32)}

    def run(self, y, out, rows, bufs, call, plan):
        ops.gated_linear_attention(self, y, out, rows.s, bufs.get("gla_ws"), call, plan)


MIXERS = {Mixer: MixedHeads, LatentMixer: LatentHeads, GlaMixer: LinearState}
