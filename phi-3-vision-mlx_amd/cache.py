"""Cache states: what one prompt batch (or one slot group of the engine) keeps on the device between calls."""
import torch

from .config import GlaMixer, LatentMixer, Mixer, head_dim
from .ops import BF16, F32, I32


def padded_columns(T):
    """Columns a cache of T tokens is allocated with."""
    # row/column stride of the caches: whole 128-key tiles (the decode attention takes one 128-key tile per workgroup
    # when the capacity allows it)
    gran = 128
    Tp = (T + gran - 1) // gran * gran
    if (Tp // gran) % 2 == 0:
        # V^T rows are Tp * 2 bytes apart: at multiples of 512 B the 96 rows of a tile crowd the same memory channels
        # (measured decode step at B = 1: +3.5 % at Tp = 2560, +2 % at 3584, +1.4 % at 4096, +5.7 % at 33024 = 258 tiles
        # against the neighbouring lengths) -- an ODD number of 128-key tiles keeps the stride off that grid
        Tp += gran
    return Tp


class CacheState:
    """All layers' KV cache + per-prompt RoPE tables / pad lengths.

    Mirrors reference KVCache (phi.py:509-548) semantics: `offset` auto-advances
    by L, can be rewound (`advance_offset`), `max_tokens < 1` disables caching,
    `n_beam > 1` reads the cache without writing it."""

    def __init__(self, cfg, B, S, max_tokens, device):
        self.B, self.S, self.max_tokens = B, S, max_tokens
        self.T = S + max(max_tokens, 0)
        self.quantized = bool(getattr(cfg, "use_quantized_cache", False))
        # cache_format="mlx4" (opt-in): the reference's OWN quantised cache -- MLX 4-bit group-32 codes of the PROMPT's K / V, later
        # tokens unquantised (phi.py:528-540).  The codes are kept in the reference's format (k4 / v4 + scale | bias), and the
        # bf16 cache rows hold their dequantised values, which is what every later call of the reference attends on: the decode
        # path is then the plain bf16 one.  (Default for quantize_cache=True: int8 for all tokens, BASELINE config 5.)
        self.mlx4 = self.quantized and getattr(cfg, "cache_format", "int8") == "mlx4"
        if self.quantized and getattr(cfg, "cache_format", "int8") not in ("int8", "mlx4"):
            raise ValueError(f"cache_format must be 'int8' or 'mlx4', got {cfg.cache_format!r}")
        if self.mlx4:
            self.quantized = False
        self.Tp = padded_columns(self.T)
        nl, nkv, hd = cfg.num_hidden_layers, cfg.num_key_value_heads, head_dim(cfg)
        if self.quantized:
            # int8 KV (quantize_cache=True): offset-binary bytes + one fp32 scale per (layer, row, head, token);
            # one bf16 K / V^T scratch layer holds the exact prompt keys while a layer's prefill attends (phi.py:531-533)
            self.k8 = torch.full((nl, B, nkv, self.Tp, hd), 128, dtype=torch.uint8, device=device)
            self.v8 = torch.full((nl, B, nkv, hd, self.Tp), 128, dtype=torch.uint8, device=device)
            self.ks = torch.ones((nl, B, nkv, self.Tp), dtype=F32, device=device)
            self.vs = torch.ones((nl, B, nkv, self.Tp), dtype=F32, device=device)
            self.k_tmp = torch.empty((B, nkv, self.Tp, hd), dtype=BF16, device=device)
            self.v_tmp = torch.zeros((B, nkv, hd, self.Tp), dtype=BF16, device=device)
        else:
            self.k = torch.empty((nl, B, nkv, self.Tp, hd), dtype=BF16, device=device)    # K   [.., t, hd]
            self.v = torch.zeros((nl, B, nkv, hd, self.Tp), dtype=BF16, device=device)    # V^T [.., hd, t] (zero: tail keys stay finite)
        if self.mlx4:
            g = hd // 32
            self.k4 = torch.zeros((nl, B, nkv, max(S, 1), g, 4), dtype=I32, device=device)
            self.v4 = torch.zeros_like(self.k4)
            self.k_sb = torch.zeros((nl, B, nkv, max(S, 1), g, 2), dtype=F32, device=device)
            self.v_sb = torch.zeros_like(self.k_sb)
            self.mlx4_tokens = 0                                # prompt tokens held as codes (set by the first call)
        self._loop_state()
        self.cos = self.sin = None

    def _loop_state(self):
        self.offset = 0
        self.pad_len = None
        self.graphs = {}
        self.epoch = None                                       # model.epoch the graphs were captured under
        self.shared = {"dirty": False}                          # shared by the per-request views of a captured-prefill entry (copy.copy)

    def mark_dirty(self):
        """An unrecovered failed step may have left NaN rows beyond the offset and half-armed buffers in the decode graph: a
        captured-prefill entry built on these buffers must not be reused (model._prefill_captured drops it)."""
        self.shared["dirty"] = True

    def note_written(self, lo, hi, kept=None):
        """A call is about to write columns [lo, hi), of which [lo, kept) stay (None: all): states that keep a bounded history beside the
        cache check and record it."""

    def row_view(self, rows, S, offset, epoch):
        """Batch rows `rows` (a slice) as a state of their own over the same memory, at cache column `offset`, for the prefill of
        prompts of S tokens: columns left of `offset` hold nothing these rows may see (pad_len >= offset)."""
        view = type(self).__new__(type(self))
        view.__dict__.update(B=rows.stop - rows.start, S=S, max_tokens=self.max_tokens, T=self.T, Tp=self.Tp, quantized=self.quantized,
                             offset=offset, graphs={}, epoch=epoch, pad_len=self.pad_len[rows], fresh_rows=True)
        self._view_rows(view, rows)
        return view

    def _view_rows(self, view, rows):
        view.__dict__.update(cos=self.cos[rows], sin=self.sin[rows])
        if self.quantized:
            view.__dict__.update(k8=self.k8[:, rows], v8=self.v8[:, rows], ks=self.ks[:, rows], vs=self.vs[:, rows],
                                 k_tmp=self.k_tmp[rows], v_tmp=self.v_tmp[rows])
        else:
            view.__dict__.update(k=self.k[:, rows], v=self.v[:, rows])

    def scrub(self, lo, hi):
        """Forget cache positions [lo, hi) that a FAILED step wrote (api.greedy_loop's recovery): a poisoned step leaves NaN there,
        and the decode attention multiplies every V^T column of a tile -- live or not -- by its (zero) probability."""
        hi = min(hi, self.Tp)
        if hi <= lo:
            return
        if self.quantized:
            self.v8[..., lo:hi] = 128
            self.k8[:, :, :, lo:hi] = 128
            self.vs[..., lo:hi] = 1.0
            self.ks[..., lo:hi] = 1.0
        else:
            self.v[..., lo:hi] = 0
            self.k[:, :, :, lo:hi] = 0


class LayerCache:
    """`cache[i]` view with the reference's `.offset` attribute."""

    def __init__(self, state, i):
        self.state, self.i = state, i

    @property
    def offset(self):
        return self.state.offset

    @offset.setter
    def offset(self, v):
        self.state.offset = int(v)


def round_up(n, m):
    return (n + m - 1) // m * m


class KVRows:
    """Keys and values of one attention layer: k [B, G, Tp, dimp], v [B, G, Tp / 16, vdimp, 16], the widths rounded up to 32 with zeros."""
    recurrent = False

    def __init__(self, m, B, Tp, R, dt, device):
        self.k = torch.zeros((B, m.kv_heads, Tp, round_up(m.dim, 32)), dtype=dt, device=device)
        self.v = torch.zeros((B, m.kv_heads, Tp // 16, round_up(m.vdim, 32), 16), dtype=dt, device=device)

    @staticmethod
    def token_bytes(m, e):
        return e * m.kv_heads * (round_up(m.dim, 32) + round_up(m.vdim, 32))

    def rows(self, sel):
        return self._of(k=self.k[sel], v=self.v[sel])

    def beams(self, n, Tp):
        return self._of(k=_repeat(self.k, n, 2, Tp), v=_repeat(self.v, n, 2, Tp // 16))

    def scrub(self, lo, hi):
        self.k[:, :, lo:hi] = 0
        for c in range(lo, hi):
            self.v[:, :, c // 16, :, c % 16] = 0

    def _of(self, **kw):
        new = type(self).__new__(type(self))
        new.__dict__.update(kw)
        return new


class LatentRows(KVRows):
    """Latent attention's cache: c [B, Tp, rankp + rotp], a row = the normed latent (rank, zeros up to a multiple of 64), then the
    rotated key part all heads share (zeros up to a multiple of 32)."""

    def __init__(self, m, B, Tp, R, dt, device):
        self.c = torch.zeros((B, Tp, latent_width(m)), dtype=dt, device=device)
        self.cos = self.sin = None                               # rotation tables [>= Tp, rot / 2] fp32 by position (the model sets them)

    @staticmethod
    def token_bytes(m, e):
        return e * latent_width(m)

    def rows(self, sel):
        return self._of(c=self.c[sel], cos=self.cos, sin=self.sin)

    def beams(self, n, Tp):
        return self._of(c=_repeat(self.c, n, 1, Tp), cos=self.cos, sin=self.sin)

    def scrub(self, lo, hi):
        self.c[:, lo:hi] = 0


class RecurrentRows(KVRows):
    """A recurrent layer's states: s [B, R, H, dim, vdim] fp32, the state behind t columns in slot t % R."""
    recurrent = True

    def __init__(self, m, B, Tp, R, dt, device):
        self.s = torch.zeros((B, R, m.heads, m.dim, m.vdim), dtype=F32, device=device)

    @staticmethod
    def token_bytes(m, e):
        return 0

    def rows(self, sel):
        return self._of(s=self.s[sel])

    def beams(self, n, Tp):
        return self._of(s=self.s.repeat_interleave(n, dim=0))

    def scrub(self, lo, hi):
        pass                                                     # (a step replaces the whole state, out of the slot before)


MIXER_ROWS = {Mixer: KVRows, LatentMixer: LatentRows, GlaMixer: RecurrentRows}


def latent_width(m):
    return round_up(m.rank, 64) + round_up(m.rot.dims, 32)


def _repeat(t, n, dim, cols):
    out = torch.zeros((t.shape[0] * n,) + t.shape[1:dim] + (cols,) + t.shape[dim + 1:], dtype=t.dtype, device=t.device)
    src = min(cols, t.shape[dim])
    out.narrow(dim, 0, src).copy_(t.narrow(dim, 0, src).repeat_interleave(n, dim=0))
    return out


class LayeredCacheState(CacheState):
    """State of a layered decoder (config.LayerSpec): per layer what its mixer keeps (mix[i], also of a layer that uses another one's
    weights), and with a token shift

        shift[i] [B, R, width] fp32           the mixer's unshifted inputs of the last R columns (column c in row c % R)

    A cache is rewound by lowering `offset`.  The token shift then needs the input of the token before, so the state keeps a ring of
    shift_rows of them: a rewind of up to that many less one is exact.  A recurrent layer needs the state itself; the ring of state_rows
    of them holds those behind the last calls (`held`).  Any other rewind raises."""

    def __init__(self, cfg, B, S, max_tokens, device):
        self.B, self.S, self.max_tokens = B, S, max_tokens
        self.T = S + max(max_tokens, 0)
        self.quantized = False
        self.Tp = padded_columns(self.T)
        self.R, self.state_rows = cfg.shift_rows, cfg.state_rows
        self.hist_max, self.held = 0, frozenset()
        dt = F32 if cfg.dtype == "float32" else BF16
        self.mix = [MIXER_ROWS[type(ly.mixer)](ly.mixer, B, self.Tp, self.state_rows, dt, device) for ly in cfg.layers]
        self.shift = [torch.zeros((B, self.R, cfg.hidden_size), dtype=F32, device=device) if cfg.design.token_shift else None for _ in cfg.layers]
        self._loop_state()

    @property
    def k(self):
        return [getattr(m, "k", None) for m in self.mix]

    @property
    def v(self):
        return [getattr(m, "v", None) for m in self.mix]

    @property
    def recurrent(self):
        return any(m.recurrent for m in self.mix)

    def note_written(self, lo, hi, kept=None):
        """Columns [lo, hi) are about to be written, [lo, kept) of them to stay (None: all)."""
        kept = hi if kept is None else kept
        if getattr(self, "slots", False) or getattr(self, "fresh_rows", False):
            return                                              # (every row's history is rewritten by its own prefill)
        if self.recurrent and not lo <= kept <= hi:
            raise ValueError(f"columns [{lo}, {hi}) of which {kept - lo} stay: a recurrent state cannot follow")
        if lo == 0:
            self.hist_max, self.held = 0, frozenset((0,))
        elif self.recurrent and lo not in self.held:
            raise ValueError(f"cache rewound to {lo}: the recurrent states held are those behind {sorted(self.held)} columns")
        elif self.shift[0] is not None and lo <= self.hist_max - self.R:
            raise ValueError(f"cache rewound to {lo}: the token-shift history holds the last {self.R} of {self.hist_max} columns")
        self.hist_max = max(self.hist_max, hi)
        if kept > lo:
            self.held = frozenset(t for t in self.held if t <= lo and (t - kept) % self.state_rows) | {kept}

    def _view_rows(self, view, rows):
        view.__dict__.update(mix=[m.rows(rows) for m in self.mix], shift=[None if t is None else t[rows] for t in self.shift], R=self.R,
                             state_rows=self.state_rows, hist_max=0, held=frozenset())

    def beams(self, n, L):
        """A scratch copy with every row repeated n times and room for L more columns (beam calls read the cache, never write it)."""
        view = type(self).__new__(type(self))
        Tp = round_up(self.offset + L, 64)
        view.__dict__.update(B=self.B * n, S=self.S, max_tokens=self.max_tokens, T=Tp, Tp=Tp, quantized=False, offset=self.offset, graphs={},
                             epoch=self.epoch, R=self.R, state_rows=self.state_rows, hist_max=self.hist_max, held=self.held, fresh_rows=True,
                             pad_len=None if self.pad_len is None else self.pad_len.repeat_interleave(n),
                             mix=[m.beams(n, Tp) for m in self.mix],
                             shift=[None if t is None else t.repeat_interleave(n, dim=0) for t in self.shift])
        return view

    def scrub(self, lo, hi):
        hi = min(hi, self.Tp)
        for m, h in zip(self.mix, self.shift):
            m.scrub(lo, hi)
            if h is not None:
                for c in range(lo, hi):
                    h[:, c % self.R] = 0
