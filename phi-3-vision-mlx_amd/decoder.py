"""What every decoder of the framework shares: the call contract, the slot states of the engine, the captured greedy step and the
captured short-prompt prefill.  A model class (model.Phi3VModel, layered.LayeredModel) supplies the layers:

    x_dtype, act_dtype                       residual stream / logits
    _new_state(B, S, max_tokens, pids, mask) a CacheState
    _slot_rows(st, row, lens)                per-row tables of a slot prefill (none by default)
    _alloc_bufs(B, L), _step_bufs(st)        activations of one call / of the captured step
    _embed(ids, out=None), _layers(...), _head(x, out=None, bufs=None)    (_layers' keep: how many of the L columns stay)
    _step(g, st)                             the launches of one captured greedy step
    _prefill_key(S, max_tokens), _cache_token_bytes()   what a captured prefill depends on (None: not capturable), its cache size
"""
import copy
import functools
import os
import weakref

import numpy as np
import torch

from . import ops
from .cache import LayerCache
from .ops import BF16, F32, I32


def on_device(fn):
    """Run a model entry point with the model's GPU as the current device: ops.py launches on
    `torch.cuda.current_stream()` of the CURRENT device, and a thread other than the one that loaded the model (the
    server's engine thread) starts on device 0."""
    @functools.wraps(fn)
    def wrapped(self, *a, **kw):
        with torch.cuda.device(self.device):
            return fn(self, *a, **kw)
    return wrapped


class DecoderModel:
    x_dtype = act_dtype = BF16
    vision = False
    rope_regimes = False                             # does a call's length pick one of two position tables (engine.py)?

    def _init_decoder(self, cfg, device):
        if not torch.cuda.is_available():
            raise RuntimeError(f"{type(self).__name__} needs a GPU: the hot path is HIP-only (no CPU fallback)")
        ops.L.lib()                                  # fail loudly if the library is missing
        self.cfg, self.device = cfg, torch.device(device)
        self.hidden_hook = None                      # fn(layer, x [B*L, H], B, L) after every decoder layer (diagnostics)
        # A long-lived owner that may share the GPU with other streams / processes (server.py) sets this: the decode step then
        # uses no launch that needs all of its workgroups resident at once.  One-shot generate() on an exclusive GPU keeps them.
        self.serving = os.environ.get("P3V_SHARED_GPU", "0") == "1"
        self.epoch = 0                               # bumped whenever captured decode graphs become stale
        self._prefill_graphs = {}                    # (S, max_tokens, ..) -> captured short-prompt prefill (see _prefill_captured)
        self._prefill_seen = {}
        self._states = weakref.WeakSet()             # every live CacheState (their graphs bake pointers into this model)

    def _slot_rows(self, st, row, lens):
        pass

    # ------------------------------------------------------------------ slot state of the continuous-batching engine
    @on_device
    def new_slot_state(self, slots, window):
        """A cache of `slots` batch rows and `window` columns that is not tied to one prompt batch (engine.py): every row
        has its OWN left padding and position table, so a request can be prefilled into a free row while the other rows
        are mid-generation.  All rows start empty (pad_len = window: every key masked).  The window fixes the RoPE regime
        of every row (phi.py:492: one choice per call from prompt + max_tokens): window <= 4096 -> short factors, beyond
        -> long factors; the engine admits only requests that would pick the same factors alone.  With
        `quantize_cache=True` the rows keep the int8 KV cache."""
        st = self._new_state(slots, 0, window, None, None, shared_tables=False)
        st.pad_len = torch.full((slots,), window, dtype=I32, device=self.device)
        st.slots = True
        return st

    @on_device
    def prefill_slot(self, st, row, inputs, return_logits=False):
        """Prefill one request (a B = 1 `processor(...)` result) -- or n requests as one batch (`collate_requests` of them:
        equal lengths, or shorter rows left-padded inside the group) -- into the batch rows row .. row+n-1 of a slot state so
        that every row's LAST prompt token sits in column st.offset - 1: row i gets left padding pad_i = st.offset - S_i and
        position ids 0..S_i-1 from column pad_i on.  Keys left of pad_i (stale rows of an earlier occupant, the group's own
        padding) are masked by pad_len.  Returns the first greedy tokens (int32 [n, 1] on the device; with return_logits also
        the last-position logits).  Each row computes what a B = 1 run of its request computes (pad invariance)."""
        ids = np.asarray(inputs["input_ids"])
        ids = ids[None] if ids.ndim == 1 else ids
        n, S = ids.shape
        lens = np.full(n, S, dtype=np.int64)
        if "mask" in inputs:
            m = np.asarray(inputs["mask"]).reshape(n, S)
            lens = m.sum(1).astype(np.int64)
            if not all(int(m[i, S - lens[i]:].sum()) == lens[i] for i in range(n)) or lens.min() < 1:
                raise ValueError("prefill_slot takes LEFT-padded rows")
        win = st.offset - S                                      # first column the group's batch writes
        if win < 0:
            raise ValueError(f"prompt of {S} tokens does not fit left of column {st.offset}")
        pads = torch.as_tensor(st.offset - lens, dtype=torch.int32)
        rows = slice(row, row + n)
        self._slot_rows(st, row, lens)
        st.pad_len[rows].copy_(pads.to(self.device))
        view = st.row_view(rows, S, win, self.epoch)            # these rows as an n-row cache at offset `win`
        kw = {k: v for k, v in inputs.items() if k in ("pixel_values", "image_sizes", "positions")}
        logits, _ = self(input_ids=ids, cache=[LayerCache(view, i) for i in range(self.cfg.num_hidden_layers)], full_logits=False, **kw)
        assert view.offset == st.offset
        tok = ops.argmax(logits[:, -1, :].contiguous())[:, None]
        return (tok, logits) if return_logits else tok

    @on_device
    def decode_graph(self, st):
        """The captured greedy step of a state (built on first use): its `tok` / `next_tok` / `d_past` device buffers."""
        if st.epoch != self.epoch:
            st.graphs.clear()
            st.epoch = self.epoch
        g = st.graphs.get("greedy")
        if g is None:
            g = st.graphs["greedy"] = self._build_decode_graph(st)
            g["host_tok"] = None
        return g

    # ------------------------------------------------------------------ graph-replayed greedy decode step
    def _build_decode_graph(self, st):
        """Capture ONE greedy decode step (embed -> 32 layers -> norm+lm_head -> argmax ->
        bookkeeping) as a hipGraph.  All loop state lives in HBM: `tok` (next input ids),
        `d_past` (cache length), `d_step`, `history` -- so replays need no host input and
        a token costs one graph launch instead of ~170 kernel launches."""
        cfg, B, dev = self.cfg, st.B, self.device
        g = dict(tok=torch.zeros((B,), dtype=I32, device=dev), d_past=torch.zeros((1,), dtype=I32, device=dev),
                 d_step=torch.zeros((1,), dtype=I32, device=dev),
                 # the step's tokens land in PINNED HOST memory straight from `k_step_end` (one 4-byte store per row and step):
                 # the host loop reads them after the step's event, no D2H copy node sits between two replays (api.greedy_loop)
                 history=torch.zeros((B, max(1, st.max_tokens) + 1), dtype=I32).pin_memory(),
                 x=torch.empty((B, cfg.hidden_size), dtype=self.x_dtype, device=dev),
                 logits=torch.empty((B, cfg.vocab_size), dtype=self.act_dtype, device=dev),
                 next_tok=torch.zeros((B,), dtype=I32, device=dev), ticket=torch.zeros((1,), dtype=I32, device=dev))
        bufs = self._step_bufs(st)
        g["bufs"] = bufs

        g["amax_ws"] = torch.zeros((ops.L.GEMV_STEP_WS_BYTES // 4,), dtype=F32, device=dev)   # (its arrival counters start at zero)

        def step():
            self._step(g, st)
        g["d_past"].fill_(st.offset)
        g["gemm_ws"] = {}                                        # B > 16 rows: the projections are split-K GEMMs; their workspace
        with ops.owned_gemm_workspace(g["gemm_ws"], frozen=False):   # belongs to the graph (sized here, baked in below)
            step()                                               # warm-up run (sets func attributes, pages code in)
        torch.cuda.synchronize()
        graph = ops.Graph()
        side = torch.cuda.Stream(device=dev)
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side), ops.owned_gemm_workspace(g["gemm_ws"], frozen=True):
            graph.begin()
            step()
            graph.end()
        torch.cuda.current_stream().wait_stream(side)
        g["d_step"].zero_()                                      # the warm-up run above counted as a step
        g["graph"] = graph
        return g

    @on_device
    def greedy_prefill(self, max_tokens, **inputs):
        """Prefill + first greedy token: `logits, cache = model(**inputs, max_tokens); argmax(logits[:, -1])`
        (reference phi_3_vision_mlx.py:385-386).  Returns (token [B,1] int32 on the device, cache)."""
        logits, cache = self(**inputs, max_tokens=max_tokens)
        return ops.argmax(logits[:, -1, :].contiguous())[:, None], cache

    @on_device
    def greedy_step(self, token, cache):
        """One greedy decode step through the captured graph.  Equivalent to
        `logits, cache = model(input_ids=token, cache=cache); next = argmax(logits[:, -1])`
        (reference phi_3_vision_mlx.py:391-392).  Returns (logits [B,1,V], next_token [B,1])
        -- views of persistent buffers, valid until the next call."""
        st = cache[0].state
        if st.offset + 1 > st.T:
            raise ValueError(f"KV cache overflow: {st.offset}+1 > {st.T} (prompt + max_tokens)")
        if st.epoch != self.epoch:                              # adapters changed since the capture: stale pointers
            st.graphs.clear()
            st.epoch = self.epoch
        st.note_written(st.offset, st.offset + 1)
        g = st.graphs.get("greedy")
        if g is not None and st.offset < g["bufs"].get("past_lb", -1):   # the cache was rewound below the captured lower bound
            g = None
        if g is None:
            g = st.graphs["greedy"] = self._build_decode_graph(st)
            g["host_tok"] = None
        if g["host_tok"] is None or token is not g["host_tok"]:
            g["tok"].copy_(token.reshape(-1).to(self.device, I32))   # first step / caller-chosen token
        g["d_past"].fill_(st.offset) if g.get("synced_offset") != st.offset else None
        g["graph"].launch()
        g["n_replays"] = g.get("n_replays", 0) + 1              # replay r wrote its token to history[:, r - 1] (while it fits)
        st.offset += 1
        g["synced_offset"] = st.offset
        g["host_tok"] = g["next_tok"].view(-1, 1)
        return g["logits"].view(st.B, 1, -1), g["host_tok"]

    @on_device
    def __call__(self, input_ids, pixel_values=None, image_sizes=None, positions=None, cache=None, pids=None, mask=None,
                 max_tokens=0, advance_offset=None, n_beam=1, full_logits=None):
        """Phi3ForCausalLM.__call__ (phi.py:606-608) + Phi3F.__call__ (phi.py:576-592).

        Returns (logits [B, L', V] in the model's activation type, cache).  On a prefill call (cache is None)
        only the last position is projected through lm_head (L' = 1) unless
        `full_logits=True`: every caller in the reference reads `logits[:, -1]`
        of a prefill only; cached calls return all L rows."""
        cfg = self.cfg
        if torch.is_tensor(input_ids):
            ids = input_ids.to(self.device, I32)
        else:
            ids = torch.as_tensor(np.asarray(input_ids).astype(np.int32)).to(self.device)
        if ids.dim() == 1:
            ids = ids[None]
        ids = ids.contiguous()
        B, L = ids.shape
        H = cfg.hidden_size
        prefill = cache is None
        if prefill and pixel_values is None and B == 1 and pids is None and mask is None and n_beam == 1 and not full_logits \
                and advance_offset is None:
            got = self._prefill_captured(ids, L, max_tokens)
            if got is not None:
                return got
        if prefill:
            # (before the vision tower is enqueued: the host is launch-bound through the ViT's ~280 launches, so whatever it does between
            #  the tower and the decoder -- cache allocation, its zero fill, the rotation tables -- would show as idle GPU time there)
            st = self._new_state(B, L, max_tokens, pids, mask)
            cache = [LayerCache(st, i) for i in range(cfg.num_hidden_layers)]
        else:
            st = cache[0].state
        x = self._embed(ids.view(-1))
        if pixel_values is not None and self.vision:
            self.vision_embed(x, pixel_values, image_sizes, positions, L)
        past = st.offset
        if n_beam == 1 and past + L > st.T:
            raise ValueError(f"KV cache overflow: {past}+{L} > {st.T} (prompt + max_tokens)")
        if full_logits is None:
            full_logits = not prefill
        keep = L if advance_offset is None else advance_offset
        if n_beam == 1:
            st.note_written(past, past + L, past + keep)
        x = self._layers(x, st, B, L, past, n_beam, last_only=not full_logits, keep=keep)
        if n_beam == 1:
            st.offset = past + L                                 # KVCache.__call__ auto-advance (phi.py:544-547)
        if advance_offset is not None:
            st.offset = past + advance_offset                    # phi.py:589-591
        if not full_logits and x.shape[0] != B:
            x = x.view(B, L, H)[:, -1, :].contiguous()
        logits = self._head(x)
        return logits.view(B, -1, cfg.vocab_size), cache

    # ------------------------------------------------------------------ captured prefill of short text prompts
    PREFILL_GRAPH_MAX_S = 512
    PREFILL_GRAPH_ENTRIES = 4
    PREFILL_GRAPH_MAX_CACHE_BYTES = 2 << 30                       # an entry pins its (S + max_tokens) KV cache: 393 KB per token at full size

    def _prefill_captured(self, ids, S, max_tokens):
        """Short text prompts (B = 1, 17 .. 512 tokens) are launch-bound: ~390 launches of a few microseconds each, every one paid
        for in Python + ctypes time (4.5 ms of wall time for 3.6 ms of kernels).  A (length, max_tokens) pair seen
        for the SECOND time is captured as ONE hipGraph over buffers the entry owns -- ids, activations, rotation tables, the KV
        cache itself -- and later prompts of that geometry cost one 0.5 KB copy + one graph launch.  The entry's cache is LEASED to
        the caller: every call gets its own CacheState object (a shallow copy of the entry's: same tensors, same decode graphs, its
        own offset) and the lease IS that object -- while it is alive, through the returned cache list or through a kept
        `cache[i].state`, a new prompt of the same geometry takes the eager path, so a caller that keeps two caches gets two caches
        (the reference's contract).  An entry whose caller died in an unrecovered failed step is dropped (`CacheState.mark_dirty`),
        and entries whose cache would exceed PREFILL_GRAPH_MAX_CACHE_BYTES are not made.  Bit-identical to the eager path (same
        kernels, same order).  P3V_PREFILL_GRAPH=0 switches it off.  Returns None when not applicable."""
        key = None
        if (os.environ.get("P3V_PREFILL_GRAPH", "1") != "0" and ops.L.DECODE_MAX_L < S <= self.PREFILL_GRAPH_MAX_S and max_tokens >= 1
                and self.hidden_hook is None
                and self._cache_token_bytes() * (S + max_tokens + 256) <= self.PREFILL_GRAPH_MAX_CACHE_BYTES):
            key = self._prefill_key(S, max_tokens)
        if key is None:
            return None
        e = self._prefill_graphs.get(key)
        if e is None:
            if self._prefill_seen.get(key, 0) < 1:                # first sighting: eager (one-off lengths never pay for a capture)
                if len(self._prefill_seen) > 64:
                    self._prefill_seen.clear()
                self._prefill_seen[key] = 1
                return None
            if len(self._prefill_graphs) >= self.PREFILL_GRAPH_ENTRIES:
                self._prefill_graphs.pop(next(iter(self._prefill_graphs)))
            e = self._prefill_graphs[key] = self._build_prefill_graph(S, max_tokens)
        if e["lease"] is not None and e["lease"]() is not None:    # the previous caller still holds this entry's cache
            return None
        if e["st"].shared["dirty"]:                               # its last caller died in a failed step: NaN rows, half-armed buffers
            del self._prefill_graphs[key]
            self._prefill_seen[key] = 1                           # (the next prompt of this geometry captures afresh)
            return None
        st = copy.copy(e["st"])                                   # this call's state: the entry's tensors and graphs, its own offset
        self._states.add(st)
        e["ids"].copy_(ids.view(-1), non_blocking=True)
        st.offset = 0
        g = st.graphs.get("greedy")
        if g is not None:                                         # the decode graph of this cache geometry stays valid: same buffers
            g["n_replays"], g["host_tok"], g["synced_offset"] = 0, None, None
            g["d_step"].zero_()
        e["graph"].launch()
        st.note_written(0, S)
        st.offset = S
        e["lease"] = weakref.ref(st)
        return e["logits"].clone().view(1, 1, self.cfg.vocab_size), [LayerCache(st, i) for i in range(self.cfg.num_hidden_layers)]

    def _build_prefill_graph(self, S, max_tokens):
        cfg, dev = self.cfg, self.device
        st = self._new_state(1, S, max_tokens, None, None)
        e = dict(st=st, lease=None, ids=torch.zeros((S,), dtype=I32, device=dev), x=torch.empty((S, cfg.hidden_size), dtype=self.x_dtype, device=dev),
                 logits=torch.empty((1, cfg.vocab_size), dtype=self.act_dtype, device=dev), bufs=self._alloc_bufs(1, S), ws={})

        def run():
            st.offset = 0
            self._embed(e["ids"], out=e["x"])
            xl = self._layers(e["x"], st, 1, S, 0, 1, bufs=e["bufs"], last_only=True)
            self._head(xl.view(1, -1), out=e["logits"], bufs=e["bufs"])
        with ops.owned_gemm_workspace(e["ws"], frozen=False):
            run()                                                # warm-up (sizes the split-K workspace the graph owns)
        torch.cuda.synchronize()
        graph = ops.Graph()
        side = torch.cuda.Stream(device=dev)
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side), ops.owned_gemm_workspace(e["ws"], frozen=True):
            graph.begin()
            run()
            graph.end()
        torch.cuda.current_stream().wait_stream(side)
        e["graph"] = graph
        return e

    @property
    def layers(self):
        return range(self.cfg.num_hidden_layers)
