"""Model configuration for the Phi-3-Vision / Phi-3-mini-128K hot path.

Mirrors what the reference reads from ``config.json`` into a SimpleNamespace
(reference phi_3_vision_mlx.py:359-363, keys listed in SURVEY.md App. B).
The rope factor arrays are the Phi-3-vision-128k-instruct values printed in the
reference's own notebook (assets/su_rope_explained.ipynb, cell 9); a real
``config.json`` always overrides them.
"""
import json
import math
from dataclasses import dataclass, replace
from types import SimpleNamespace
from typing import Optional, Tuple, Union

SHORT_FACTOR = [
    1.05, 1.05, 1.05, 1.1, 1.1, 1.1, 1.2500000000000002, 1.2500000000000002,
    1.4000000000000004, 1.4500000000000004, 1.5500000000000005, 1.8500000000000008,
    1.9000000000000008, 2.000000000000001, 2.000000000000001, 2.000000000000001,
    2.000000000000001, 2.000000000000001, 2.000000000000001, 2.000000000000001,
    2.000000000000001, 2.000000000000001, 2.000000000000001, 2.000000000000001,
    2.000000000000001, 2.000000000000001, 2.000000000000001, 2.000000000000001,
    2.000000000000001, 2.000000000000001, 2.000000000000001, 2.000000000000001,
    2.1000000000000005, 2.1000000000000005, 2.2, 2.3499999999999996,
    2.3499999999999996, 2.3499999999999996, 2.3499999999999996, 2.3999999999999995,
    2.3999999999999995, 2.6499999999999986, 2.6999999999999984, 2.8999999999999977,
    2.9499999999999975, 3.049999999999997, 3.049999999999997, 3.049999999999997,
]
LONG_FACTOR = [
    1.0299999713897705, 1.0499999523162842, 1.0499999523162842, 1.0799999237060547,
    1.2299998998641968, 1.2299998998641968, 1.2999999523162842, 1.4499999284744263,
    1.5999999046325684, 1.6499998569488525, 1.8999998569488525, 2.859999895095825,
    3.68999981880188, 5.419999599456787, 5.489999771118164, 5.489999771118164,
    9.09000015258789, 11.579999923706055, 15.65999984741211, 15.769999504089355,
    15.789999961853027, 18.360000610351562, 21.989999771118164, 23.079999923706055,
    30.009998321533203, 32.35000228881836, 32.590003967285156, 35.56000518798828,
    39.95000457763672, 53.840003967285156, 56.20000457763672, 57.95000457763672,
    59.29000473022461, 59.77000427246094, 59.920005798339844, 61.190006256103516,
    61.96000671386719, 62.50000762939453, 63.3700065612793, 63.48000717163086,
    63.48000717163086, 63.66000747680664, 63.850006103515625, 64.08000946044922,
    64.760009765625, 64.80001068115234, 64.81001281738281, 64.81001281738281,
]

# CLIP ViT-L/14-336 is hard-coded in the reference (phi.py:375-384).
CLIP_L_336 = dict(hidden_size=1024, image_size=336, intermediate_size=4096,
                  layer_norm_eps=1e-05, num_attention_heads=16, num_channels=3,
                  num_hidden_layers=24, patch_size=14)


def phi3v_config_dict(vision=True):
    """Full-size Phi-3-Vision (or blind Phi-3-mini-128K) config as a dict."""
    d = dict(
        architectures=["Phi3VForCausalLM" if vision else "Phi3ForCausalLM"],
        hidden_size=3072, num_attention_heads=32, num_key_value_heads=32,
        num_hidden_layers=32, intermediate_size=8192, vocab_size=32064,
        rms_norm_eps=1e-05, rope_theta=10000.0, max_position_embeddings=131072,
        original_max_position_embeddings=4096,
        rope_scaling=dict(type="su", short_factor=list(SHORT_FACTOR), long_factor=list(LONG_FACTOR)),
    )
    if vision:
        d["img_processor"] = dict(image_dim_out=1024, name="clip_vision_model", num_img_tokens=144)
        d["clip"] = dict(CLIP_L_336)
    return d


def tiny_config_dict(vision=True):
    """A tiny config with the same structure (head_dim stays 96 so the same
    kernels are exercised; CLIP head_dim stays 64; image stays 336/14 so the
    reference's HD transform and token-count formula apply unchanged)."""
    n = 48
    d = dict(
        architectures=["Phi3VForCausalLM" if vision else "Phi3ForCausalLM"],
        hidden_size=192, num_attention_heads=2, num_key_value_heads=2,
        num_hidden_layers=2, intermediate_size=256, vocab_size=32064,
        rms_norm_eps=1e-05, rope_theta=10000.0, max_position_embeddings=131072,
        original_max_position_embeddings=4096,
        rope_scaling=dict(type="su", short_factor=list(SHORT_FACTOR[:n]), long_factor=list(LONG_FACTOR[:n])),
    )
    if vision:
        d["img_processor"] = dict(image_dim_out=128, name="clip_vision_model", num_img_tokens=144)
        d["clip"] = dict(hidden_size=128, image_size=336, intermediate_size=256,
                         layer_norm_eps=1e-05, num_attention_heads=2, num_channels=3,
                         num_hidden_layers=3, patch_size=14)
    return d


def make_config(d=None, **kwargs):
    """dict (+ kwargs overlay, as reference `_get_cfg`) -> SimpleNamespace."""
    d = dict(d if d is not None else phi3v_config_dict())
    if "architecture" in d:
        return layered_config(d, **kwargs)
    if kwargs.get("dtype") not in (None, "bfloat16"):
        raise ValueError(f"dtype {kwargs['dtype']!r}: this model runs in bfloat16")
    d.update(kwargs)
    cfg = SimpleNamespace(**d)
    if getattr(cfg, "img_processor", None) is not None and not hasattr(cfg, "clip"):
        cfg.clip = dict(CLIP_L_336)
    return cfg


# ---------------------------------------------------------------- layered text decoders
@dataclass(frozen=True)
class Mixer:
    """One attention mixer: H query heads over G key / value heads (query head h uses key / value head h // (H / G))."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    v_mix: bool


@dataclass(frozen=True)
class Rotary:
    """Rotary positions on `dims` dimensions, dimension i paired with i + dims / 2.  yarn: None, or (factor, original, fast, slow)."""
    dims: int
    base: float
    yarn: Optional[Tuple[float, float, float, float]] = None

    def frequencies(self):
        """(angle per position of every pair, factor on cos and sin), float64."""
        pair = range(self.dims // 2)
        f = [self.base ** (-2.0 * i / self.dims) for i in pair]
        if self.yarn is None:
            return f, 1.0
        factor, original, fast, slow = self.yarn

        def dim_of(turns):
            return self.dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(self.base))
        lo, hi = max(math.floor(dim_of(fast)), 0), min(math.ceil(dim_of(slow)), self.dims - 1)
        ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in pair]
        return [x / factor * r + x * (1 - r) for x, r in zip(f, ramp)], 0.1 * math.log(factor) + 1.0


@dataclass(frozen=True)
class LatentMixer:
    """Latent attention: one latent of `rank` values and one rotated key part of `rot.dims` values per token, shared by the heads."""
    heads: int
    dim: int
    vdim: int
    rank: int
    rot: Rotary
    scale: float


@dataclass(frozen=True)
class GlaMixer:
    """Gated linear attention: a [dim, vdim] state per head, a decay per key channel out of a low-rank projection.  gate_rank: its rank
    (None: what the checkpoint's tensors have)."""
    heads: int
    dim: int
    vdim: int
    tau: float
    gate_rank: Optional[int] = None


@dataclass(frozen=True)
class Mlp:
    ff: int


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[Mixer, LatentMixer, GlaMixer]
    mlp: Optional[Mlp]
    owner: Optional[int] = None                      # the layer whose tensors this one uses (None: its own)


def _attention(i, m):
    mixer = Mixer(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]), bool(m["v_mix"]))
    if mixer.heads % mixer.kv_heads:
        raise ValueError(f"layer {i}: {mixer.heads} query heads over {mixer.kv_heads} key / value heads")
    return mixer


def _latent_attention(i, m):
    rot, s = m["rot"], m["rot"].get("scaling")
    if int(rot.get("dims", m["rot_dim"])) != int(m["rot_dim"]) or int(m["rot_dim"]) % 2:
        raise ValueError(f"layer {i}: rotary dimensions {rot.get('dims')} of a rotated part of {m['rot_dim']}")
    yarn = None if s is None else tuple(float(s[k]) for k in ("factor", "original", "fast", "slow"))
    return LatentMixer(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), Rotary(int(m["rot_dim"]), float(rot["base"]), yarn),
                       float(m["scale"]))


def _gla(i, m):
    return GlaMixer(int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["tau"]), None if m.get("gate_rank") is None else int(m["gate_rank"]))


@dataclass(frozen=True)
class Design:
    """What is the same in every model of a layered design: its mixers ('type' of a layer -> reader of its sizes), the norm in front of
    a branch ("dyt" | "rms"), the activation of its feed-forward, what the branches carry, whether the head is the embedding table."""
    mixers: dict
    norm: str
    act: str
    token_shift: bool = False
    layer_scale: bool = False
    tied_head: bool = False


DESIGNS = {
    "Pelalix": Design({"attention": _attention}, norm="dyt", act="silu", token_shift=True, layer_scale=True),
    "Pudisun": Design({"latent_attention": _latent_attention, "gla": _gla}, norm="rms", act="gelu_tanh", tied_head=True),
}


def _layer_spec(design, i, d):
    if d["type"] not in design.mixers:
        raise ValueError(f"layer {i}: unknown mixer type {d['type']!r}")
    mixer = design.mixers[d["type"]](i, d["mixer"])
    mlp = d.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
    return LayerSpec(mixer, None if mlp is None else Mlp(int(mlp["ff"])), d.get("weights_of"))


def _resolve_owners(layers):
    """Layers that use another one's tensors name the layer that has them."""
    out = []
    for i, s in enumerate(layers):
        j, seen = s.owner, {i}
        while j is not None and 0 <= j < len(layers) and j not in seen and layers[j].owner is not None:
            seen.add(j)
            j = layers[j].owner
        if j is not None:
            if not 0 <= j < len(layers) or j in seen:
                raise ValueError(f"layer {i}: no layer has the weights it names ({s.owner})")
            if (layers[j].mixer, layers[j].mlp) != (s.mixer, s.mlp):
                raise ValueError(f"layer {i}: other sizes than layer {j}, whose weights it uses")
        out.append(replace(s, owner=j))
    return tuple(out)


def layered_config(d, dtype=None, shift_rows=128, state_rows=2, **kwargs):
    """config.json of a layered decoder -> SimpleNamespace.  dtype: "bfloat16" (default) or "float32" activations; shift_rows /
    state_rows: columns of token-shift history / recurrent states a cache keeps (how far it can be rewound)."""
    for k in ("use_quantized_cache", "quantized_fp8", "quantized_int4"):
        if kwargs.pop(k, False):
            raise ValueError(f"{k} is not available for {d['architecture']}")
    if dtype not in (None, "bfloat16", "float32"):
        raise ValueError(f"dtype must be 'bfloat16' or 'float32', got {dtype!r}")
    if d["architecture"] not in DESIGNS:
        raise ValueError(f"unknown architecture {d['architecture']!r}")
    design = DESIGNS[d["architecture"]]
    layers = _resolve_owners([_layer_spec(design, i, x) for i, x in enumerate(d["layers"])])
    mixing = {s.mixer.kv_heads * s.mixer.vdim for s in layers if getattr(s.mixer, "v_mix", False)}
    if len(mixing) > 1:
        raise ValueError(f"value-mixing layers of different value widths {sorted(mixing)}")
    if not layers:
        raise ValueError("a model without layers")
    if float(d.get("residual_mult", 1.0)) == 0.0:
        raise ValueError("residual_mult 0: the layers would not reach the output")
    return SimpleNamespace(architectures=[d["architecture"]], design=design, layers=layers, num_hidden_layers=len(layers),
                           hidden_size=int(d["width"]), vocab_size=int(d["vocab"]), norm_eps=float(d["norm"]["eps"]),
                           embed_scale=float(d.get("embedding", {}).get("scale", 1.0)), residual_mult=float(d.get("residual_mult", 1.0)),
                           logit_scale=float(d.get("logit_scale", 1.0)), dtype=dtype or "bfloat16", shift_rows=int(shift_rows),
                           state_rows=int(state_rows), **kwargs)


def load_config(json_path, **kwargs):
    """Same error behaviour as reference `_get_cfg` (phi_3_vision_mlx.py:359-369)."""
    try:
        with open(json_path, "r") as f:
            d = json.load(f)
    except FileNotFoundError:
        raise FileNotFoundError(f"Configuration file not found: {json_path}")
    except json.JSONDecodeError:
        raise ValueError(f"Invalid JSON in configuration file: {json_path}")
    return make_config(d, **kwargs)


def is_vision(cfg):
    return cfg.architectures[0].startswith("Phi3V")


def head_dim(cfg):
    return cfg.hidden_size // cfg.num_attention_heads


def rope_scaling_factor(cfg):
    """sqrt(1 + ln(max/orig)/ln(orig)) (reference phi.py:491)."""
    return math.sqrt(1 + math.log(cfg.max_position_embeddings / cfg.original_max_position_embeddings)
                     / math.log(cfg.original_max_position_embeddings))
