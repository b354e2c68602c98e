#!/usr/bin/env python3
"""Headline benchmark: Phi-3-Vision bf16 single-image VQA on MI355X
(BASELINE.json `configs[1]`): prefill ms + decode tokens/s, with the rooflines
of the dominant decode kernel and of the prefill, and the CPU oracle timed beside it.

    python bench.py --gpus N --steps K --warmup W            (N > 1 without a launcher: this process starts the N ranks itself)
    python -m torch.distributed.run --nnodes=1 --nproc-per-node N ... bench.py --gpus N ...
    python bench.py --config4 [--gpus N]                     (8 mixed image + text requests per GPU, B = 8)

One process per GPU, each with its own replica and its own request(s) (batch
sharding, no data-path collective -> "weak" scaling); RCCL is used for the
barriers, the max-over-ranks of the timed span and the token gather.
A "step" = one greedy decode step (one new token per sequence) through the
same graph-replayed path `generate()` uses; timing definitions follow the
reference (phi_3_vision_mlx.py:384-403): prefill = first `model(**inputs)` +
argmax + sync, timer started AFTER preprocessing.
Synthetic data: seeded random weights of the real architecture, one seeded
random 336x336 image (-> 1344x1344 HD, 17 crops, 2509 image tokens) + 20
random text tokens.  Prints ONE JSON line on rank 0.

`value` is the REFERENCE-DEFINED rate: (gen_len - 1) / gen_time over the K timed steps through `_generate`'s own loop
(per-token D2H copy = the reference's mx.eval, Streamer, TokenStopper, detokenisation; phi_3_vision_mlx.py:390-403);
`device_rate` is K further steps as back-to-back graph replays between two syncs (what the kernels sustain), run AFTER that loop.
At N = 1 the line also carries `configs`: BASELINE configs[0], [2], [3] (one GPU's share) and [4] measured in the same
process with the same definitions, each with its own roofline fractions (`--no-configs` skips them).
"""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0          # MI355X_MICROARCH.md: HBM3E 8 TB/s spec (6.29 TB/s measured copy)
MFMA_BF16_PEAK_TFLOPS = 2500.0  # MI355X_MICROARCH.md: dense bf16 MFMA peak


def parse():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--prefill-reps", type=int, default=5)
    ap.add_argument("--no-cpu-baseline", action="store_true")
    ap.add_argument("--no-configs", action="store_true", help="skip the `configs` object (the other BASELINE configs, N = 1 only)")
    ap.add_argument("--configs-steps", type=int, default=32, help="timed decode steps per entry of `configs`")
    ap.add_argument("--config4", action="store_true", help="BASELINE configs[3]: 8 mixed image+text requests per GPU, batched (B = 8)")
    ap.add_argument("--config5", action="store_true", help="BASELINE configs[4]: fp8 (e4m3) weights, W8A8 prefill on the fp8 MFMA, int8 KV cache")
    ap.add_argument("--fp8-weight-only", action="store_true", help="with --config5: fp8_activations=False (dequantise + bf16 MFMA prefill)")
    ap.add_argument("--layered", nargs="?", const="Pelalix", default=None, choices=("Pelalix", "Pudisun"),
                    help="a layered text decoder (layers of realistic sizes, random weights) beside Phi-3 layers (Pudisun: and Pelalix layers) of equal "
                    "size: prefill and decode throughput; its own JSON line instead of the headline one")
    ap.add_argument("--tiny", action="store_true", help="tiny config (debug only; the result is NOT the headline metric)")
    return ap.parse_args()


def spawn_ranks(args):
    """`python bench.py --gpus N` without a launcher: start the N ranks (one per GPU) as a CHILD torchrun before this
    process has touched the GPU, relay its output, exit with its code."""
    import socket
    import subprocess
    s = socket.socket()
    s.bind(("127.0.0.1", 0))
    port = s.getsockname()[1]
    s.close()
    cmd = [sys.executable, "-m", "torch.distributed.run", "--nnodes=1", f"--nproc-per-node={args.gpus}", "--master-addr", "127.0.0.1",
           "--master-port", str(port), os.path.abspath(__file__)] + sys.argv[1:]
    sys.exit(subprocess.run(cmd).returncode)


def usable_cores(cap=64):
    """Threads the CPU leg may really use: affinity mask and cgroup CPU quota, capped."""
    n = len(os.sched_getaffinity(0)) if hasattr(os, "sched_getaffinity") else (os.cpu_count() or 1)
    try:
        q, per = open("/sys/fs/cgroup/cpu.max").read().split()
        if q != "max":
            n = min(n, max(1, int(int(q) / int(per))))
    except Exception:
        pass
    return max(1, min(n, cap))


def cpu_baseline(model, n_decode=32, runs=3, warm_decode=2):
    """the CPU oracle (torch-CPU restatement of phi.py, kind "port") on BASELINE config 1 --
    text-only, 128-token prompt, greedy, ALL layers -- on this box's host cores: one warm-up pass (prefill + `warm_decode`
    steps), then `runs` timed passes of prefill + `n_decode` decode steps (median); prefill ms and decode tokens/s with the
    reference's definitions (phi_3_vision_mlx.py:384-403).  BOUNDED sample of the 128 new tokens BASELINE.md names: 32 steps
    per pass at ~1.7 tok/s (3 passes ~ 60 s of CPU work in all); a decode step's cost is flat in the step index at this
    context (weights dominate).  Baseline only -- never on the product path."""
    import numpy as np
    import torch
    sys.path.insert(0, os.path.join(ROOT, "oracle"))
    import phi3v_oracle as orc
    cfg = model.cfg
    cores = usable_cores()
    torch.set_num_threads(cores)
    w = {k: v.cpu() for k, v in model.w.items() if k.startswith("model.layers.") or k in
         ("model.embed_tokens.weight", "model.norm.weight", "lm_head.weight")}
    # a quantised build (--config5, 4-bit) keeps no bf16 copy of its decoder projections: the baseline's oracle gets the
    # dequantised values (its TIMING is what is reported; config 1 on bf16-valued weights either way)
    from phi_3_vision_mlx_amd import ops
    for k, (q, sc) in getattr(model, "w8", {}).items():
        if k not in w and (k.startswith("model.layers.") or k == "lm_head.weight"):
            w[k] = ops.dequant_fp8(q, sc).cpu()
    for k, (q, sb) in getattr(model, "w4", {}).items():
        if k not in w and (k.startswith("model.layers.") or k == "lm_head.weight"):
            w[k] = ops.dequant_q4(q, sb).cpu()
    o = orc.OraclePhi3V(cfg, w, cache_fp32=True)
    o.vision = False
    ids = np.random.default_rng(0).integers(3, 32000, (1, 128)).astype(np.int64)
    pre, dec = [], []
    for run in range(runs + 1):
        nd = warm_decode if run == 0 else n_decode
        t0 = time.perf_counter()
        logits, cache = o(input_ids=ids, max_tokens=nd + 1)
        tok = torch.argmax(logits[:, -1].float(), dim=-1)[:, None]
        t1 = time.perf_counter()
        for _ in range(nd):
            logits, cache = o(input_ids=tok, cache=cache)
            tok = torch.argmax(logits[:, -1].float(), dim=-1)[:, None]
        t2 = time.perf_counter()
        if run > 0:                                               # run 0 = warm-up (builds the fp32 weight copies)
            pre.append((t1 - t0) * 1e3), dec.append(nd / (t2 - t1))
    return {"value": round(float(np.median(dec)), 3), "unit": "tokens/s", "cores": cores, "kind": "port",
            "prefill_ms": round(float(np.median(pre)), 1),
            "sample": f"BASELINE config 1 (text-only, 128-token prompt, all {cfg.num_hidden_layers} layers, fp32 attention/KV as "
                      f"phi.py) on torch-CPU: 1 warm-up pass + {runs} timed pass(es); {n_decode} of the 128 decode steps per pass"}


PMC_TRAFFIC_FILE = "r06_pmc_hbm_traffic.json"      # written by tools/pmc_round6.sh from separate rocprofv3 --pmc passes


def kernel_source_sha16():
    """Identity of the dominant kernel's sources (the GEMV translation unit and what it includes)."""
    import hashlib
    h = hashlib.sha256()
    for f in ("p3v_gemv.hip", "p3v_gemv3_body.h", "p3v_common.h"):
        with open(os.path.join(ROOT, "phi-3-vision-mlx_amd", "csrc", f), "rb") as fh:
            h.update(fh.read())
    return h.hexdigest()[:16]


def prefill_flops(cfg, S, n_img_tokens, n_crops):
    """Algorithmic FLOPs of the prefill: decoder linears (lm_head on the last row only), causal attention
    (lower triangle), ViT on the live crops, projector."""
    H, I, V, NL = cfg.hidden_size, cfg.intermediate_size, cfg.vocab_size, cfg.num_hidden_layers
    hd = H // cfg.num_attention_heads
    per_tok = NL * ((cfg.num_attention_heads + 2 * cfg.num_key_value_heads) * hd * H + H * H + 2 * I * H + I * H)
    f = 2.0 * S * per_tok + 2.0 * V * H + 2.0 * NL * S * S * H
    if n_crops:
        c = cfg.clip
        D, DI, T, P = c["hidden_size"], c["intermediate_size"], (c["image_size"] // c["patch_size"]) ** 2 + 1, c["patch_size"]
        vit = (c["num_hidden_layers"] - 1) * (2.0 * T * (4 * D * D + 2 * D * DI) + 4.0 * T * T * D) + 2.0 * (T - 1) * 3 * P * P * D
        f += n_crops * vit + 2.0 * n_img_tokens * (4 * cfg.img_processor["image_dim_out"] * H + H * H)
    return f


def decode_bytes(model, cfg, valid_tokens, B, steps_done, kv_elt):
    """Algorithmic HBM bytes of one decode step: every decoder + lm_head weight once (in its storage format) +
    the K / V rows of every live position."""
    hd = cfg.hidden_size // cfg.num_attention_heads
    kv = 2 * cfg.num_hidden_layers * cfg.num_key_value_heads * hd * kv_elt * (valid_tokens + B * steps_done)
    w = sum(v.numel() * 2 for k, v in model.w.items() if k.startswith("model.layers.") or k == "lm_head.weight") \
        + sum(v[0].numel() for v in model.w8.values())
    return w + kv


def measure_request_set(model, processor, reqs, steps, warmup, prefill_reps, kv_elt=2):
    """One entry of `configs` (single GPU): `reqs` = B = 1 model inputs; prefill (median of `prefill_reps` after two warm-ups;
    several requests: the length-bucketed batch prefill of dist.prefill_requests) + `steps` timed greedy steps twice -- through
    `_generate`'s loop (reference-defined rate) and as bare graph replays (device rate).  Definitions as the headline's."""
    import numpy as np
    import torch
    from phi_3_vision_mlx_amd import api, ops
    from phi_3_vision_mlx_amd.dist import prefill_requests
    cfg = model.cfg
    B = len(reqs)
    max_tokens = 2 * (warmup + steps) + 8
    pms = []
    n_warm = 2        # untimed: the first sight of a geometry runs eager, the second captures its graphs (short-prompt prefill, vision tower)
    for rep in range(prefill_reps + n_warm):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        if B > 1:
            token, cache, _ = prefill_requests(model, reqs, max_tokens)
        else:
            logits, cache = model(**reqs[0], max_tokens=max_tokens)
            token = ops.argmax(logits[:, -1, :].contiguous())[:, None]
        first = token.tolist()
        if rep >= n_warm:
            pms.append((time.perf_counter() - t0) * 1e3)
        if rep < prefill_reps + n_warm - 1:
            del cache
    prefill = float(np.median(pms))
    print(f"configs: prefill reps ms (B={B}, {len(reqs)} request(s)):", [round(v, 1) for v in pms], file=sys.stderr)
    for _ in range(warmup):
        _, token = model.greedy_step(token, cache)
    torch.cuda.synchronize()
    streamer, stopper = api.Streamer(processor, False, True), api.TokenStopper(processor, B)   # the reference-defined loop first,
    t0 = time.perf_counter()                                                                     # the bare replays after it (as main())
    streamer(api._rows(token))
    token = api.greedy_loop(model, token, cache, steps, streamer, stopper)
    _, gen_len = streamer.end()
    torch.cuda.synchronize()
    gen_s = time.perf_counter() - t0
    t0 = time.perf_counter()
    for _ in range(steps):
        _, token = model.greedy_step(token, cache)
    torch.cuda.synchronize()
    dev_s = (time.perf_counter() - t0) / steps
    lens = [int(np.asarray(r["input_ids"]).shape[-1]) for r in reqs]
    valid = sum(lens)
    nbytes = decode_bytes(model, cfg, valid, B, warmup + steps // 2, kv_elt)
    flops = 0.0
    for r in reqs:
        ids = np.asarray(r["input_ids"])
        n_img = int((ids < 0).sum())
        n_crops = int(sum(h * w + 1 for h, w in (np.asarray(r["image_sizes"]) // 336).tolist())) if "image_sizes" in r else 0
        flops += prefill_flops(cfg, ids.shape[-1], n_img, n_crops)
    del cache
    return {
        "batch": B, "prompt_tokens": lens if B > 1 else lens[0], "steps": steps, "prefill_ms": round(prefill, 3),
        "decode_tokens_per_s": round((gen_len - 1) / gen_s, 2), "device_tokens_per_s": round(B / dev_s, 2),
        "ms_per_step": round(dev_s * 1e3, 4), "first_token": first,
        "roofline_decode": {"bound": "hbm", "algorithmic_GB_per_step": round(nbytes / 1e9, 3), "achieved": round(nbytes / dev_s / 1e9, 1),
                            "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": round(nbytes / dev_s / 1e9 / HBM_PEAK_GBS, 4)},
        "roofline_prefill": {"bound": "mfma", "algorithmic_TFLOP": round(flops / 1e12, 2), "achieved": round(flops / (prefill * 1e-3) / 1e12, 1),
                             "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": round(flops / (prefill * 1e-3) / 1e12 / MFMA_BF16_PEAK_TFLOPS, 4)},
    }


def other_configs(model, processor, dev, args):
    """BASELINE.json configs[0], [2], [3] (one GPU's share) and [4] on this GPU, driver-timed inside the default run."""
    import numpy as np
    import torch
    from phi_3_vision_mlx_amd.api import load_synthetic
    from phi_3_vision_mlx_amd.workloads import c4_share, vqa_request
    ip = processor.img_processor
    K, W = args.configs_steps, 4
    rng = np.random.default_rng(0)
    out = {}
    t_all = time.perf_counter()
    # text-only, 128-token prompt (the CPU reference's case; same decoder weights as the blind model)
    ids = rng.integers(3, 32000, (1, 128)).astype(np.int64)
    out["c1_text_128"] = dict(measure_request_set(model, processor, [{"input_ids": ids}], max(K, 64), W, 3),
                              workload="BASELINE configs[0]: text-only greedy, 128-token prompt, B=1")
    # 32k-token long-context prefill + decode (long RoPE factors)
    S3 = 5000 if args.tiny else 32768
    ids = np.random.default_rng(4).integers(3, 32000, (1, S3)).astype(np.int64)
    out["c3_long_32k"] = dict(measure_request_set(model, processor, [{"input_ids": ids}], K, W, 3),    # (3 reps: one in ~4 takes 1.5x)
                              workload=f"BASELINE configs[2]: {S3}-token text prompt (Su/LongRoPE long factors), prefill + decode at that context, B=1")
    torch.cuda.empty_cache()
    # one GPU's share of the 64-request mixed batch: 4 single-image VQA + 4 text prompts as one B = 8 decode batch
    reqs = c4_share(ip, 0, device=dev)
    out["c4_share_b8"] = dict(measure_request_set(model, processor, reqs, K, W, 2),
                              workload="BASELINE configs[3], one GPU's share (8 of 64 requests): 4 single-image VQA (2531 tokens) + 4 text "
                                       "prompts (16..256 tokens), length-bucketed prefill, one B=8 decode batch; x8 GPUs = the config")
    # fp8 weights (W8A8 prompt projections on the fp8 MFMA) + int8 KV on the headline request
    m5, p5 = load_synthetic(blind_model=False, tiny=args.tiny, seed=0, device=dev, quantized_fp8=True, use_quantized_cache=True)
    r5 = measure_request_set(m5, p5, [vqa_request(p5.img_processor, 0, device=dev)], max(K, 64), W, 3, kv_elt=1)
    r5["roofline_prefill"]["peak_note"] = "bf16 dense peak; the decoder projections run on the fp8 MFMA (2x that peak), the ViT stays bf16"
    out["c5_fp8_int8kv"] = dict(r5, workload="BASELINE configs[4]: configs[1]'s request with e4m3 decoder weights (per-row scales), e4m3 "
                                           "prompt activations (fp8 MFMA), int8 KV cache", dtype="fp8(e4m3)+int8kv")
    del m5
    torch.cuda.empty_cache()
    out["seconds"] = round(time.perf_counter() - t_all, 1)
    return out


LAYERED_SIZES = [(3072, 32, 32, 96, 8192), (3072, 32, 8, 96, 8192), (1536, 16, 4, 96, 4096)]     # width, heads, kv heads, head size, ff
LAYERED_LAYERS, LAYERED_VOCAB = 8, 32064


def layered_config_dict(width, heads, kv, dim, ff, layers=LAYERED_LAYERS):
    """A Pelalix config with the layer sizes of a Phi-3 decoder."""
    layer = {"type": "attention", "mlp": {"kind": "dense", "ff": ff},
             "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "v_mix": True}}
    return {"architecture": "Pelalix", "width": width, "vocab": LAYERED_VOCAB, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0}, "layers": [layer] * layers}


# Pudisun: width, ff, latent attention (heads, dim, rotated dim, vdim, rank), gated linear attention (heads, dim, vdim); the layers alternate.
# Beside them Phi-3 and Pelalix layers of the same width and feed-forward whose attention has as many 96-wide heads as the width holds.
PUDISUN_SIZES = [(3072, 8192, (32, 64, 32, 96, 512), (32, 64, 96)), (3072, 8192, (24, 128, 64, 128, 512), (16, 96, 192)),
                 (1536, 4096, (16, 64, 32, 96, 256), (16, 48, 96))]


def pudisun_config_dict(width, ff, latent, gla, layers=LAYERED_LAYERS):
    H, dim, rot, vdim, rank = latent
    rotary = {"base": 10000.0, "dims": rot, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}
    mixers = [("latent_attention", {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": rotary, "scale": (dim + rot) ** -0.5}),
              ("gla", {"heads": gla[0], "dim": gla[1], "vdim": gla[2], "tau": 16.0})]
    return {"architecture": "Pudisun", "width": width, "vocab": LAYERED_VOCAB, "norm": {"eps": 1e-5}, "residual_mult": 0.5, "logit_scale": 1.0,
            "layers": [{"type": t, "mixer": m, "mlp": {"kind": "dense", "ff": ff}} for t, m in (mixers * layers)[:layers]]}


def layered_run(model, prompts, decodes, steps, reps=5):
    """{prompt length: (ms, tokens/s)} of the whole prompt call and {(batch, context): (ms per step, tokens/s)} of the captured greedy step."""
    import numpy as np
    import torch
    from phi_3_vision_mlx_amd import ops
    out = {"prefill": {}, "decode": {}}
    rng = np.random.default_rng(0)
    for S in prompts:
        ids, ms = rng.integers(3, 32000, (1, S)), []
        for rep in range(reps + 2):
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            logits, cache = model(input_ids=ids, max_tokens=8)
            ops.argmax(logits[:, -1, :].contiguous()).tolist()
            ms.append((time.perf_counter() - t0) * 1e3)
            del logits, cache
        t = float(np.median(ms[2:]))
        out["prefill"][str(S)] = {"ms": round(t, 3), "tokens_per_s": round(S / t * 1e3, 1)}
        print("layered: prefill", S, out["prefill"][str(S)], file=sys.stderr, flush=True)
    for B, S in decodes:
        logits, cache = model(input_ids=rng.integers(3, 32000, (B, S)), max_tokens=4 * steps + 16)
        tok = ops.argmax(logits[:, -1, :].contiguous())[:, None]
        ts = []
        for rep in range(4):                                      # (the first region warms up and captures)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            for _ in range(steps):
                _, tok = model.greedy_step(tok, cache)
            torch.cuda.synchronize()
            ts.append((time.perf_counter() - t0) / steps * 1e3)
        t = float(np.median(ts[1:]))
        out["decode"][f"B{B}@{S}"] = {"ms_per_step": round(t, 4), "tokens_per_s": round(B / t * 1e3, 1)}
        print("layered: decode", B, S, out["decode"][f"B{B}@{S}"], file=sys.stderr, flush=True)
        del cache
    return out


def bench_layered(args):
    import torch
    from phi_3_vision_mlx_amd.api import load_synthetic
    from phi_3_vision_mlx_amd.config import phi3v_config_dict
    torch.cuda.set_device(0)
    prompts, decodes = (512, 2048, 8192), ((1, 512), (1, 2048), (1, 8192), (8, 2048))
    own = args.layered.lower()

    def phi3(width, heads, kv, ff):
        return dict(phi3v_config_dict(vision=False), hidden_size=width, num_attention_heads=heads, num_key_value_heads=kv, intermediate_size=ff,
                    num_hidden_layers=LAYERED_LAYERS)
    if own == "pelalix":
        sizes = [({"width": width, "heads": heads, "kv_heads": kv, "head_size": dim, "ff": ff},
                  {"pelalix": layered_config_dict(width, heads, kv, dim, ff), "phi3": phi3(width, heads, kv, ff)})
                 for width, heads, kv, dim, ff in LAYERED_SIZES]
    else:
        sizes = [({"width": width, "ff": ff, "latent_heads_dim_rot_vdim_rank": latent, "gla_heads_dim_vdim": gla},
                  {"pudisun": pudisun_config_dict(width, ff, latent, gla), "pelalix": layered_config_dict(width, width // 96, width // 96, 96, ff),
                   "phi3": phi3(width, width // 96, width // 96, ff)}) for width, ff, latent, gla in PUDISUN_SIZES]
    rows = []
    for size, configs in sizes:
        row = dict(size, layers=LAYERED_LAYERS, vocab=LAYERED_VOCAB)
        for name, cfg in configs.items():
            model, _ = load_synthetic(config=cfg, device="cuda:0")
            print("layered:", name, size, file=sys.stderr, flush=True)
            row[name] = layered_run(model, prompts, decodes, args.steps if args.steps != 128 else 48)
            del model
            torch.cuda.empty_cache()
        for other in configs:
            if other != own:
                row[f"{own}_over_{other}_time"] = {k: {s: round(row[own][k][s][f] / row[other][k][s][f], 3) for s in row[other][k]}
                                                   for k, f in (("prefill", "ms"), ("decode", "ms_per_step"))}
        rows.append(row)
    print(json.dumps({"metric": f"layered decoders ({args.layered}): prefill ms and decode ms per step beside layers of equal size of the other models",
                      "dtype": "bf16", "data": "synthetic", "higher_is_better": False, "sizes": rows}), flush=True)


def main():
    args = parse()
    if args.layered:
        return bench_layered(args)
    if args.gpus > 1 and "WORLD_SIZE" not in os.environ:
        spawn_ranks(args)                                         # does not return
    import numpy as np
    import torch
    import torch.distributed as dist

    world = int(os.environ.get("WORLD_SIZE", "1"))
    rank = int(os.environ.get("RANK", "0"))
    local = int(os.environ.get("LOCAL_RANK", "0"))
    assert world == args.gpus, f"WORLD_SIZE={world} but --gpus {args.gpus}"
    share = bool(os.environ.get("P3V_BENCH_SHARE_GPU"))           # debug only: all ranks on GPU 0 over gloo (1-GPU boxes)
    if share:
        local = 0
        os.environ.setdefault("P3V_SHARED_GPU", "1")               # several processes on one GPU: no launch that needs the whole chip resident
    elif torch.cuda.device_count() <= local:
        raise SystemExit(f"rank {rank}: needs GPU {local}, {torch.cuda.device_count()} visible (one rank per GPU)")
    torch.cuda.set_device(local)
    dev = f"cuda:{local}"
    if world > 1:
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        if share:
            dist.init_process_group("gloo", rank=rank, world_size=world)
        else:
            dist.init_process_group("nccl", rank=rank, world_size=world, device_id=torch.device(dev))

    from phi_3_vision_mlx_amd import api, ops
    from phi_3_vision_mlx_amd.api import load_synthetic
    from phi_3_vision_mlx_amd.processor import collate_requests
    from phi_3_vision_mlx_amd.workloads import c4_share, vqa_request

    t0 = time.perf_counter()
    q5 = dict(quantized_fp8=True, use_quantized_cache=True, fp8_activations=not args.fp8_weight_only) if args.config5 else {}
    model, processor = load_synthetic(blind_model=False, tiny=args.tiny, seed=0, device=dev, **q5)
    torch.cuda.synchronize()
    t_weights = time.perf_counter() - t0
    cfg = model.cfg
    ip = processor.img_processor

    # ---- request(s): the image stage exactly as `processor(text, images)` runs it -- resize / pad / normalise / crop on
    #      the GPU (same bits as the host path; P3V_HOST_PREPROCESS=1 selects that one), outside the prefill timer like
    #      the reference's processor.  Default: one 336x336 image (seed = rank) + 20 random text tokens;
    #      --config4: this rank's 4 image + 4 text requests as ONE left-padded batch
    host_pre = os.environ.get("P3V_HOST_PREPROCESS") == "1"
    pdev = None if host_pre else dev

    share_reqs = []

    def build():
        if args.config4:
            share_reqs[:] = c4_share(ip, rank, device=pdev)
            return collate_requests(share_reqs)                   # (the padded batch: shapes / token counts for the report)
        return vqa_request(ip, rank, device=pdev)
    if not host_pre:
        build()                                                   # warm-up (first launch of the preprocessing kernels)
        torch.cuda.synchronize()
    t0 = time.perf_counter()
    inputs = build()
    if host_pre:
        inputs["pixel_values"] = processor._to_device(inputs["pixel_values"])
    torch.cuda.synchronize()
    host_pre_ms = (time.perf_counter() - t0) * 1e3
    B, S = inputs["input_ids"].shape
    n_img = int((np.asarray(inputs["input_ids"]) < 0).sum())
    n_crops = int(sum(h * w + 1 for h, w in (np.asarray(inputs["image_sizes"]) // 336).tolist()))
    max_tokens = 2 * (args.warmup + args.steps) + 8

    def barrier():
        if world > 1:
            dist.barrier()
        torch.cuda.synchronize()

    # ---- prefill (ViT + projector + decoder prefill + lm_head + argmax + sync)
    prefill_ms = []
    n_warm = 2      # untimed: the first sight of a geometry runs eager, the second captures the vision tower's graph
    for rep in range(args.prefill_reps + n_warm):
        barrier()
        t0 = time.perf_counter()
        pre = None
        if args.config4 and not os.environ.get("P3V_C4_PADDED"):
            from phi_3_vision_mlx_amd.dist import prefill_requests
            pre = prefill_requests(model, share_reqs, max_tokens)    # length-bucketed prefill into one decode batch (no pad rows)
        if pre is not None:
            token, cache, _ = pre
        else:
            logits, cache = model(**inputs, max_tokens=max_tokens)
            token = ops.argmax(logits[:, -1, :].contiguous())[:, None]
        first = token.tolist()
        dt = (time.perf_counter() - t0) * 1e3
        if rep >= n_warm:
            prefill_ms.append(dt)
    prefill = float(np.median(prefill_ms))
    print("prefill reps ms:", [round(v, 1) for v in prefill_ms], file=sys.stderr)

    # ---- decode, the reference-defined rate FIRST (the K steps that follow the prefill, as phi_3_vision_mlx.py:390-403 times them):
    #      W untimed steps, then K steps through `_generate`'s own loop -- the step's tokens read per step (the reference's mx.eval),
    #      Streamer, TokenStopper, detokenisation in Streamer.end() inside the span
    streamer = api.Streamer(processor, False, True)
    stopper = api.TokenStopper(processor, B)
    for _ in range(args.warmup):
        logits, token = model.greedy_step(token, cache)
    barrier()
    t0 = time.perf_counter()
    streamer(api._rows(token))
    token = api.greedy_loop(model, token, cache, args.steps, streamer, stopper)   # (EOS from random weights: not expected)
    _, gen_len = streamer.end()
    barrier()
    gen_elapsed = time.perf_counter() - t0
    gen_tps = (gen_len - 1) / gen_elapsed

    # ---- the same number of steps as bare graph replays (device rate: no host work between replays; K keys further into the cache)
    for _ in range(args.warmup):
        logits, token = model.greedy_step(token, cache)
    barrier()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        logits, token = model.greedy_step(token, cache)
    barrier()
    elapsed = time.perf_counter() - t0
    local_elapsed = elapsed                                        # this rank's own span (the reported one is the max over ranks)
    # ---- how repeatable is that span?  (20 driver-timed steps are a 35 ms region, ~1 % of run-to-run noise.)  The same K
    #      replays again, REWOUND to the same cache offset each time (same context, same bytes), until >= 0.25 s have been timed in all
    #      (3 .. 40 regions); `steps` / `ms_per_step` / `value` above keep describing the one contracted region, the spread goes beside it.
    st_ = cache[0].state
    rep_ms = [elapsed / args.steps * 1e3]
    total_s = elapsed
    n_regions = int(min(40, max(3, np.ceil(0.25 / max(elapsed, 1e-6)))))
    if world > 1:                                                 # (every rank runs the same number of bracketed regions)
        nr = torch.tensor([n_regions], device="cpu" if share else dev)
        dist.all_reduce(nr, op=dist.ReduceOp.MAX)
        n_regions = int(nr.item())
    while len(rep_ms) < n_regions:
        cache[0].offset = st_.offset - args.steps                   # (the graph re-synchronises its device-side length: model.greedy_step)
        barrier()
        t0 = time.perf_counter()
        for _ in range(args.steps):
            logits, token = model.greedy_step(token, cache)
        barrier()
        dt = time.perf_counter() - t0
        total_s += dt
        rep_ms.append(dt / args.steps * 1e3)
    if world > 1:
        t = torch.tensor([elapsed, prefill, gen_elapsed], device="cpu" if share else dev)
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed, prefill, gen_elapsed = t.tolist()
        gen_tps = (gen_len - 1) / gen_elapsed
        hist = cache[0].state.graphs["greedy"]["history"]
        hist = hist.cpu() if share else hist.to(dev)                # (the graph keeps it in pinned host memory)
        gathered = [torch.empty_like(hist) for _ in range(world)] if rank == 0 else None
        dist.gather(hist, gathered, dst=0)                        # token gather over RCCL (request boundary only)
    tokens_per_s = world * B * args.steps / elapsed                # device rate: K graph replays between two syncs
    rccl = None
    if world > 1:                                                 # how many ranks really joined, counted on DEVICE tensors over RCCL
        one = torch.ones(1, device="cpu" if share else dev)
        dist.all_reduce(one)
        per_rank = [torch.zeros(1, device="cpu" if share else dev) for _ in range(world)]
        dist.all_gather(per_rank, torch.tensor([B * args.steps / local_elapsed], device="cpu" if share else dev))
        rccl = {"backend": dist.get_backend(), "ranks": int(one.item()), "world_size": dist.get_world_size(),
                "per_rank_tokens_per_s": [round(float(t.item()), 2) for t in per_rank]}

    # ---- roofline of the dominant decode kernel (gate_up GEMV + fused RMSNorm + SiLU*up): the 32 layers' launches
    #      replayed as one hipGraph on the launch stream (exactly the launches of a B = 1 decode step, weights of every
    #      layer in turn so nothing is cache-resident), HIP events around the replay
    I, H, L = cfg.intermediate_size, cfg.hidden_size, cfg.num_hidden_layers
    wbytes = 1 if model.w8 else 2
    alg_bytes = 2 * I * H * wbytes                                # [2I, H] weights (bf16, or e4m3 under --config5) streamed once per launch
    xb = torch.randn((1, H), device=dev).to(torch.bfloat16)
    ab = torch.empty((1, I), dtype=torch.bfloat16, device=dev)

    def gate_up_all_layers():
        for i in range(L):
            k, nw = f"model.layers.{i}.mlp.gate_up_proj.weight", model.w[f"model.layers.{i}.post_attention_layernorm.weight"]
            if model.w8:
                ops.gemv_fp8(xb, *model.w8[k], ops.EPI_SILU_MUL, norm_w=nw, norm_eps=cfg.rms_norm_eps, out=ab)
            else:
                ops.gemv(xb, model.w[k], ops.EPI_SILU_MUL, norm_w=nw, norm_eps=cfg.rms_norm_eps, out=ab)
    side = torch.cuda.Stream(device=dev)
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        gate_up_all_layers()
        gr = ops.Graph()
        gr.begin()
        gate_up_all_layers()
        gr.end()
        gr.launch()
        side.synchronize()
        reps = []
        for _ in range(5):
            e0, e1 = ops.Event(), ops.Event()
            e0.record()
            gr.launch()
            e1.record()
            side.synchronize()
            reps.append(e0.elapsed_ms(e1) / L)
    k_ms = float(np.median(reps))
    achieved = alg_bytes / (k_ms * 1e-3) / 1e9

    # HBM bytes per launch from the PMC passes (tools/pmc_gemv.sh: rocprofv3 --pmc FETCH_SIZE / WRITE_SIZE in separate
    # runs, FETCH_SIZE x2 on gfx950); a committed measurement, not re-collected inside the timed benchmark
    traffic = None
    try:
        if not model.w8:
            with open(os.path.join(ROOT, "profiles", PMC_TRAFFIC_FILE)) as f:
                rec = json.load(f)
            # the counters belong to ONE build of the kernel: a record taken from other sources is stale -> null
            if rec.get("kernel_source_sha16") == kernel_source_sha16():
                traffic = rec["gemv"]["hbm_bytes_per_launch_corrected"]
    except Exception:
        pass
    hd = cfg.hidden_size // cfg.num_attention_heads
    valid = int(np.asarray(inputs["mask"]).sum()) if "mask" in inputs else B * S
    kv_elt = 1 if args.config5 else 2
    kv_bytes = 2 * L * cfg.num_key_value_heads * hd * kv_elt * (valid + B * (args.warmup + args.steps // 2))
    w_bytes = sum(v.numel() * 2 for k, v in model.w.items() if k.startswith("model.layers.") or k == "lm_head.weight") \
        + sum(v[0].numel() for v in model.w8.values())
    step_s = elapsed / args.steps
    pf = prefill_flops(cfg, S, n_img, n_crops) if B == 1 else None
    if args.config4:
        workload = (f"BASELINE configs[3], one GPU's share per rank: {B} requests = {n_crops // 17} single-image VQA (2531 tokens) + "
                    f"{B - n_crops // 17} text prompts (16..256 tokens) as one left-padded batch; greedy, EOS suppressed")
        metric = "decode tokens/sec through generate()'s loop (reference-defined; bare graph replays: device_rate) + prefill ms, Phi-3-Vision bf16, batched mixed image+text generate (config 4 share)"
    else:
        workload = ("Phi-3-Vision single 336x336 image VQA (BASELINE configs[1]); 17 crops, "
                    f"{n_img} image tokens + 22 text tokens, prompt {S}, B=1 per GPU, greedy, EOS suppressed")
        metric = "decode tokens/sec through generate()'s loop (reference-defined; bare graph replays: device_rate) + prefill ms, Phi-3-Vision bf16 1-image VQA"
    if args.config5:
        workload += ("; BASELINE configs[4]: e4m3 decoder weights (per-row scales), " +
                     ("bf16 activations (weight-only)" if args.fp8_weight_only else "e4m3 activations in the prompt-sized projections (fp8 MFMA)") +
                     ", int8 KV cache")
        metric = metric.replace("bf16", "fp8 weights + int8 KV")
    out = {
        "metric": metric,
        "value": round(world * gen_tps, 2), "unit": "tokens/s", "n_gpus": world, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(gen_elapsed / args.steps * 1e3, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "value_definition": "reference-defined rate: (gen_len - 1) / gen_time over the K timed steps through _generate's loop "
                            "(api.greedy_loop) -- per-token D2H copy, Streamer, TokenStopper, detokenisation (phi_3_vision_mlx.py:390-403); the "
                            "loop runs one graph-replayed step ahead of the host, so that host work overlaps the next step; "
                            "whole-job aggregate = n_gpus x the slowest rank's rate.  Batches (B > 1, the config-4 share): gen_len counts "
                            "B tokens per step INCLUDING the B first tokens the prefill produced while gen_time starts after the prefill, "
                            "so the figure is (B * (K + 1) - 1) / gen_time -- slightly above the device rate B * K / time by construction "
                            "(phi_3_vision_mlx.py:77,401-403), not a faster step",
        "device_rate": {"tokens_per_s": round(tokens_per_s, 2), "ms_per_step": round(step_s * 1e3, 4),
                        "definition": "K further steps as back-to-back graph replays between two syncs (no per-token host work; run after the reference-defined loop, K keys deeper into the cache)",
                        "repeats": {"regions": len(rep_ms), "steps_each": args.steps, "timed_s": round(total_s, 3),
                                    "ms_per_step_median": round(float(np.median(rep_ms)), 4), "ms_per_step_min": round(min(rep_ms), 4),
                                    "ms_per_step_max": round(max(rep_ms), 4),
                                    "spread_pct": round((max(rep_ms) - min(rep_ms)) / float(np.median(rep_ms)) * 100, 2),
                                    "note": "this rank's own spans of the same K replays, rewound to the same cache offset; region 0 is the reported one"}},
        "rccl": rccl,
        "dtype": "fp8(e4m3)+int8kv" if args.config5 else "bf16", "data": "synthetic",
        "config": {"workload": workload, "parallelism": f"batch-sharded replicas x{world}", "batch_per_gpu": int(B), "tiny": bool(args.tiny)},
        "prefill_ms": round(prefill, 3), "prefill_tokens": int(valid), "preprocess_ms": round(host_pre_ms, 1),
        "preprocess": "host" if host_pre else "device",
        "decode_step_hbm": {"span": "device-rate step", "algorithmic_GB_per_token": round((w_bytes + kv_bytes) / 1e9, 3),
                            "achieved_GBps": round((w_bytes + kv_bytes) / step_s / 1e9, 1),
                            "frac_of_peak": round((w_bytes + kv_bytes) / step_s / 1e9 / HBM_PEAK_GBS, 4)},
        "roofline": {"bound": "hbm", "kernel": ("k_gemv3_f8" if model.w8 else "k_gemv3<1,1,6>") + " (RMSNorm + gate_up_proj + SiLU*up), 32 launches per B=1 step", "achieved": round(achieved, 1),
                     "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": round(achieved / HBM_PEAK_GBS, 4), "traffic": traffic,
                     "algorithmic_bytes_per_launch": alg_bytes, "avg_launch_ms": round(k_ms, 5)},
        "roofline_prefill": None if pf is None else {
            "bound": "mfma", "algorithmic_TFLOP": round(pf / 1e12, 2), "achieved": round(pf / (prefill * 1e-3) / 1e12, 1),
            "peak": MFMA_BF16_PEAK_TFLOPS, "unit": "TFLOP/s", "frac": round(pf / (prefill * 1e-3) / 1e12 / MFMA_BF16_PEAK_TFLOPS, 4),
            "peak_note": "bf16 dense MFMA peak (under --config5 the decoder projections run on the fp8 MFMA, 2x that peak; the ViT stays bf16)",
            "span": "whole prefill wall time (ViT + projector + 32 layers + lm_head + argmax + sync), not a single kernel"},
        "first_token": first, "weights_init_s": round(t_weights, 1),
    }
    if rank == 0 and not args.no_cpu_baseline and world == 1 and not args.tiny:
        out["cpu_baseline"] = cpu_baseline(model)
    elif rank == 0:
        out["cpu_baseline"] = None
    if rank == 0 and world == 1 and not args.no_configs and not (args.config4 or args.config5):
        out["configs"] = other_configs(model, processor, dev, args)
    if rank == 0:
        print(json.dumps(out), flush=True)
    if world > 1:
        dist.barrier()
        dist.destroy_process_group()


if __name__ == "__main__":
    main()
