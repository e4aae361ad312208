"""Throughput of a layered model (Vudelix, Lezepel) beside a Llama model of equal size, Lezepel also beside Vudelix: a
2048-position prompt pass and batch-1 decoding after it, random weights.  Run through bench.py (--workload vudelix-... or
lezepel-...)."""
import json
import time

import numpy as np

HBM_PEAK = 8e12    # bytes/s
MFMA_PEAK = 2.5e15  # dense bf16 FLOP/s


def config(name):
    """layers of the size of a real model's, dense and expert feed-forwards in turn, and the Llama shape that goes with it.
    Vudelix: three delta-rule layers to one of attention.  Lezepel: six layers, two of which run twice."""
    from . import layered as L
    W, H, G, ff, experts, top, eff, q_rank, kv_rank = {"tiny": (512, 4, 2, 1024, 8, 2, 256, 192, 128),  # for a quick functional run
                                                       "2k": (2048, 16, 4, 8192, 32, 4, 1024, 768, 512),
                                                       "4k": (4096, 32, 8, 14336, 64, 4, 2048, 1536, 512)}[name.split("-")[1]]
    layers = []
    llama = dict(dim=W, hidden_dim=ff, n_layers=8, n_heads=H, n_kv_heads=G, vocab_size=32000, seq_len=4096, rope_freq_base=500000.0)
    if name.startswith("lezepel"):
        for i in range(6):
            f = dict(ff=L.FF_DENSE, ff_dim=ff, ff_act=L.RELU) if i % 2 == 0 else \
                dict(ff=L.FF_EXPERTS, ff_dim=eff, ff_act=L.SILU, n_experts=experts, top=top, route=L.ROUTE_SOFTMAX_OUT, router_bias=True)
            layers.append(L.LayerSpec(mixer=L.LATENT, n_heads=H, n_kv_heads=H, dim=128, vdim=128, q_rank=q_rank, kv_rank=kv_rank, rot_size=64,
                                      rot_dims=64, rot_base=500000.0, rot_half=True, out_gate=True, parallel=True, ff_gated=True,
                                      scale=192 ** -0.5, **f))
        return L.LayeredConfig(width=W, vocab_size=32000, layers=layers, norm_eps=1e-5, embed_scale=16.0, loop=(2, 4, 2), seq_len=4096,
                               architecture="Lezepel"), llama
    for i in range(8):
        f = dict(ff=L.FF_DENSE, ff_dim=ff, ff_act=L.GELU_ERF) if i % 2 == 0 else \
            dict(ff=L.FF_EXPERTS, ff_dim=eff, ff_act=L.RELU2, n_experts=experts, top=top)
        if i % 4 == 3:
            m = dict(mixer=L.ATTENTION, n_heads=H, n_kv_heads=G, dim=128, vdim=128, window=1024, rot_dims=128, rot_base=500000.0,
                     qk_norm=True, head_gate=True, scale=128 ** -0.5)
        else:
            m = dict(mixer=L.CHANNEL_DELTA, n_heads=H, n_kv_heads=H, dim=128, vdim=128, taps=4, decay_rank=128, gate_rank=128)
        layers.append(L.LayerSpec(**m, **f))
    cfg = L.LayeredConfig(width=W, vocab_size=32000, layers=layers, norm_eps=1e-5, residual_mult=0.4, side_dim=256, seq_len=4096,
                          architecture="Vudelix")
    return cfg, llama


def work(cfg, n_prompt):
    """(bytes one decode step reads and writes, FLOP of the prompt pass's products and mixers)"""
    from . import layered as L
    W, by, fl = cfg.width, 0, 0
    for i in cfg.runs:
        s = cfg.layers[i]
        H, G, D, V = s.n_heads, s.n_kv_heads, s.dim, s.vdim
        if s.mixer == L.ATTENTION:
            mats = W * (H * D + G * (D + V) + H) + W * H * V
            by += 4 * min(s.window, n_prompt) * G * (D + V)
            pairs = sum(min(i + 1, s.window) for i in range(n_prompt))
            fl += 2 * pairs * H * (D + V)
        elif s.mixer == L.LATENT:
            C, R = s.kv_rank, s.rot_size
            mats = W * (s.q_rank + C + R + H * V) + s.q_rank * H * (D + R) + C * H * (D + V) + W * H * V
            by += 4 * n_prompt * (C + R)
            fl += n_prompt * (n_prompt + 1) * H * (D + R + V)
        else:
            mats = W * (2 * G * D + H * V + H + s.decay_rank + s.gate_rank) + H * (D * s.decay_rank + V * s.gate_rank) + W * H * V
            by += 2 * 4 * H * D * V
            fl += n_prompt * 7 * H * D * V
        if s.ff == L.FF_DENSE:
            mats += (3 if s.ff_gated else 2) * W * s.ff_dim
        elif s.ff == L.FF_EXPERTS:
            mats += W * s.n_experts + s.top * (3 if s.ff_gated else 2) * W * s.ff_dim
        mats += 2 * W * cfg.side_dim
        by += 2 * mats
        fl += 2 * mats * n_prompt
    return by + 2 * W * cfg.vocab_size, fl


def measure(pkg, ctx, dev, vocab, n_prompt, K, W, repeats, log):
    from . import synth
    prompt = synth.seeded_prompt(99, n_prompt, vocab)
    pf, dec, ids = [], [], None
    for rep in range(max(2, repeats)):
        dev.reset()
        ctx.sync()
        t0 = time.perf_counter()
        _, nxt = dev.prefill(prompt, 0, want_logits=False)
        pf.append(time.perf_counter() - t0)
        warm = dev.generate_greedy([nxt], W, pos0=n_prompt) if W else [nxt]
        ctx.sync()
        t0 = time.perf_counter()
        ids, ms = dev.generate_greedy([int(warm[-1])], K, pos0=n_prompt + W, timed=True)
        ctx.sync()
        dec.append(time.perf_counter() - t0)
        log("  repeat %d: prompt pass %.2f ms, %d tokens in %.2f ms (%.2f on the device)" % (rep, pf[-1] * 1e3, K, dec[-1] * 1e3, ms))
    return min(pf[1:]), float(np.median(dec)) / K, ids[:8].tolist()


def run(pkg, args, log):
    from . import synth
    name, n_prompt, K, W = args.workload, 2048, args.steps, args.warmup
    cfg, llama = config(name)
    if n_prompt + W + K > cfg.seq_len:
        raise SystemExit("steps + warmup + prompt exceed %d" % cfg.seq_len)
    ctx = pkg.default_context()
    lm = synth.layered_model(cfg)
    dev = lm.device()
    log("%s, %d layer runs of width %d" % (cfg.architecture, len(cfg.runs), cfg.width))
    pf, step, ids = measure(pkg, ctx, dev, cfg.vocab_size, n_prompt, K, W, args.repeats, log)
    dev.close()
    by, fl = work(cfg, n_prompt)
    beside = {}
    if cfg.architecture != "Vudelix":
        vcfg, _ = config("vudelix-" + name.split("-")[1])
        dev = synth.layered_model(vcfg).device()
        log("Vudelix, %d layers of width %d" % (vcfg.n_layers, vcfg.width))
        p, s, _ = measure(pkg, ctx, dev, vcfg.vocab_size, n_prompt, K, W, args.repeats, log)
        dev.close()
        v_by, v_fl = work(vcfg, n_prompt)
        beside["Vudelix"] = {"prefill_tok_s": round(n_prompt / p, 1), "prefill_TFLOP/s": round(v_fl / p / 1e12, 1), "decode_tok_s": round(1 / s, 1),
                             "decode_bytes": int(v_by), "decode_GB/s": round(v_by / s / 1e9, 1)}
    lcfg = pkg.ModelConfig(**llama)
    llm = synth.synthetic_model(lcfg, synth.PLAN_Q4_K_S, seed=20240607, norm_spread=0.0)
    kv = lcfg.dim // lcfg.n_heads * lcfg.n_kv_heads
    l_by = synth.weight_bytes_per_token(llm) + 2 * 4 * kv * lcfg.n_layers * n_prompt
    l_fl = 2 * n_prompt * lcfg.n_layers * (2 * lcfg.dim * lcfg.dim + 2 * lcfg.dim * kv + 3 * lcfg.dim * lcfg.hidden_dim) + \
        2 * lcfg.n_layers * n_prompt * (n_prompt + 1) * lcfg.dim
    for path, label in ((1, "kernel per phase"), (0, "automatic")):
        if path and args.path:
            continue
        dev = llm.device(path=path)
        log("Llama Q4_K_S, same width, heads and dense feed-forward, launch path %d" % dev.path)
        p, s, _ = measure(pkg, ctx, dev, lcfg.vocab_size, n_prompt, K, W, args.repeats, log)
        beside[label] = {"launch_path": dev.path, "prefill_tok_s": round(n_prompt / p, 1), "prefill_TFLOP/s": round(l_fl / p / 1e12, 1),
                         "decode_tok_s": round(1 / s, 1), "decode_bytes": int(l_by), "decode_GB/s": round(l_by / s / 1e9, 1)}
        dev.close()
    print(json.dumps({
        "metric": "decode tok/s, %s, batch 1, after a %d-token prompt" % (cfg.architecture, n_prompt), "value": round(1 / step, 2), "unit": "tok/s",
        "n_gpus": 1, "steps": K, "warmup": W, "ms_per_step": round(step * 1e3, 4), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16 weights, fp32 sums", "data": "synthetic",
        "config": {"workload": name, "width": cfg.width, "n_layers": cfg.n_layers, "layer_runs": len(cfg.runs), "prompt_tokens": n_prompt, "tokens_head": ids},
        "decode": {"bytes": int(by), "GB/s": round(by / step / 1e9, 1), "frac_of_hbm": round(by / step / HBM_PEAK, 4)},
        "prefill": {"ms": round(pf * 1e3, 3), "tok_s": round(n_prompt / pf, 1), "TFLOP/s": round(fl / pf / 1e12, 1),
                    "frac_of_mfma": round(fl / pf / MFMA_PEAK, 4)},
        "beside": beside}), flush=True)
