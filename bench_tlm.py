"""`python bench.py --workload tlm`: prefill and decode throughput of the token language models at layer shapes of a real model (random
weights), beside the Moshi temporal transformer of the same width stepped by its own engine.

One JSON line.  `value` = decoded tokens/s of the largest size at 64 sequences; `sizes` holds, per size, prompt tokens/s (one prompt of
2048 tokens per step) and decoded tokens/s (1, 16 and 64 sequences 2048 tokens deep), each with the bytes it must move (weights that the
step's tokens reach, cache in the windows, recurrent state) or the products it must form, and the fraction of the 8 TB/s / 2.5 PFLOP/s
that is; `moshi` the temporal transformer's step at equal width, layer count and batch.  `--tlm-design bibapel`: that design, and beside it
(`kesirax`) the other one at equal width and layer count.
"""
from __future__ import annotations

import json
import time

import torch

from bench_lm import HBM_PEAK_GBS

MFMA_PEAK = 2.5e15
DEPTH = 2048
PREFILL = 2048


def sizes():
    from moshi_amd.config import LatentAttentionConfig, MinGRUConfig, MoEConfig, TokenLayerConfig, TokenLMConfig

    def model(width, gru, heads, q_rank, kv_rank, window, experts, top, ff, vocab=32000):
        att = LatentAttentionConfig(heads=heads, dim=128, vdim=128, rot_dim=64, q_rank=q_rank, kv_rank=kv_rank, scale=192 ** -0.5, rot_base=1e6, window=window)
        moe = MoEConfig(experts=experts, top=top, ff=ff)
        kinds = [MinGRUConfig(gru), MinGRUConfig(gru), att, att, MinGRUConfig(gru), MinGRUConfig(gru)]
        return TokenLMConfig("Kesirax", vocab=vocab, width=width, layers=[TokenLayerConfig(k, moe) for k in kinds], norm_groups=4, loop_start=1, loop_stop=3,
                             loop_times=2)
    return {"1024": model(1024, 1280, 8, 512, 128, 1024, 8, 1, 2048), "2048": model(2048, 2560, 16, 1024, 256, 1024, 16, 2, 2048),
            "4096": model(4096, 5120, 32, 1536, 512, 2048, 8, 2, 5632)}


def bibapel_sizes():
    from moshi_amd.config import (BigramConfig, ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LightningConfig, TokenLayerConfig, TokenLMConfig)

    def model(width, ff, window, vocab=32000):
        n = width // 128
        delta = ChannelDeltaConfig(heads=n, kv_heads=n, dim=128, vdim=128, conv=4, decay_rank=128, gate_rank=128)
        att = GroupedAttentionConfig(heads=n, kv_heads=n // 4, dim=128, vdim=128, scale=128 ** -0.5, window=window, keep_first=4, sink=True)
        light = LightningConfig(heads=n, dim=128, vdim=128, decay=[1 - 2.0 ** (-1 - 8 * i / n) for i in range(n)])
        return TokenLMConfig("Bibapel", vocab=vocab, width=width, layers=[TokenLayerConfig(k, DenseGLUConfig(ff=ff, limit=7.0)) for k in (delta, att, light, light, delta, att)],
                             loop_start=0, loop_stop=2, loop_times=2, loop_inject="project", norms=2, layer_scales=False, tied_head=True,
                             bigram=BigramConfig(buckets=65521, mul_prev=40503, mul_cur=9176), max_positions=8192)
    return {"1024": model(1024, 2816, 1024), "2048": model(2048, 5632, 1024), "4096": model(4096, 11264, 2048)}


def layer_costs(cfg, B, depth, T_per_seq=1):
    """(bytes, products) of one step of B sequences x T tokens at `depth`: weights once per execution, experts as far as the tokens can
    reach them, keys inside the window, state."""
    from moshi_amd.config import ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LatentAttentionConfig, LightningConfig
    D, n = cfg.width, B * T_per_seq
    nbytes, flops = 2 * cfg.vocab * D + n * D * 2, 2 * cfg.vocab * D * B
    for i in cfg.layer_runs:
        layer = cfg.layers[i]
        m = layer.mixer
        if isinstance(m, LatentAttentionConfig):
            w = D * (m.q_rank + m.kv_rank + m.rot_dim + m.heads) + m.q_rank * m.heads * (m.dim + m.rot_dim) + m.kv_rank * m.heads * (m.dim + m.vdim) + D * m.heads * m.vdim
            keys = min(depth + T_per_seq, m.window) if m.window else depth + T_per_seq
            nbytes += 2 * w + B * 2 * keys * (2 * m.kv_rank + m.rot_dim)
            flops += 2 * w * n + 2 * n * min(keys, depth + T_per_seq / 2) * m.heads * (2 * m.kv_rank + m.rot_dim)
        elif isinstance(m, GroupedAttentionConfig):
            w = D * (m.heads * (m.dim + m.vdim) + m.kv_heads * (m.dim + m.vdim))
            keys = min(depth + T_per_seq, m.window + m.keep_first) if m.window else depth + T_per_seq
            nbytes += 2 * w + B * 2 * keys * m.kv_heads * (m.dim + m.vdim)
            flops += 2 * w * n + 2 * n * min(keys, depth + T_per_seq / 2) * m.heads * (m.dim + m.vdim)
        elif isinstance(m, (ChannelDeltaConfig, LightningConfig)):
            if isinstance(m, LightningConfig):
                w = D * m.heads * (2 * m.dim + 3 * m.vdim)
            else:
                w = D * (2 * m.kv_heads * m.dim + 2 * m.heads * m.vdim + m.heads + m.decay_rank + m.gate_rank) + m.heads * (m.dim * m.decay_rank + m.vdim * m.gate_rank)
            nbytes += 2 * w + B * 8 * m.heads * m.dim * m.vdim
            flops += 2 * w * n + 4 * n * m.heads * m.dim * m.vdim
        else:
            w = 4 * D * m.width
            nbytes += 2 * w + B * 8 * m.width
            flops += 2 * w * n
        if isinstance(layer.mlp, DenseGLUConfig):
            nbytes += 2 * 3 * D * layer.mlp.ff
            flops += 2 * 3 * D * layer.mlp.ff * n
        elif layer.mlp is not None:
            e = layer.mlp
            reached = e.experts * (1 - (1 - e.top / e.experts) ** n)
            nbytes += 2 * 2 * D * e.ff * reached
            flops += 2 * 2 * D * e.ff * e.top * n
    if cfg.loop_inject == "project":
        nbytes += cfg.loop_times * 4 * D * D
        flops += cfg.loop_times * 4 * D * D * n
    return nbytes, flops


def timed(fn, steps, warmup, dev):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize(dev)
    t0 = time.perf_counter()
    for _ in range(steps):
        fn()
    torch.cuda.synchronize(dev)
    return (time.perf_counter() - t0) / steps


def bench_model(cfg, dev, steps, warmup, batches=(1, 16, 64), dtype=torch.bfloat16, launch_lists=None, tag=""):
    from moshi_amd.tlm import TokenLM
    from moshi_amd.weights import random_token_lm_state_dict
    sd = random_token_lm_state_dict(cfg, seed=1, device=dev)
    maxb = max(batches)
    lm = TokenLM(sd, cfg, device=dev, dtype=dtype, max_slots=maxb, max_tokens=(maxb + 1) * (DEPTH + 512), max_step_tokens=max(PREFILL, maxb))
    del sd
    torch.cuda.empty_cache()
    gen = torch.Generator().manual_seed(0)
    prompt = torch.randint(0, cfg.vocab, (PREFILL,), generator=gen).tolist()
    out = {"weight_gb": round(lm.info(6) / 1e9, 3), "decode": {}}

    def dump(name):
        if launch_lists:
            from pathlib import Path
            Path(launch_lists).mkdir(parents=True, exist_ok=True)
            (Path(launch_lists) / f"launch_list_tlm_{tag}_{name}.tsv").write_text("".join(f"{s}\t{k}\t{b}\n" for s, k, b in lm.launch_list()))

    one = torch.empty((1, cfg.vocab), dtype=torch.float32, device=dev)

    def prefill():
        s = lm.open()
        lm.step([(s, prompt, [PREFILL - 1])], out=one)
        lm.close(s)
    dt = timed(prefill, max(4, steps // 2), max(2, warmup // 2), dev)
    dump("prefill")
    nb, fl = layer_costs(cfg, 1, 0, PREFILL)
    out["prefill"] = {"tokens": PREFILL, "ms": 1e3 * dt, "tokens_per_s": PREFILL / dt, "tflop_per_s": fl / dt / 1e12, "mfma_frac": fl / dt / MFMA_PEAK}
    for B in batches:
        slots = [lm.open() for _ in range(B)]
        for s in slots:
            lm.step([(s, prompt, [])])
        logits = torch.empty((B, cfg.vocab), dtype=torch.float32, device=dev)
        lm.sample(lm.step([(s, [i % cfg.vocab], [0]) for i, s in enumerate(slots)], out=logits), slots)

        def decode():
            lm.step([(s, [-1], [0]) for s in slots], out=logits)
            lm.sample(logits, slots)
        dt = timed(decode, steps, warmup, dev)
        dump(f"decode{B}")
        nb, _ = layer_costs(cfg, B, DEPTH)
        out["decode"][str(B)] = {"ms": 1e3 * dt, "tokens_per_s": B / dt, "gb_per_step": nb / 1e9, "gb_per_s": nb / dt / 1e9, "hbm_frac": nb / dt / 1e9 / HBM_PEAK_GBS}
        for s in slots:
            lm.close(s)
    return out


def bench_moshi(width, layers, dev, steps, warmup, batches, launch_lists=None):
    """The temporal transformer alone (no depth transformer), same width, layer count, ring depth and batch."""
    from moshi_amd.config import LMConfig
    from moshi_amd.lm import LMGen, LMModel
    from moshi_amd.weights import random_lm_state_dict
    out = {}
    for B in batches:
        cfg = LMConfig(dim=width, num_heads=width // 128, num_layers=layers, context=3000, n_q=8, dep_q=0, delays=[0] * 9)
        lm = LMModel(random_lm_state_dict(cfg, seed=2, device=dev), cfg, device=dev, max_batch=B)
        gen = LMGen(lm, use_sampling=False)
        gen.streaming_forever(B)
        codes = torch.randint(0, cfg.card, (B, 8, 1), device=dev)
        for _ in range(3):
            gen.step(codes)
        gen.seek([DEPTH] * B)
        dt = timed(lambda: gen.step(codes), steps, warmup, dev)
        if launch_lists:
            from pathlib import Path
            from moshi_amd import _capi
            ll = _capi.launch_list(lambda b, n: lm._lib.mmi_lm_launch_list(lm._handle, b, n), with_bytes=True)
            (Path(launch_lists) / f"launch_list_moshi_{width}_decode{B}.tsv").write_text("".join(f"{s}\t{k}\t{b}\n" for s, k, b in ll))
        h = cfg.ffn_hidden
        nb = 2 * (layers * (4 * width * width + 3 * h * width) + cfg.text_card * width) + B * layers * 2 * 2 * width * DEPTH
        out[str(B)] = {"ms": 1e3 * dt, "tokens_per_s": B / dt, "gb_per_step": nb / 1e9, "gb_per_s": nb / dt / 1e9, "hbm_frac": nb / dt / 1e9 / HBM_PEAK_GBS}
        del gen, lm
        torch.cuda.empty_cache()
    return out


def main(args, dev):
    res = {}
    batches = tuple(int(b) for b in args.tlm_batches.split(","))
    bibapel = args.tlm_design == "bibapel"
    for name, cfg in (bibapel_sizes() if bibapel else sizes()).items():
        if args.tlm_size and name not in args.tlm_size.split(","):
            continue
        res[name] = bench_model(cfg, dev, args.steps, args.warmup, batches, launch_lists=args.launch_lists, tag=("bibapel_" if bibapel else "") + name)
        if not args.no_extras and bibapel:
            res[name]["kesirax"] = bench_model(sizes()[name], dev, args.steps, args.warmup, batches, launch_lists=args.launch_lists, tag=name)
        if not args.no_extras:
            res[name]["moshi"] = bench_moshi(cfg.width, len(cfg.layer_runs), dev, args.steps, args.warmup, batches, args.launch_lists)
    last = list(res)[-1]
    d = res[last]["decode"][str(batches[-1])]
    print(json.dumps({"metric": "decoded tokens/s, token language model", "value": d["tokens_per_s"], "unit": "tokens/s", "n_gpus": 1, "steps": args.steps,
                      "warmup": args.warmup, "ms_per_step": d["ms"], "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16",
                      "data": "synthetic", "config": {"model": f"{cfg.architecture}, width {last}, random weights", "global_batch": batches[-1], "seq_len": DEPTH,
                                                      "parallelism": "dp1"}, "sizes": res}), flush=True)
