"""Prefill and decode throughput of the hybrid decoder (Sasilorn) beside the rotary decoder at equal width, depth, feed-
forward parameters and key/value heads (random weights), through the engine: `python bench.py --hybrid`.

  prefill  engine steps of whole prompts (scheduler, input builder, eager forward, head over the last rows, sampler)
  decode   captured steps in bursts of 8 on one stream, every sequence `ctx` tokens long

`--hybrid-only NAME` runs one of the cases ("hybrid/4096/decode"; prefixes select several), for a kernel trace.
"""
import time

import torch

# width: (parallel layer, time-mix layer, rotary decoder), 4 + 4 layers against 8
SIZES = {
    2048: dict(left=(16, 4, 128, 64), right=(8, 128, 128), wkv=(32, 64), ff=8448, rotary=(16, 4, 5632)),
    4096: dict(left=(32, 8, 128, 128), right=(16, 128, 128), wkv=(64, 64), ff=21504, rotary=(32, 8, 14336)),
}
VOCAB, PAIRS = 32000, 4
PREFILL = ((1, 4096), (4, 2048))             # prompts x tokens of one step
DECODE = ((1, 1024), (32, 1024), (32, 4096))  # sequences, context


def hybrid_config(width):
    from light_vllm_amd.engine.hybrid_config import HybridModelConfig
    s = SIZES[width]
    (h, g, d, v), (rh, rd, rv), (wh, wd) = s["left"], s["right"], s["wkv"]
    mlp = {"kind": "dense", "ff": s["ff"]}
    layers = [{"type": "parallel", "mlp": mlp, "mixer": {
                  "left": {"heads": h, "kv_heads": g, "dim": d, "vdim": v, "scale": d ** -0.5},
                  "right": {"heads": rh, "dim": rd, "vdim": rv, "tau": 16.0}, "left_scale": 0.7, "right_scale": 0.7}},
              {"type": "wkv", "mlp": mlp, "mixer": {"heads": wh, "dim": wd}}] * PAIRS
    c = HybridModelConfig.from_dict({"architecture": "Sasilorn", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-5},
                                     "layers": layers})
    c.random_rank = 64
    return c


def rotary_config(width):
    from light_vllm_amd.engine.config import ModelConfig
    h, g, ff = SIZES[width]["rotary"]
    return ModelConfig(hidden_size=width, intermediate_size=ff, num_hidden_layers=2 * PAIRS, num_attention_heads=h,
                       num_key_value_heads=g, vocab_size=VOCAB)


def engine(cfg, dev, seqs, max_len, burst):
    from light_vllm_amd.engine.config import CacheConfig, SchedulerConfig
    from light_vllm_amd.engine.llm_engine import LLMEngine
    max_len = (max_len + 511) // 512 * 512
    return LLMEngine(cfg, CacheConfig(num_gpu_blocks=seqs * (max_len // 16 + 1) + 64, num_cpu_blocks=0),
                     SchedulerConfig(max_num_batched_tokens=8192, max_num_seqs=max(seqs, 1), max_model_len=max_len,
                                     use_v2_block_manager=burst > 1, num_scheduler_steps=burst), device=dev, seed=1)


def prefill(cfg, dev, prompts, n, iters=6):
    eng = engine(cfg, dev, prompts, n + 16, 1)
    gen, times = torch.Generator().manual_seed(0), []
    for it in range(iters):
        for i in range(prompts):
            eng.add_request(f"{it}.{i}", torch.randint(0, VOCAB, (n,), generator=gen).tolist(), max_tokens=1)
        torch.cuda.synchronize(dev)
        t0 = time.perf_counter()
        while eng.has_unfinished_requests():
            eng.step()
        torch.cuda.synchronize(dev)
        times.append(time.perf_counter() - t0)
    eng.shutdown()
    t = sorted(times[2:])[(iters - 2) // 2]
    return {"tokens_per_s": round(prompts * n / t, 1), "ms": round(t * 1e3, 3)}


def decode(cfg, dev, seqs, ctx, steps=64, burst=8):
    eng = engine(cfg, dev, seqs, ctx + 2 * steps + 4 * burst, burst)
    eng.step_returns_outputs = False
    gen = torch.Generator().manual_seed(0)
    for i in range(seqs):
        eng.add_request(str(i), torch.randint(0, VOCAB, (ctx,), generator=gen).tolist(), max_tokens=4 * steps)
    eng.prefill_synthetic(seed=3)
    eng.capture_decode_graphs(seqs)
    for _ in range(2):
        eng.step()
    times = []
    for _ in range(3):
        torch.cuda.synchronize(dev)
        t0 = time.perf_counter()
        for _ in range(steps // burst // 2):
            eng.step()
        torch.cuda.synchronize(dev)
        times.append((time.perf_counter() - t0) / (steps // 2))
    weights = eng.worker.model.weight_bytes()
    eng.shutdown()
    t = sorted(times)[1]
    return {"tokens_per_s": round(seqs / t, 1), "ms_per_step": round(t * 1e3, 4), "weight_bytes": weights}


def run(dev, only=None):
    torch.cuda.set_device(dev)
    import light_vllm_amd  # noqa: F401
    out = {}
    for width in SIZES:
        for kind, cases, fn in (("prefill", PREFILL, prefill), ("decode", DECODE, decode)):
            for a, b in cases:
                for model, make in (("hybrid", hybrid_config), ("rotary", rotary_config)):
                    name = f"{model}/{width}/{kind}/{a}x{b}"
                    if only and not name.startswith(only):
                        continue
                    out[name] = fn(make(width), dev, a, b)
                    print(name, out[name], flush=True)
                    torch.cuda.empty_cache()
    return out
