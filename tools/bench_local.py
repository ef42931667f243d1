"""Prefill and decode throughput of the local decoder (Lizazen) beside the hybrid decoder (Sasilorn) at equal width, depth,
key/value heads and feed-forward parameters per token (random weights), through the engine: `python bench.py --local`.  Prefill
and decode are measured as tools/bench_hybrid.py does.  Windows and chunks hold the whole context, so that both models' attention
reads the same keys.

`--local-only NAME` runs one of the cases ("local/4096/decode"; prefixes select several), for a kernel trace.
"""
import torch

from bench_hybrid import DECODE, PREFILL, VOCAB, decode, prefill

# width: attention (heads, kv heads, size), retention (heads, size), ff, experts (number, top, ff, shared ff)
SIZES = {
    2048: dict(attn=(16, 4, 128), retention=(8, 128), ff=5632, moe=(32, 2, 1408, 2816)),
    4096: dict(attn=(32, 8, 128), retention=(16, 128), ff=14336, moe=(16, 2, 4096, 6144)),
}
WINDOW, KEPT = 8192, 64


def local_config(width):
    """Twice: retention beside chunks, a window with normed queries and keys, two layers of differential attention."""
    from light_vllm_amd.engine.local_config import LocalModelConfig
    s = SIZES[width]
    (h, g, d), (rh, rd), (n, top, ff, shared) = s["attn"], s["retention"], s["moe"]
    rot = {"dims": d, "base": 500000.0}
    dense = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
    moe = {"kind": "moe", "router": {"experts": n, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}
    heads = {"heads": h, "kv_heads": g, "dim": d, "vdim": d, "scale": d ** -0.5, "rot": rot, "mask": {"size": WINDOW}}
    diff = {"type": "attention_2", "mixer": {**heads, "dim": d // 2, "scale": (d // 2) ** -0.5, "diff": 0.3,
                                             "rot": {"dims": d // 2, "base": 500000.0},
                                             "mask": {"size": WINDOW, "keep_first": KEPT}}}
    right = {"heads": rh, "dim": rd, "vdim": rd, "rot": {"dims": rd, "base": 10000.0},
             "decay": [1 - 2.0 ** (-5 - 6 * i / rh) for i in range(rh)]}
    layers = [{"type": "parallel", "mixer": {"left": heads, "right": right}, "mlp": dense},
              {"type": "attention", "mlp": moe, "mixer": {**heads, "softcap": 50.0, "rot": {
                  **rot, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}},
              {**diff, "mlp": dense}, {**diff, "mlp": moe}] * 2
    return LocalModelConfig.from_dict({"architecture": "Lizazen", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-6},
                                       "embedding": {"bigram": {"buckets": 65536, "mul_prev": 31, "mul_cur": 7}},
                                       "layers": layers})


def hybrid_config(width):
    from bench_hybrid import hybrid_config
    cfg = hybrid_config(width)
    if width == 2048:  # equal key and value sizes
        from dataclasses import replace
        h, g, d = SIZES[width]["attn"]
        for i, l in enumerate(cfg.layers):
            if hasattr(l.mixer, "left"):
                cfg.layers[i] = replace(l, mixer=replace(l.mixer, left=replace(l.mixer.left, heads=h, kv_heads=g, dim=d, vdim=d)))
    return cfg


def run(dev, only=None):
    torch.cuda.set_device(dev)
    import light_vllm_amd  # noqa: F401
    out = {}
    for width in SIZES:
        for kind, cases, fn in (("prefill", PREFILL, prefill), ("decode", DECODE, decode)):
            for a, b in cases:
                for model, make in (("local", local_config), ("hybrid", hybrid_config)):
                    name = f"{model}/{width}/{kind}/{a}x{b}"
                    if only and not name.startswith(only):
                        continue
                    out[name] = fn(make(width), dev, a, b)
                    print(name, out[name], flush=True)
                    torch.cuda.empty_cache()
    return out
