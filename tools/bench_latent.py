"""Prefill and decode throughput of the latent decoder (Lepalorn) beside the rotary decoder at equal width, depth and active
feed-forward parameters per token (random weights), through the engine: `python bench.py --latent`.  Prefill and decode are
measured as tools/bench_hybrid.py does.

`--latent-only NAME` runs one of the cases ("latent/4096/decode"; prefixes select several), for a kernel trace.
"""
import torch

from bench_hybrid import DECODE, PREFILL, VOCAB, decode, prefill

LAYERS = 8
# width: attention (heads, dim, rot_dim, vdim, kv_rank), experts (number, top, ff, shared ff), rotary (heads, kv heads, ff)
SIZES = {
    2048: dict(attn=(16, 128, 64, 128, 512), moe=(64, 6, 1408, 2816), rotary=(16, 4, 11264)),
    4096: dict(attn=(32, 128, 64, 128, 512), moe=(32, 4, 2048, 6144), rotary=(32, 8, 14336)),
}
WINDOW = 4096


def latent_config(width):
    """Four layers with a cache of their own, four that read one of them."""
    from light_vllm_amd.engine.latent_config import LatentModelConfig
    (h, d, r, v, rank), (n, top, ff, shared) = SIZES[width]["attn"], SIZES[width]["moe"]
    layers = []
    for i in range(LAYERS):
        m = {"heads": h, "dim": d, "rot_dim": r, "vdim": v, "kv_rank": rank, "scale": (d + r) ** -0.5,
             "rot": {"dims": r, "base": 10000.0}, "mask": {"size": WINDOW}}
        if i % 2:
            m["kv_from"] = i - 1
        layers.append({"type": "latent_attention", "mixer": m, "mlp": {
            "kind": "moe", "router": {"experts": n, "top": top}, "expert": {"ff": ff, "limit": 7.0},
            "shared": {"ff": shared, "limit": 7.0}}})
    return LatentModelConfig.from_dict({"architecture": "Lepalorn", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-5},
                                        "embedding": {"scale": 1.0}, "layers": layers})


def rotary_config(width):
    from light_vllm_amd.engine.config import ModelConfig
    h, g, ff = SIZES[width]["rotary"]
    return ModelConfig(hidden_size=width, intermediate_size=ff, num_hidden_layers=LAYERS, num_attention_heads=h,
                       num_key_value_heads=g, vocab_size=VOCAB)


def run(dev, only=None):
    torch.cuda.set_device(dev)
    import light_vllm_amd  # noqa: F401
    out = {}
    for width in SIZES:
        for kind, cases, fn in (("prefill", PREFILL, prefill), ("decode", DECODE, decode)):
            for a, b in cases:
                for model, make in (("latent", latent_config), ("rotary", rotary_config)):
                    name = f"{model}/{width}/{kind}/{a}x{b}"
                    if only and not name.startswith(only):
                        continue
                    out[name] = fn(make(width), dev, a, b)
                    print(name, out[name], flush=True)
                    torch.cuda.empty_cache()
    return out
