"""Prefill and decode throughput of the stream decoder (Susalorn) beside the latent decoder (Lepalorn) at equal width, depth,
latents and feed-forward parameters per token (random weights), through the engine: `python bench.py --stream`.  Prefill and decode
are measured as tools/bench_hybrid.py does.  The latent decoder's window holds the whole context, so that both models' attention
reads all keys.

`--stream-only NAME` runs one of the cases ("stream/4096/decode"; prefixes select several), for a kernel trace; the hybrid decoder,
whose recurrence is the nearest to the delta rule, is "hybrid/..." there.
"""
import torch

from bench_hybrid import DECODE, PREFILL, VOCAB, decode, prefill

LAYERS = 8
# width: attention (heads, dim, rot_dim, vdim, kv_rank, q_rank), delta rule (heads, dim, rank), experts (number, top, ff, groups,
# kept), dense ff; the latent decoder's experts (number, top, ff, shared ff)
SIZES = {
    2048: dict(attn=(16, 128, 64, 128, 512, 1536), delta=(16, 128, 128), moe=(64, 6, 2816, 8, 4), ff=11264,
               latent=(64, 6, 1408, 2816)),
    4096: dict(attn=(32, 128, 64, 128, 512, 1536), delta=(32, 128, 128), moe=(32, 4, 5376, 4, 2), ff=14336,
               latent=(32, 4, 2048, 6144)),
}
WINDOW, STREAMS = 8192, 4


def stream_config(width):
    """One dense layer, then mixtures; delta-rule layers and latent attention in turn."""
    from light_vllm_amd.engine.stream_config import StreamModelConfig
    s = SIZES[width]
    (h, d, r, v, rank, q_rank), (dh, dd, low), (n, top, ff, groups, keep) = s["attn"], s["delta"], s["moe"]
    latent = {"type": "latent_attention", "mixer": {
        "heads": h, "dim": d, "rot_dim": r, "vdim": v, "kv_rank": rank, "q_rank": q_rank, "scale": (d + r) ** -0.5,
        "rot": {"dims": r, "base": 10000.0, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}
    delta = {"type": "channel_delta", "mixer": {"heads": dh, "kv_heads": dh, "dim": dd, "vdim": dd, "conv": 4}}
    moe = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": n, "top": top, "groups": {"count": groups, "keep": keep}, "scale": 2.5}}
    layers = [{**(latent if i % 2 else delta), "mlp": moe if i else {"kind": "dense", "ff": s["ff"]}} for i in range(LAYERS)]
    c = StreamModelConfig.from_dict({"architecture": "Susalorn", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-5},
                                     "streams": STREAMS, "loop": None, "layers": layers})
    c.random_rank = low
    return c


def latent_config(width):
    from bench_latent import latent_config
    from dataclasses import replace
    cfg = latent_config(width)
    cfg.layers = [replace(l, mixer=replace(l.mixer, kv_from=None, window=WINDOW)) for l in cfg.layers]
    return cfg


def run(dev, only=None):
    torch.cuda.set_device(dev)
    import light_vllm_amd  # noqa: F401
    from bench_hybrid import hybrid_config
    models = [("stream", stream_config), ("latent", latent_config)] + ([("hybrid", hybrid_config)] if only else [])
    out = {}
    for width in SIZES:
        for kind, cases, fn in (("prefill", PREFILL, prefill), ("decode", DECODE, decode)):
            for a, b in cases:
                for model, make in models:
                    name = f"{model}/{width}/{kind}/{a}x{b}"
                    if only and not name.startswith(only):
                        continue
                    out[name] = fn(make(width), dev, a, b)
                    print(name, out[name], flush=True)
                    torch.cuda.empty_cache()
    return out
