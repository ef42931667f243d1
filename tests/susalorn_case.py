"""Small Susalorn models for the tests: configurations and random weights (scores of a few units, so that single keys carry most of
a softmax row; sinks that take a share of it; memories from a few tokens to hundreds; streams that differ)."""
import functools

import torch

from layered_case import tokens
from oracle import susalorn


def rot(dims, base, scaling=None):
    out = {"dims": dims, "base": base}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return out


def latent(heads, dim, rot_dim, vdim, rank, q_rank, scale, base=1e4, scaling=(4.0, 64, 8.0, 1.0)):
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
                                "scale": scale, "rot": rot(rot_dim, base, scaling)}


def delta(heads, kv_heads, dim, vdim, taps):
    return "channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, count, keep, scale):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale}}


def model(vocab, width, eps, streams, loop, layers):
    return {"architecture": "Susalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams,
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)),
            "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}


CONFIGS = {
    # every kind of layer, a loop in the middle, layers without a feed-forward, shared keys
    "all": model(176, 96, 1e-4, 2, (1, 4, 2), [
        (latent(3, 24, 16, 40, 48, 40, 0.21, 5e3), moe(6, 2, 40, 3, 2, 2.5)),
        (delta(4, 2, 24, 40, 4), dense(72)),
        (latent(5, 40, 24, 24, 64, 72, 0.17, 3e4, (2.0, 32, 4.0, 0.5)), None),
        (delta(3, 3, 16, 24, 3), moe(8, 3, 24, 4, 2, 1.0)),
        (latent(2, 32, 8, 32, 48, 24, 0.3, 1e3, (8.0, 512, 32.0, 1.0)), dense(40)),
        (delta(6, 1, 32, 16, 2), None)]),
    # nothing is a multiple of a vector or a tile; one stream, no loop (a large eps: small read-outs are divided by their size)
    "odd": model(131, 90, 3e-3, 1, None, [
        (delta(3, 1, 11, 9, 5), dense(33)),
        (latent(3, 13, 6, 21, 35, 19, 0.3, 777.0), moe(9, 2, 19, 3, 1, 0.7)),
        (delta(2, 2, 7, 21, 1), moe(5, 2, 45, 1, 1, 1.2)),
        (latent(1, 7, 10, 5, 22, 33, 0.4, 3e4, (16.0, 20, 2.0, 0.1)), dense(51))]),
    # sizes of the matrix-core bodies, many heads on one latent, many experts
    "mfma": model(320, 192, 1e-5, 4, (1, 3, 2), [
        (latent(20, 64, 32, 64, 128, 96, 0.11, 2e4), moe(70, 5, 64, 10, 4, 0.8)),
        (delta(8, 4, 64, 64, 4), moe(16, 4, 96, 8, 3, 1.0)),
        (latent(4, 64, 64, 128, 256, 160, 0.1), dense(128)),
        (delta(4, 4, 32, 128, 4), dense(96))]),
    # a large latent and states past the registers of a workgroup
    "large": model(208, 128, 1e-5, 5, (1, 2, 2), [
        (delta(2, 1, 144, 200, 7), moe(16, 6, 64, 4, 4, 0.5)),
        (latent(16, 128, 64, 128, 512, 320, 0.08), None),
        (delta(1, 1, 256, 264, 4), dense(160)),
        (delta(3, 3, 128, 96, 16), None)]),
    # one kind of layer alone: states without a cache, caches without a state
    "states": model(120, 64, 1e-4, 3, (0, 1, 2), [(delta(4, 4, 16, 32, 4), dense(48)), (delta(2, 1, 32, 16, 3), None)]),
    "caches": model(120, 64, 1e-4, 3, (0, 2, 2), [
        (latent(2, 16, 16, 24, 32, 24, 0.25), None), (latent(4, 24, 8, 16, 64, 40, 0.2, 5e3, None), moe(4, 1, 48, 2, 1, 1.3))]),
}


def delta_weights(put, lin, q, m, width, rank, out):
    H, G = m["heads"], m["kv_heads"]
    for s, n in (("q", G * m["dim"]), ("k", G * m["dim"]), ("v", H * m["vdim"])):
        lin(q + s, n, width)
        put(f"{q}{s}.conv", (n, m["conv"]), 0.5)
    lin(q + "b", H, width, 1.5)
    put(q + "A_log", (H,), 0.7, 0.8)
    put(q + "norm", (m["vdim"],), 0.2, 1.0)
    lin(q + "a1", rank, width)
    lin(q + "a2", H * m["dim"], rank, 1.5)
    put(q + "dt_bias", (H * m["dim"],), 2.5, -4.0)
    out[q + "dt_bias"][::13] = 20.0  # channels that forget at once
    lin(q + "g1", rank, width)
    lin(q + "g2", H * m["vdim"], rank, 2.0)
    lin(q + "o", width, H * m["vdim"], 1.5)


SPREAD = {"mfma": 1.2, "odd": 1.8}  # of the scores: many layers of sharp rows would amplify 16-bit rounding


def latent_weights(put, lin, q, m, width, spread=2.5):
    H, qd = m["heads"], m["dim"] + m["rot_dim"]
    # a score is (q . k) * scale with entries of q and k about the gains
    gain = (spread / (m["scale"] * qd ** 0.5)) ** 0.5
    lin(q + "dq", m["q_rank"], width)
    put(q + "dq.norm", (m["q_rank"],), 0.2, 1.0)
    lin(q + "uq", H * qd, m["q_rank"], gain)
    lin(q + "dkv", m["kv_rank"] + m["rot_dim"], width, gain)
    put(q + "dkv.norm", (m["kv_rank"],), 0.2, 1.0)
    lin(q + "uk", H * m["dim"], m["kv_rank"], gain)
    lin(q + "uv", H * m["vdim"], m["kv_rank"])
    put(q + "sink", (H,), 1.0, 2.0)
    lin(q + "o", width, H * m["vdim"], 1.5)


def random_weights(cfg, seed=0, spread=2.5):
    """bfloat16-representable float32 tensors by name."""
    gen = torch.Generator().manual_seed(seed)
    width, n, out = cfg["width"], cfg["streams"], {}

    def put(name, shape, std=1.0, mean=0.0):
        out[name] = (mean + std * torch.randn(shape, generator=gen)).bfloat16().float()

    def lin(name, rows, cols, gain=1.0):
        put(name, (rows, cols), gain * cols ** -0.5)
    put("embed", (cfg["vocab"], width), 0.4)
    put("final.norm", (width,), 0.2, 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, f = f"l{i}.", l["mlp"]
        for sub in (1, 2) if f is not None else (1,):
            put(f"{p}norm{sub}", (width,), 0.2, 1.0)
            put(f"{p}hc{sub}.in", (n,), 0.5 / n, 1.0 / n)
            put(f"{p}hc{sub}.out", (n,), 0.2, 0.6)
            out[f"{p}hc{sub}.mix"] = (0.7 * torch.eye(n) + 0.3 / n + 0.2 / n * torch.randn(n, n, generator=gen)).bfloat16().float()
        if l["type"] == "latent_attention":
            latent_weights(put, lin, p + "mix.", l["mixer"], width, spread)
        else:
            delta_weights(put, lin, p + "mix.", l["mixer"], width, (24, 9, 33, 64)[i % 4], out)
        if f is None:
            continue
        if f["kind"] == "dense":
            experts = [("", f["ff"])]
            lin(p + "mlp.gate", f["ff"], width, 1.5)
        else:
            experts = [(f"e{j}.", f["expert"]["ff"]) for j in range(f["router"]["experts"])]
            lin(p + "mlp.router", f["router"]["experts"], width, 2.0)
        for e, ff in experts:
            lin(f"{p}mlp.{e}up", ff, width, 1.2)
            lin(f"{p}mlp.{e}down", width, ff)
    return out


@functools.lru_cache(maxsize=None)
def case(name, seed=0):
    cfg = CONFIGS[name]
    return cfg, random_weights(cfg, seed, SPREAD.get(name, 2.5))


@functools.lru_cache(maxsize=None)
def expected(name, n, seed):
    """(tokens, float64 logits) of a random sequence."""
    cfg, w = case(name)
    t = tokens(cfg, n, seed)
    return t, susalorn.forward(cfg, w, t)


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def mixer_weights(kind, m, width, rank=24, seed=0):
    """Weights of one mixer by their names in it."""
    gen, out = torch.Generator().manual_seed(seed), {}

    def put(name, shape, std=1.0, mean=0.0):
        out[name] = (mean + std * torch.randn(shape, generator=gen)).bfloat16().float()

    def lin(name, rows, cols, gain=1.0):
        put(name, (rows, cols), gain * cols ** -0.5)
    if kind == "latent_attention":
        latent_weights(put, lin, "", m, width)
    else:
        delta_weights(put, lin, "", m, width, rank, out)
    return out
