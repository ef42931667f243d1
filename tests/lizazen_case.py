"""Small Lizazen models for the tests: configurations and random weights (scores of a few units, so that single keys carry
most of a softmax row; caps, sinks, limits and decays that matter)."""
import functools

import torch

from layered_case import tokens
from oracle import lizazen


def rot(dims, base, scaling=None):
    out = {"dims": dims, "base": base}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def plain(heads, kv_heads, dim, window, r, scale, softcap):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": window}, "rot": r,
                         "scale": scale, "softcap": softcap}


def diff(heads, kv_heads, dim, vdim, window, keep, r, scale, d):
    return "attention_2", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                           "mask": {"size": window, "keep_first": keep}, "rot": r, "scale": scale, "diff": d}


def both(heads, kv_heads, dim, vdim, chunk, r, scale, rheads, rdim, rvdim, rr, decay):
    return "parallel", {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "rot": r, "scale": scale},
        "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "rot": rr, "decay": decay}}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, shared_ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared_ff}}


def model(vocab, width, eps, bigram, layers):
    return {"architecture": "Lizazen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))},
            "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}


CONFIGS = {
    # every kind of layer, one without a feed-forward, several experts per token, windows and chunks that share no factor
    "all": model(176, 96, 1e-4, (97, 5, 3), [
        (plain(3, 1, 40, 33, rot(24, 5e3, (4.0, 1.0, 3.0, 64)), 0.3, 4.0), dense(72, 0.8)),
        (diff(4, 2, 24, 40, 21, 3, rot(24, 3e4), 0.25, 0.4), moe(7, 3, 24, 56)),
        (both(4, 4, 32, 16, 19, rot(8, 777.0), 0.3, 3, 24, 40, rot(16, 2e4), [0.8, 0.97, 0.998]), None),
        (diff(2, 2, 32, 32, 16, 17, rot(16, 1e3), 0.2, 0.1), dense(40, 2.5)),
        (plain(2, 2, 16, 50, rot(16, 1e5), 0.4, 9.0), moe(4, 1, 40, 24))]),
    # nothing is a multiple of a vector or a tile
    "odd": model(131, 90, 1e-6, (50, 1, 0), [
        (both(3, 1, 13, 21, 7, rot(6, 300.0), 0.4, 2, 11, 9, rot(10, 50.0), [0.5, 1.0]), dense(33, 1.1)),
        (plain(5, 5, 10, 17, rot(2, 60.0, (2.0, 0.5, 6.0, 40)), 0.5, 3.0), moe(5, 2, 19, 45)),
        (diff(3, 1, 7, 11, 2, 1, rot(6, 1e4), 0.6, 0.7), dense(51, 0.6))]),
    # sizes of the matrix-core bodies, many experts, kept tokens past a tile's end
    "mfma": model(320, 192, 1e-5, (1000, 31, 17), [
        (diff(8, 2, 64, 128, 48, 70, rot(64, 2e4), 0.15, 0.3), dense(64, 1.0)),
        (both(8, 2, 64, 96, 40, rot(32, 1e4), 0.15, 4, 64, 64, rot(64, 1e4), [0.9, 0.99, 0.999, 0.75]), dense(256, 1.7)),
        (plain(16, 2, 96, 100, rot(96, 1e6, (8.0, 1.0, 4.0, 128)), 0.12, 20.0), moe(8, 2, 96, 32)),
        (diff(3, 3, 32, 64, 64, 4, rot(32, 5e4), 0.2, 0.6), moe(70, 5, 64, 160))]),
    # sizes past the matrix-core bodies, values in several slices, one head of each
    "large": model(208, 128, 1e-5, (300, 2, 9), [
        (both(2, 1, 272, 48, 64, rot(100, 1e4), 0.07, 2, 144, 200, rot(144, 1e4), [0.95, 0.9995]), dense(96, 1.3)),
        (diff(1, 1, 160, 272, 80, 8, rot(64, 1e4), 0.1, 0.2), moe(3, 3, 32, 96)),
        (plain(1, 1, 256, 30, rot(256, 1e4), 0.08, 6.0), dense(160, 1.0)),
        (both(1, 1, 64, 256, 33, rot(64, 1e4), 0.15, 5, 64, 136, rot(32, 1e3), [0.6, 0.7, 0.8, 0.9, 0.99]), None)]),
}


def attention_weights(put, lin, q, kind, m, width):
    """A score is scale * (q . k): a spread of 2 to 3."""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    maps = 2 if kind == "diff" else 1
    gain = (2.5 / (m["scale"] * d ** 0.5)) ** 0.5
    lin(q + "q", H * maps * d, width, gain)
    lin(q + "k", G * maps * d, width, 1.0 if kind == "plain" else gain)
    if kind != "plain":
        lin(q + "v", G * m["vdim"], width)
    lin(q + "o", width, H * m["vdim"])
    if kind != "diff":
        for s, n in (("q", H * d), ("k", G * d), ("o", width)) + ((("v", G * m["vdim"]),) if kind == "chunk" else ()):
            put(f"{q}{s}.b", (n,), 0.3)
    if kind == "plain":
        put(q + "q.norm", (H * d,), 0.3 * gain, gain)
        put(q + "k.norm", (G * d,), 0.3 * gain, gain)
        put(q + "sink", (H,), 1.0, 2.0)
    if kind == "diff":
        for s in ("lq1", "lk1", "lq2", "lk2"):
            put(q + s, (d,), 0.5 * d ** -0.25)


def random_weights(cfg, seed=0):
    """bfloat16-representable float32 tensors by name."""
    gen = torch.Generator().manual_seed(seed)
    width, out = cfg["width"], {}

    def put(name, shape, std=1.0, mean=0.0):
        out[name] = (mean + std * torch.randn(shape, generator=gen)).bfloat16().float()

    def lin(name, n, k, gain=1.0):
        put(name, (n, k), gain * k ** -0.5)
    put("embed", (cfg["vocab"], width))
    put("bigram", (cfg["embedding"]["bigram"]["buckets"] + 1, width), 0.7)
    lin("head", cfg["vocab"], width)
    put("final.norm", (width,), 0.2, 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] is not None else ()):
            put(p + n, (width,), 0.2, 1.0)
        if l["type"] == "parallel":
            attention_weights(put, lin, p + "mix.left.", "chunk", m["left"], width)
            r, q = m["right"], p + "mix.right."
            for s, n in (("q", r["dim"]), ("k", r["dim"]), ("v", r["vdim"]), ("g", r["vdim"])):
                lin(q + s, r["heads"] * n, width)
            lin(q + "o", width, r["heads"] * r["vdim"])
            put(p + "mix.left.out", (width,), 0.2, 1.0)
            put(p + "mix.right.out", (width,), 0.2, 1.0)
        else:
            attention_weights(put, lin, p + "mix.", "plain" if l["type"] == "attention" else "diff", m, width)
        f = l["mlp"]
        if f is None:
            continue
        names = [("", f["ff"])] if f["kind"] == "dense" else [(f"e{j}.", f["expert"]["ff"]) for j in range(f["router"]["experts"])]
        if f["kind"] == "moe":
            names.append(("shared.", f["shared"]["ff"]))
            lin(p + "mlp.router", f["router"]["experts"], width, 2.0)
        for e, ff in names:
            lin(f"{p}mlp.{e}gate", ff, width, 1.5)
            lin(f"{p}mlp.{e}up", ff, width, 1.5)
            lin(f"{p}mlp.{e}down", width, ff)
    return out


@functools.lru_cache(maxsize=None)
def case(name, seed=0):
    cfg = CONFIGS[name]
    return cfg, random_weights(cfg, seed)


@functools.lru_cache(maxsize=None)
def expected(name, n, seed):
    """(tokens, float64 logits) of a random sequence."""
    cfg, w = case(name)
    t = tokens(cfg, n, seed)
    return t, lizazen.forward(cfg, w, t)


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))
