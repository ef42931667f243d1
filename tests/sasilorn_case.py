"""Small Sasilorn models for the tests: configurations, random weights (every projection scaled so that single keys,
decays and tokens stand out in the logits)."""
import functools

import torch

from layered_case import error, play, portions, replay, tokens, write_model  # noqa: F401
from oracle import sasilorn


def parallel(lh, lg, ld, lv, scale, rh, rd, rv, tau, left_scale, right_scale, ff):
    return {"type": "parallel", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"left": {"heads": lh, "kv_heads": lg, "dim": ld, "vdim": lv, "scale": scale},
                      "right": {"heads": rh, "dim": rd, "vdim": rv, "tau": tau},
                      "left_scale": left_scale, "right_scale": right_scale}}


def wkv(heads, dim, ff=None):
    return {"type": "wkv", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "dim": dim}}


def model(vocab, width, eps, layers):
    return {"architecture": "Sasilorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


def tied(layer, j):
    return {**layer, "weights_of": j}


_P = parallel(6, 2, 40, 24, 0.21, 3, 24, 40, 8.0, 0.8, 1.3, 144)
_W = wkv(3, 32, 80)
_W2 = wkv(1, 64)
CONFIGS = {
    # unequal sizes everywhere, tied layers of both kinds, a parallel layer without and a time-mix layer with a feed-forward
    "tied": model(176, 96, 1e-4, [_W, _P, tied(_W, 0), parallel(5, 1, 72, 72, 0.1, 2, 16, 16, 1.0, 1.0, 1.0, None),
                                  tied(_P, 1), _W2]),
    # nothing is a multiple of a vector or a tile
    "odd": model(131, 90, 1e-6, [parallel(3, 3, 20, 33, 0.3, 1, 10, 7, 2.5, 1.7, 0.4, 51), wkv(5, 9), wkv(2, 13, 35)]),
    # sizes of the matrix-core bodies, a wide query group
    "mfma": model(320, 192, 1e-5, [parallel(20, 1, 128, 64, 0.09, 2, 64, 128, 16.0, 0.9, 0.7, 256), wkv(2, 128, 128),
                                   parallel(4, 4, 64, 128, 0.125, 2, 128, 32, 4.0, 0.5, 1.1, 64)]),
}


def random_weights(cfg, seed=0, rank=12):
    """bfloat16-representable float32 tensors by name.  Query / key norms of 1.6 make one key in hundreds carry most of a
    softmax row; decays reach from a few tokens to thousands."""
    gen = torch.Generator().manual_seed(seed)
    width, out = cfg["width"], {}

    def put(name, shape, std=1.0, mean=0.0):
        out[name] = (mean + std * torch.randn(shape, generator=gen)).bfloat16().float()

    def lin(name, n, k, gain=1.0):
        put(name, (n, k), gain * k ** -0.5)

    def norm(name):
        put(name, (width,), 0.2, 1.0)
        put(name + ".b", (width,), 0.1)
        put(name + ".alpha", (), 0.1, 0.7)
    put("embed", (cfg["vocab"], width))
    lin("head", cfg["vocab"], width)
    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}", layer["mixer"]
        norm(p + ".norm1")
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            q = p + ".mix.left."
            for s, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"]),
                         ("g", a["heads"])):
                lin(q + s, n, width, 2.0)
            lin(q + "o", width, a["heads"] * a["vdim"])
            put(q + "q.norm", (a["dim"],), 0.2, 1.6)
            put(q + "k.norm", (a["dim"],), 0.2, 1.6)
            q, n = p + ".mix.right.", r["heads"] * r["dim"]
            for s, k in (("q", n), ("k", n), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"]), ("a1", rank)):
                lin(q + s, k, width, 2.0)
            lin(q + "o", width, r["heads"] * r["vdim"])
            put(q + "norm", (r["vdim"],), 0.2, 1.0)
            lin(q + "a2", n, rank, 1.5)
            put(q + "a2.b", (n,), 2.0, 1.0)
        else:
            q, n = p + ".mix.", m["heads"] * m["dim"]
            for s in "rkvgw":
                out[f"{q}mu.{s}"] = torch.rand(width, generator=gen).bfloat16().float()
            for s in "rkvg":
                lin(q + s, n, width, 2.0)
            lin(q + "w1", rank, width, 2.0)
            lin(q + "w2", n, rank)
            put(q + "w0", (n,), 3.0, -3.0)
            put(q + "u", (m["heads"], m["dim"]), 0.8)
            put(q + "norm", (n,), 0.2, 1.0)
            lin(q + "o", width, n)
        if layer["mlp"] is not None:
            norm(p + ".norm2")
            lin(p + ".mlp.up", layer["mlp"]["ff"], width)
            lin(p + ".mlp.down", width, layer["mlp"]["ff"])
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
    return t, sasilorn.forward(cfg, w, t)
