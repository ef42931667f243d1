"""Small Lepalorn models for the tests: configurations and random weights (scores of a few units, so that single keys carry
most of a softmax row; gains, limits and depth averages of their own in every layer)."""
import functools

import pytest
import torch

from layered_case import tokens
from oracle import lepalorn


def layer(heads, dim, rot, vdim, rank, window, scale, base=1e4, kv_from=None, mlp=None, rot_dims=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale,
         "rot": {"dims": rot if rot_dims is None else rot_dims, "base": base}, "mask": {"size": window}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def moe(experts, top, ff, limit, shared_ff, shared_limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit},
            "shared": {"ff": shared_ff, "limit": shared_limit}}


def model(vocab, width, eps, scale, layers):
    return {"architecture": "Lepalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


CONFIGS = {
    # caches read by later layers with other heads, sizes and windows; a layer without a feed-forward; one expert per token
    "shared": model(176, 96, 1e-4, 3.0, [
        layer(3, 24, 16, 40, 48, 33, 0.21, 5e3, mlp=moe(6, 1, 40, 1.5, 72, 0.7)),
        layer(5, 40, 16, 24, 48, 20, 0.17, 5e3, kv_from=0, mlp=moe(9, 3, 24, 2.5, 16, 3.0)),
        layer(2, 32, 8, 32, 64, 50, 0.3, 1e5),
        layer(4, 16, 16, 16, 48, 70, 0.25, 5e3, kv_from=0, mlp=moe(4, 4, 56, 1.0, 56, 1.0)),
        layer(1, 48, 8, 56, 64, 16, 0.2, 1e5, kv_from=2, mlp=moe(5, 2, 33, 0.5, 90, 2.0))]),
    # nothing is a multiple of a vector or a tile
    "odd": model(131, 90, 1e-6, 0.7, [
        layer(3, 13, 6, 21, 35, 17, 0.3, 777.0, mlp=moe(7, 2, 19, 1.1, 45, 1.7)),
        layer(1, 7, 10, 5, 22, 65, 0.4, 3e4, mlp=moe(3, 1, 51, 4.0, 7, 0.4)),
        layer(2, 9, 6, 11, 35, 2, 0.35, 777.0, kv_from=0)]),
    # sizes of the matrix-core bodies, many heads on one latent, many experts
    "mfma": model(320, 192, 1e-5, 12.0, [
        layer(20, 64, 32, 64, 128, 48, 0.11, 2e4, mlp=moe(70, 5, 64, 1.4, 160, 1.2)),
        layer(4, 64, 64, 128, 256, 100, 0.1, 1e4, mlp=moe(8, 2, 128, 2.0, 64, 0.9)),
        layer(8, 32, 32, 96, 128, 90, 0.14, 2e4, kv_from=0, mlp=moe(12, 4, 96, 0.8, 96, 0.8))]),
    # one large latent
    "large": model(208, 128, 1e-5, 2.0, [
        layer(16, 128, 64, 128, 512, 80, 0.08, 1e4, mlp=moe(16, 6, 64, 1.0, 128, 1.3)),
        layer(33, 32, 64, 32, 512, 130, 0.1, 1e4, kv_from=0)]),
}


def random_weights(cfg, seed=0):
    """bfloat16-representable float32 tensors by name."""
    gen = torch.Generator().manual_seed(seed)
    width, out = cfg["width"], {}

    def put(name, shape, std=1.0, mean=0.0):
        out[name] = (mean + std * torch.randn(shape, generator=gen)).bfloat16().float()

    def lin(name, n, k, gain=1.0):
        put(name, (n, k), gain * k ** -0.5)
    put("embed", (cfg["vocab"], width), 1.0 / cfg["embedding"]["scale"])
    lin("head", cfg["vocab"], width)
    put("final.norm", (), 0.2, 1.0)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}", l["mixer"]
        put(p + ".norm1", (), 0.2, 1.0)
        out[p + ".dwa"] = (0.2 + 0.3 * torch.randn(i + 2, generator=gen) + 0.5 * (torch.arange(i + 2) == i + 1)).bfloat16().float()
        q = p + ".mix."
        # a score is (q . k) * scale with entries of q and k about the gains: a spread of 2 to 3
        gain = (2.5 / (m["scale"] * (m["dim"] + m["rot_dim"]) ** 0.5)) ** 0.5
        lin(q + "q", m["heads"] * (m["dim"] + m["rot_dim"]), width, gain)
        if m.get("kv_from") is None:
            lin(q + "dkv", m["kv_rank"] + m["rot_dim"], width, gain)
            put(q + "dkv.norm", (m["kv_rank"],), 0.2, 1.0)
        lin(q + "uk", m["heads"] * m["dim"], m["kv_rank"], gain)
        lin(q + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        lin(q + "g", m["heads"], width, 2.0)
        lin(q + "o", width, m["heads"] * m["vdim"])
        f = l["mlp"]
        if f is None:
            continue
        put(p + ".norm2", (), 0.2, 1.0)
        lin(p + ".mlp.router", f["router"]["experts"], width, 2.0)
        put(p + ".mlp.router.b", (f["router"]["experts"],), 1.0)
        lin(p + ".mlp.shared.sg", 1, width, 2.0)
        for e in [f"e{j}" for j in range(f["router"]["experts"])] + ["shared"]:
            ff = f["shared" if e == "shared" else "expert"]["ff"]
            lin(f"{p}.mlp.{e}.gate", ff, width, 1.5)
            lin(f"{p}.mlp.{e}.up", ff, width, 1.5)
            lin(f"{p}.mlp.{e}.down", width, ff)
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
    return t, lepalorn.forward(cfg, w, t)


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def mixer_case(sizes, seed=0):
    """(configuration of one mixer, its weights by name)"""
    heads, dim, rot, dims, vdim, rank = sizes
    cfg = layer(heads, dim, rot, vdim, rank, 0, 2.5 * (dim + rot) ** -0.5, 3e3, rot_dims=dims)["mixer"]
    width = 64
    w = {"q": rand(heads * (dim + rot), width, seed=seed + 1) / 8, "g": rand(heads, width, seed=seed + 2) / 16,
         "dkv": rand(rank + rot, width, seed=seed + 3) / 8, "dkv.norm": 1 + 0.2 * rand(rank, seed=seed + 4),
         "uk": rand(heads * dim, rank, seed=seed + 5) * rank ** -0.5, "uv": rand(heads * vdim, rank, seed=seed + 6) * rank ** -0.5,
         "o": rand(width, heads * vdim, seed=seed + 7) * (heads * vdim) ** -0.5}
    return cfg, {k: t.bfloat16().float() for k, t in w.items()}


def edge_inputs(cfg, w, n, window, seed):
    """Rows of one sequence whose last token's first head looks for two keys: the first its window has and the one before
    that.  Their latents point along the query (and differ in what is left), so that each would carry most of the softmax."""
    x = rand(n, w["q"].shape[1], seed=seed).double()
    x[-1] *= 2  # (latents are normed: the query alone decides how far the best key is ahead)
    q = w["q"][:cfg["dim"]].double() @ x[-1]
    latent = (w["uk"][:cfg["dim"]].double() * w["dkv.norm"].double()).T @ q
    want = torch.linalg.lstsq(w["dkv"][:cfg["kv_rank"]].double(), latent[:, None]).solution[:, 0]
    want = want / want.norm() * x.shape[1] ** 0.5
    for j, other in ((n - window, 0.8), (n - 1 - window, 0.1)):  # (the one outside would win)
        if 0 <= j < n - 1:
            x[j] = want + other * x[j]
    return x.bfloat16().float()


def dense_mixer(h, m, w, lat, window):
    """lepalorn.latent_attention with the softmax over a masked matrix (its own loop takes every row and head)."""
    def attention(q, k, v, scale, size):
        i = torch.arange(q.shape[0])
        seen = (i[:, None] >= i[None]) & (i[:, None] - i[None] < size)
        s = (q.transpose(0, 1) @ k.permute(1, 2, 0) * scale).masked_fill(~seen, float("-inf"))
        return (s.softmax(-1) @ v.transpose(0, 1)).transpose(0, 1)
    with pytest.MonkeyPatch.context() as mp:
        mp.setattr(lepalorn, "window_attention", attention)
        mp.setattr(lepalorn, "rotate", fast_rotate)
        return lepalorn.latent_attention(h, dict(m, mask={"size": window}), lambda s: w[s].double(), lat)


def fast_rotate(x, positions, dims, base):
    p = torch.tensor(list(positions), dtype=torch.float64)
    a = p[:, None] * base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
    a = a.view(x.shape[0], *[1] * (x.dim() - 2), -1)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2], out[..., 1:dims:2] = u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()
    return out
