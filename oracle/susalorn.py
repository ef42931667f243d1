"""Plain, slow restatement of the Susalorn decoder on the CPU: one function per mechanism.  It shares no code with the
product and is what its tests compare with.

Weights are a mapping name -> tensor; every function works in the dtype of its inputs (tests use float64).  A configuration
is the parsed config.json of a model folder."""
import math

import torch
import torch.nn.functional as F


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


# ---- latent attention ----
def frequencies(rot):
    """Radians per position of every pair: those that turn often within `original` positions keep theirs, slow ones are divided
    by `factor`, a ramp over the pairs between."""
    dims, base, s = rot["dims"], rot["base"], rot.get("scaling")
    out = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if s is None:
        return out

    def pair_of(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair_of(s["fast"])), 0), min(math.ceil(pair_of(s["slow"])), dims - 1)
    ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return [f / s["factor"] * r + f * (1 - r) for f, r in zip(out, ramp)]


def magnitude(rot):
    """What cosines and sines are multiplied by."""
    s = rot.get("scaling")
    return 1.0 if s is None else 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [n, ..., dims]: entries i and i + dims / 2 turn by position * frequency i."""
    half, m = rot["dims"] // 2, magnitude(rot)
    a = torch.tensor([[p * f for f in frequencies(rot)] for p in positions], dtype=torch.float64).view(len(positions), half)
    a = a.view(len(positions), *[1] * (x.dim() - 2), half)
    c, s = (m * a.cos()).to(x.dtype), (m * a.sin()).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def attend(q, k, v, scale, sink):
    """Causal softmax attention, q, k [n, H, d], v [n, H, e]; `sink` [H]: a score without a key."""
    n, heads, _ = q.shape
    future = torch.ones(n, n, dtype=torch.bool).triu(1)
    out = torch.empty(n, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        s = (q[:, h] @ k[:, h].T * scale).masked_fill(future, float("-inf"))
        m = torch.maximum(s.max(1, keepdim=True).values, sink[h])
        p = torch.exp(s - m)
        out[:, h] = p @ v[:, h] / (p.sum(1, keepdim=True) + torch.exp(sink[h] - m))
    return out


def latent_attention(h, m, get, eps):
    n, H, d, r, e, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms_norm(h @ get("dq").T, get("dq.norm"), eps) @ get("uq").T).view(n, H, d + r)
    kv = h @ get("dkv").T
    c = rms_norm(kv[:, :rank], get("dkv.norm"), eps)
    q = torch.cat([q[..., :d], rotate(q[..., d:], range(n), m["rot"])], -1)
    shared = rotate(kv[:, rank:], range(n), m["rot"])
    k = torch.cat([(c @ get("uk").T).view(n, H, d), shared[:, None].expand(n, H, r)], -1)
    o = attend(q, k, (c @ get("uv").T).view(n, H, e), m["scale"], get("sink"))
    return o.reshape(n, -1) @ get("o").T


# ---- gated delta rule ----
def short_conv(x, taps):
    """x [n, channels], taps [channels, T]: a sum over the last T rows per channel (the last tap is the row's own), then silu."""
    T = taps.shape[1]
    padded = torch.cat([x.new_zeros(T - 1, x.shape[1]), x])
    return F.silu(sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(T)))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_decay(h, get, heads, dim):
    """Per head and key channel, [n, heads, dim]."""
    z = (h @ get("a1").T) @ get("a2").T + get("dt_bias")
    step = torch.where(z > 30, z, torch.log1p(torch.exp(z.clamp(max=30))))
    return torch.exp(-torch.exp(get("A_log"))[:, None] * step.view(-1, heads, dim))


def delta_rule(q, k, v, g, beta):
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k, g [n, H, d], v [n, H, e], beta [n, H]."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.empty(n, H, v.shape[2], dtype=q.dtype)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def channel_delta(h, m, get, eps):
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ get(s).T, get(s + ".conv")) for s in "qkv")
    q = (unit(q.view(n, G, d)) * d ** -0.5).repeat_interleave(H // G, 1)
    k = unit(k.view(n, G, d)).repeat_interleave(H // G, 1)
    o = delta_rule(q, k, v.view(n, H, e), channel_decay(h, get, H, d), torch.sigmoid(h @ get("b").T))
    gate = torch.sigmoid((h @ get("g1").T) @ get("g2").T).view(n, H, e)
    return (rms_norm(o, get("norm"), eps) * gate).reshape(n, -1) @ get("o").T


def mixer(h, layer, get, eps):
    return {"latent_attention": latent_attention, "channel_delta": channel_delta}[layer["type"]](h, layer["mixer"], get, eps)


# ---- feed-forwards ----
def dense(h, get):
    return (F.silu(h @ get("gate").T) * (h @ get("up").T)) @ get("down").T


def expert(h, get, name):
    return torch.relu(h @ get(name + ".up").T).square() @ get(name + ".down").T


def route(z, router):
    """z [n, experts] -> (chosen [n, top], weights): of the groups with the largest best scores."""
    s = torch.softmax(z, -1)
    groups = router["groups"]
    n, size = z.shape[0], z.shape[1] // groups["count"]
    best = s.view(n, groups["count"], size).max(-1).values.topk(groups["keep"], dim=-1).indices
    open_ = torch.zeros(n, groups["count"], dtype=torch.bool).scatter_(1, best, True).repeat_interleave(size, 1)
    idx = s.masked_fill(~open_, -1.0).topk(router["top"], dim=-1).indices
    w = s.gather(1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20) * router["scale"]


def mixture(h, mlp, get):
    idx, w = route(h @ get("router").T, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), w[t]):
            out[t] += s * expert(h[t:t + 1], get, f"e{e}")[0]
    return out


def feed_forward(h, mlp, get):
    return dense(h, get) if mlp["kind"] == "dense" else mixture(h, mlp, get)


# ---- the decoder ----
def read_streams(x, weights):
    """x [streams, n, width] -> the sublayer's input [n, width]."""
    return torch.einsum("s,snw->nw", weights, x)


def write_streams(x, mix, out, y):
    """Every stream from all old ones (mix [from, to]) and the sublayer's output."""
    return torch.einsum("st,snw->tnw", mix, x) + out[:, None, None] * y


def passes(config):
    """The layers in the order they run."""
    loop, n = config.get("loop"), len(config["layers"])
    if loop is None:
        return list(range(n))
    return [*range(loop["start"]), *(list(range(loop["start"], loop["stop"])) * loop["times"]), *range(loop["stop"], n)]


def forward(config, weights, tokens, dtype=torch.float64, on_layer=None):
    """The logits [n, vocab] of one whole sequence; on_layer(i, x) sees the streams' sum after the i-th layer that runs."""
    def tensor(name):
        return weights[name].to(dtype)
    eps = config["norm"]["eps"]
    x = tensor("embed")[[int(t) for t in tokens]].expand(config["streams"], -1, -1)
    for at, i in enumerate(passes(config)):
        layer, p = config["layers"][i], f"l{i}."
        sublayers = [lambda h: mixer(h, layer, lambda s: tensor(p + "mix." + s), eps)]
        if layer["mlp"] is not None:
            sublayers.append(lambda h: feed_forward(h, layer["mlp"], lambda s: tensor(p + "mlp." + s)))
        for q, sublayer in enumerate(sublayers, 1):
            hc = f"{p}hc{q}."
            y = sublayer(rms_norm(read_streams(x, tensor(hc + "in")), tensor(f"{p}norm{q}"), eps))
            x = write_streams(x, tensor(hc + "mix"), tensor(hc + "out"), y)
        if on_layer is not None:
            on_layer(at, x.sum(0))
    return rms_norm(x.sum(0), tensor("final.norm"), eps) @ tensor("embed").T
