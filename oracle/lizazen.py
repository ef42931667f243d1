"""Plain, slow restatement of the Lizazen decoder on the CPU: one function per mechanism.  It shares no code with the
product and is what its tests compare with.

Weights are a mapping name -> tensor; every function works in the dtype of its inputs (tests use float64).  A configuration
is the parsed config.json of a model folder."""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def bigram_rows(tokens, bigram):
    """The row of the second table that each token adds: a hash of the token before it and itself; the last row at the start."""
    out = []
    for i, t in enumerate(tokens):
        if i == 0:
            out.append(bigram["buckets"])
        else:
            out.append((tokens[i - 1] * bigram["mul_prev"] + t * bigram["mul_cur"]) % bigram["buckets"])
    return out


def frequencies(rot):
    """Radians per position of every pair."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        s = rot.get("scaling")
        if s is not None:
            turns = s["original"] * f / (2 * math.pi)  # the original length in wavelengths
            if turns > s["high"]:
                pass
            elif turns < s["low"]:
                f = f / s["factor"]
            else:
                a = (turns - s["low"]) / (s["high"] - s["low"])
                f = (1 - a) * f / s["factor"] + a * f
        out.append(f)
    return out


def rotate(x, positions, rot):
    """x [n, ..., d]: entries i and i + dims / 2 turn by position * frequency i; those from dims on stay."""
    half = rot["dims"] // 2
    a = torch.tensor([[p * f for f in frequencies(rot)] for p in positions], dtype=torch.float64).view(len(positions), half)
    a = a.view(len(positions), *[1] * (x.dim() - 2), half)
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def sees_window(i, j, size, keep_first=0):
    return j <= i and (i - j < size or j < keep_first)


def sees_chunk(i, j, size):
    return j <= i and i // size == j // size


def attend(q, k, v, scale, sees, softcap=None, sink=None):
    """q [n, H, d], k [n, G, d], v [n, G, e]; sees(i, j): whether query i takes key j.  `sink` [H]: a score without a key."""
    n, heads, _ = q.shape
    group = heads // k.shape[1]
    seen = torch.tensor([[sees(i, j) for j in range(n)] for i in range(n)])
    out = torch.empty(n, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        s = q[:, h] @ k[:, h // group].T * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~seen, float("-inf"))
        m = s.max(1, keepdim=True).values
        p = torch.exp(s - m)
        total = p.sum(1, keepdim=True)
        if sink is not None:
            total = total + torch.exp(sink[h] - m)
        out[:, h] = (p / total) @ v[:, h // group]
    return out


def project(h, get, name, bias):
    y = h @ get(name).T
    return y + get(name + ".b") if bias else y


def normed_attention(h, m, get, eps):
    """Queries and keys normed over all heads at once; the projected keys are the values; a cap on the scores, a sink."""
    n, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = project(h, get, "q", True), project(h, get, "k", True)
    qn = rms_norm(q, get("q.norm"), eps).view(n, H, d)
    kn = rms_norm(k, get("k.norm"), eps).view(n, G, d)
    o = attend(rotate(qn, range(n), m["rot"]), rotate(kn, range(n), m["rot"]), k.view(n, G, d), m["scale"],
               lambda i, j: sees_window(i, j, m["mask"]["size"]), m["softcap"], get("sink"))
    return project(o.reshape(n, -1), get, "o", True)


def differential_weight(get, diff):
    return torch.exp((get("lq1") * get("lk1")).sum()) - torch.exp((get("lq2") * get("lk2")).sum()) + diff


def differential_attention(h, m, get, eps):
    """The difference of two attentions over the same values, normed per head."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate((h @ get("q").T).view(n, H, 2, d), range(n), m["rot"])
    k = rotate((h @ get("k").T).view(n, G, 2, d), range(n), m["rot"])
    v = (h @ get("v").T).view(n, G, e)
    a = [attend(q[:, :, i], k[:, :, i], v, m["scale"],
                lambda i, j: sees_window(i, j, m["mask"]["size"], m["mask"]["keep_first"])) for i in range(2)]
    o = rms(a[0] - differential_weight(get, m["diff"]) * a[1], eps) * (1 - m["diff"])
    return o.reshape(n, -1) @ get("o").T


def chunked_attention(h, m, get):
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (project(h, get, s, True) for s in "qkv")
    o = attend(rotate(q.view(n, H, d), range(n), m["rot"]), rotate(k.view(n, G, d), range(n), m["rot"]), v.view(n, G, e),
               m["scale"], lambda i, j: sees_chunk(i, j, m["mask"]["size"]))
    return project(o.reshape(n, -1), get, "o", True)


def retain(q, k, v, decay):
    """S <- decay S + k v^T, o = S^T q per head; q, k [n, H, d], v [n, H, e], decay [H]."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    w = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    out = torch.empty(n, H, v.shape[2], dtype=q.dtype)
    for t in range(n):
        S = w * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def retention(h, m, get, eps):
    n, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ get("q").T).view(n, H, d), range(n), m["rot"])
    k = rotate((h @ get("k").T).view(n, H, d), range(n), m["rot"]) * d ** -0.5
    o = rms(retain(q, k, (h @ get("v").T).view(n, H, e), m["decay"]), eps).reshape(n, -1)
    g = h @ get("g").T
    return (o * g * torch.sigmoid(g)) @ get("o").T


def parallel(h, m, get, eps):
    left = chunked_attention(h, m["left"], lambda s: get("left." + s))
    right = retention(h, m["right"], lambda s: get("right." + s), eps)
    return (rms_norm(left, get("left.out"), eps) + rms_norm(right, get("right.out"), eps)) / 2


def mixer(h, layer, get, eps):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return normed_attention(h, m, get, eps)
    if layer["type"] == "attention_2":
        return differential_attention(h, m, get, eps)
    assert layer["type"] == "parallel"
    return parallel(h, m, get, eps)


def clamped_unit(g, u, limit):
    """A sigmoid-gated linear unit whose gate is bounded above and whose value on both sides."""
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def dense(h, mlp, get):
    return clamped_unit(h @ get("gate").T, h @ get("up").T, mlp["limit"]) @ get("down").T


def expert(h, get, name):
    g = h @ get(name + ".gate").T
    return (g * torch.sigmoid(g) * (h @ get(name + ".up").T)) @ get(name + ".down").T


def route(z, top):
    """z [n, experts] -> (chosen [n, top], their scores)."""
    val, idx = torch.topk(z, top, dim=-1)
    return idx, torch.sigmoid(val)


def mixture(h, mlp, get):
    """Every chosen expert of the token scaled by its score, and one expert for every token."""
    idx, w = route(h @ get("router").T, mlp["router"]["top"])
    out = expert(h, get, "shared")
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), w[t]):
            out[t] += expert(s * h[t:t + 1], get, f"e{e}")[0]
    return out


def forward(config, weights, tokens, dtype=torch.float64, on_layer=None):
    """The logits [n, vocab] of one whole sequence; on_layer(i, x) sees what leaves layer i."""
    def tensor(name):
        return weights[name].to(dtype)
    eps = config["norm"]["eps"]
    tokens = [int(t) for t in tokens]
    x = tensor("embed")[tokens] + tensor("bigram")[bigram_rows(tokens, config["embedding"]["bigram"])]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        y = mixer(rms_norm(x, tensor(p + "norm1"), eps), layer, lambda s: tensor(p + "mix." + s), eps)
        x = x + rms_norm(y, tensor(p + "norm1b"), eps)
        if layer["mlp"] is not None:
            ff = dense if layer["mlp"]["kind"] == "dense" else mixture
            y = ff(rms_norm(x, tensor(p + "norm2"), eps), layer["mlp"], lambda s: tensor(p + "mlp." + s))
            x = x + rms_norm(y, tensor(p + "norm2b"), eps)
        if on_layer is not None:
            on_layer(i, x)
    return rms_norm(x, tensor("final.norm"), eps) @ tensor("head").T
