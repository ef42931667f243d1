"""Plain, slow restatement of the Lepalorn decoder on the CPU: one function per mechanism.  It shares no code with the
product and is what its tests compare with.

Weights are a mapping name -> tensor; every function works in the dtype of its inputs (tests use float64).  A configuration
is the parsed config.json of a model folder."""
import math

import torch


def scalar_norm(x, gain, eps):
    """RMS norm whose gain is one number for all coordinates."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def rms_norm(x, weight, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def rotate(x, positions, dims, base):
    """x [n, ..., d]: pairs (2i, 2i + 1) of the first `dims` entries turn by position * base^(-2i / dims)."""
    out = x.clone()
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        for t, p in enumerate(positions):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * c - v * s
            out[t, ..., 2 * i + 1] = v * c + u * s
    return out


def window_attention(q, k, v, scale, window):
    """q, k [n, H, d], v [n, H, e]: query i sees keys i - window + 1 .. i."""
    n, heads, _ = q.shape
    out = torch.empty(n, heads, v.shape[2], dtype=q.dtype)
    for i in range(n):
        a = max(0, i - window + 1)
        for h in range(heads):
            s = (k[a:i + 1, h] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[a:i + 1, h]
    return out


def latent_parts(h, m, get, eps):
    """What a layer caches: the normed latent [n, kv_rank] and the rotated key part [n, rot_dim] all heads share."""
    z = h @ get("dkv").T
    c = rms_norm(z[:, :m["kv_rank"]], get("dkv.norm"), eps)
    return c, rotate(z[:, m["kv_rank"]:], range(h.shape[0]), m["rot"]["dims"], m["rot"]["base"])


def latent_attention(h, m, get, latent):
    """The mixer of one layer over the latent parts of its own or of an earlier layer."""
    n, heads, dim, rot_dim = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    c, k_rot = latent
    q = (h @ get("q").T).view(n, heads, dim + rot_dim)
    q_rot = rotate(q[:, :, dim:], range(n), m["rot"]["dims"], m["rot"]["base"])
    k = (c @ get("uk").T).view(n, heads, dim)
    v = (c @ get("uv").T).view(n, heads, m["vdim"])
    o = window_attention(torch.cat([q[:, :, :dim], q_rot], 2), torch.cat([k, k_rot[:, None].expand(-1, heads, -1)], 2), v,
                         m["scale"], m["mask"]["size"])
    o = o * torch.sigmoid(h @ get("g").T)[:, :, None]
    return o.reshape(n, -1) @ get("o").T


def clamped_gate(g, u, limit):
    """The experts' activation: a sigmoid-gated linear unit whose gate is bounded above and whose value on both sides."""
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(h, get, name, limit):
    return clamped_gate(h @ get(name + ".gate").T, h @ get(name + ".up").T, limit) @ get(name + ".down").T


def route(z, top):
    """z [n, experts] -> (chosen [n, top], weights [n, top]: softmax over the chosen logits)."""
    val, idx = torch.topk(z, top, dim=-1)
    e = torch.exp(val - val.max(-1, keepdim=True).values)
    return idx, e / e.sum(-1, keepdim=True)


def mixture(h, mlp, get):
    """The chosen experts' weighted sum and the gated shared expert."""
    idx, w = route(h @ get("router").T + get("router.b"), mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(idx[t].tolist(), w[t]):
            out[t] += p * expert(h[t:t + 1], get, f"e{e}", mlp["expert"]["limit"])[0]
    return out + torch.sigmoid(h @ get("shared.sg").T) * expert(h, get, "shared", mlp["shared"]["limit"])


def depth_average(streams, weights):
    """One number per stream: the embedding's and every layer's so far."""
    assert len(streams) == len(weights)
    return sum(weights[j] * streams[j] for j in range(len(streams)))


def forward(config, weights, tokens, dtype=torch.float64, on_layer=None):
    """The logits [n, vocab] of one whole sequence; on_layer(i, x) sees what leaves layer i."""
    def tensor(name):
        return weights[name].to(dtype)
    eps = config["norm"]["eps"]
    x = tensor("embed")[torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    streams, latents = [x], {}
    for i, layer in enumerate(config["layers"]):
        def mix(s):
            return tensor(f"l{i}.mix.{s}")
        m = layer["mixer"]
        if m.get("kv_from") is None:
            latents[i] = latent_parts(x, m, mix, eps)
            source = i
        else:
            source = m["kv_from"]
        x = x + scalar_norm(latent_attention(x, m, mix, latents[source]), tensor(f"l{i}.norm1"), eps)
        if layer["mlp"] is not None:
            x = x + scalar_norm(mixture(x, layer["mlp"], lambda s: tensor(f"l{i}.mlp.{s}")), tensor(f"l{i}.norm2"), eps)
        streams.append(x)
        x = depth_average(streams, tensor(f"l{i}.dwa"))
        if on_layer is not None:
            on_layer(i, x)
    return scalar_norm(x, tensor("final.norm"), eps) @ tensor("head").T
