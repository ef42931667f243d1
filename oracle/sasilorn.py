"""Plain, slow restatement of the Sasilorn decoder on the CPU: one function per mechanism, one token after the other where
the mechanism is a recurrence.  It shares no code with the product and is what its tests compare with.

Weights are a mapping name -> tensor; every function works in the dtype of its inputs (tests use float64).  A configuration
is the parsed config.json of a model folder."""
import torch


def dynamic_tanh(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def rms_norm(x, eps, w=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(x):
    return x * torch.sigmoid(x)


def squared_relu(x):
    return torch.clamp(x, min=0) ** 2


def softmax_heads(q, k, v, scale):
    """q [n, H, d], k [n, G, d], v [n, G, e]: causal attention, query head h on key/value head h // (H / G)."""
    n, heads, kv_heads = q.shape[0], q.shape[1], k.shape[1]
    out = torch.empty(n, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        g = h // (heads // kv_heads)
        for i in range(n):
            s = (k[:i + 1, g] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[:i + 1, g]
    return out


def gated_linear_decay(z, tau):
    """alpha per key channel: sigmoid(z) ** (1 / tau)."""
    return torch.sigmoid(z) ** (1.0 / tau)


def gated_linear_attention(q, k, v, alpha, state=None):
    """q, k, alpha [n, H, d], v [n, H, e] -> (o [n, H, e], last state [H, d, e])."""
    n, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    o = torch.empty(n, heads, v.shape[2], dtype=q.dtype)
    for t in range(n):
        s = alpha[t][:, :, None] * s + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (s * q[t][:, :, None]).sum(1)
    return o, s


def token_shift(h, mu, before=None):
    """h [n, width]: each row moved towards the row before it (`before` ahead of the first; zeros when None)."""
    first = torch.zeros_like(h[:1]) if before is None else before[None]
    prev = torch.cat([first, h[:-1]])
    return h + (prev - h) * mu


def wkv_decay(z):
    return torch.exp(-torch.exp(z))


def wkv(r, k, v, w, u, state=None):
    """r, k, v, w [n, H, d], u [H, d] -> (o [n, H, d], last state [H, d, d])."""
    n, heads, d = r.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=r.dtype) if state is None else state.clone()
    o = torch.empty(n, heads, v.shape[2], dtype=r.dtype)
    for t in range(n):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = ((s + u[:, :, None] * kv) * r[t][:, :, None]).sum(1)
        s = w[t][:, :, None] * s + kv
    return o, s


def parallel_mixer(h, cfg, get, eps):
    n, left, right = h.shape[0], cfg["left"], cfg["right"]

    def lin(name):
        return h @ get(name).T
    q = rms_norm(lin("left.q").view(n, left["heads"], left["dim"]), eps, get("left.q.norm"))
    k = rms_norm(lin("left.k").view(n, left["kv_heads"], left["dim"]), eps, get("left.k.norm"))
    v = lin("left.v").view(n, left["kv_heads"], left["vdim"])
    o = softmax_heads(q, k, v, left["scale"]) * torch.sigmoid(lin("left.g"))[:, :, None]
    a = o.reshape(n, -1) @ get("left.o").T

    shape = (n, right["heads"], right["dim"])
    z = lin("right.a1") @ get("right.a2").T + get("right.a2.b")
    o, _ = gated_linear_attention(lin("right.q").view(shape) * right["dim"] ** -0.5, lin("right.k").view(shape),
                                  lin("right.v").view(n, right["heads"], right["vdim"]),
                                  gated_linear_decay(z, right["tau"]).view(shape))
    o = rms_norm(o, eps, get("right.norm")).reshape(n, -1) * silu(lin("right.g"))
    return cfg["left_scale"] * a + cfg["right_scale"] * (o @ get("right.o").T)


def time_mixer(h, cfg, get, eps):
    n, shape = h.shape[0], (h.shape[0], cfg["heads"], cfg["dim"])
    mix = {s: token_shift(h, get("mu." + s)) for s in "rkvgw"}
    r, k, v = ((mix[s] @ get(s).T).view(shape) for s in "rkv")
    gate = silu(mix["g"] @ get("g").T)
    z = torch.tanh(mix["w"] @ get("w1").T) @ get("w2").T + get("w0")
    o, _ = wkv(r, k, v, wkv_decay(z).view(shape), get("u"))
    return (rms_norm(o, eps).reshape(n, -1) * get("norm") * gate) @ get("o").T


def forward(config, weights, tokens, dtype=torch.float64, on_layer=None):
    """The logits [n, vocab] of one whole sequence; on_layer(i, x) sees the residual stream after layer i."""
    def tensor(name):
        return weights[name].to(dtype)

    def norm(x, name):
        return dynamic_tanh(x, tensor(name + ".alpha"), tensor(name), tensor(name + ".b"))
    eps = config["norm"]["eps"]
    x = tensor("embed")[torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(config["layers"]):
        j = i
        while config["layers"][j].get("weights_of") is not None:
            j = config["layers"][j]["weights_of"]
        mixer = {"parallel": parallel_mixer, "wkv": time_mixer}[layer["type"]]
        x = x + mixer(norm(x, f"l{j}.norm1"), layer["mixer"], lambda s: tensor(f"l{j}.mix.{s}"), eps)
        if layer["mlp"] is not None:
            x = x + squared_relu(norm(x, f"l{j}.norm2") @ tensor(f"l{j}.mlp.up").T) @ tensor(f"l{j}.mlp.down").T
        if on_layer is not None:
            on_layer(i, x)
    return norm(x, "final.norm") @ tensor("head").T
