"""Susalorn on the CPU: configuration, cache and state sizes, and the plain restatement the GPU tests compare with (closed forms,
and planted mistakes that the tests' weights must make visible)."""
import copy
import math

import pytest
import torch

import susalorn_case as sc
from layered_case import error, tokens, write_model
from oracle import susalorn

F64 = torch.float64


def load(tmp_path, name, dtype=torch.float32):
    from light_vllm_amd.engine.registry import load_model_config
    return load_model_config(write_model(tmp_path / name, *sc.case(name)), dtype)


def rand(*shape, seed=0):
    return sc.rand(*shape, seed=seed).double()


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_configuration_gives_every_size(tmp_path, name):
    from light_vllm_amd.engine.stream_model import StreamModel
    cfg, w = sc.case(name)
    c = load(tmp_path, name)
    shapes = StreamModel.tensor_shapes(c)
    low_rank = ("a1", "a2", "g1", "g2")
    assert shapes.keys() == w.keys()
    assert all(shape == tuple(w[k].shape) for k, shape in shapes.items() if not k.endswith(low_rank))
    assert (c.norm_eps, c.vocab_size, c.hidden_size, c.streams) == (cfg["norm"]["eps"], cfg["vocab"], cfg["width"], cfg["streams"])
    assert c.runs == susalorn.passes(cfg) and c.num_hidden_layers == len(c.runs)
    for i, spec, state in zip(c.runs, c.kv_cache_specs(), c.state_specs()):
        l, d = c.layers[i], cfg["layers"][i]
        m = d["mixer"]
        if d["type"] == "latent_attention":
            a = l.mixer
            assert (a.heads, a.dim, a.rot_dim, a.vdim, a.kv_rank, a.q_rank, a.scale) == tuple(
                m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale"))
            assert (a.window, a.gate, a.sink) == (0, False, True) and state == {}
            assert spec.cpad >= m["kv_rank"] and spec.rpad >= m["rot_dim"]
            assert torch.allclose(torch.tensor(a.rot.frequencies(), dtype=F64), torch.tensor(susalorn.frequencies(m["rot"]), dtype=F64))
            assert math.isclose(a.rot.grow, susalorn.magnitude(m["rot"]))
        else:
            assert spec is None and state["matrix"] == (m["heads"], m["dim"], m["vdim"])
            taps, channels = state["conv"]
            assert taps == m["conv"] and channels >= 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"]
        if d["mlp"] is None:
            assert l.mlp is None
        elif d["mlp"]["kind"] == "dense":
            assert l.mlp.ff == d["mlp"]["ff"]
        else:
            r = d["mlp"]["router"]
            assert (l.mlp.experts, l.mlp.top, l.mlp.groups, l.mlp.keep, l.mlp.weight_scale, l.mlp.expert.ff) == (
                r["experts"], r["top"], r["groups"]["count"], r["groups"]["keep"], r["scale"], d["mlp"]["expert"]["ff"])
            assert l.mlp.shared is None


def test_configuration_refuses_what_it_does_not_know():
    from light_vllm_amd.engine.stream_config import StreamModelConfig
    good = sc.CONFIGS["all"]
    StreamModelConfig.from_dict(good)

    def broken(edit):
        c = copy.deepcopy(good)
        edit(c)
        with pytest.raises(ValueError):
            StreamModelConfig.from_dict(c)
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=15))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))             # four heads
    broken(lambda c: c["layers"][1]["mixer"].update(dim=260))
    broken(lambda c: c["layers"][1]["mixer"].update(conv=0))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=5))          # of two groups of two
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4))
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4))
    broken(lambda c: c["loop"].update(stop=9))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c.update(streams=0))
    with pytest.raises(ValueError):
        StreamModelConfig.from_dict(good, dtype=torch.float16)


def test_every_pass_has_a_cache_or_a_state(tmp_path):
    from light_vllm_amd.attention.latent_backend import LatentAttnBackend
    from light_vllm_amd.engine.cache_engine import CacheEngine
    from light_vllm_amd.engine.config import CacheConfig
    c = load(tmp_path, "all", torch.bfloat16)
    assert c.runs == [0, 1, 2, 3, 1, 2, 3, 4, 5]
    e = CacheEngine(CacheConfig(num_gpu_blocks=5, num_cpu_blocks=2, num_state_slots=3), c, LatentAttnBackend(), "cpu")
    layers = e.model_caches().layers
    assert [l.kv is not None for l in layers] == [True, False, True, False, False, True, False, True, False]
    assert len({l.kv.data_ptr() for l in layers if l.kv is not None}) == 4
    state = [l.state for l in layers if l.state]
    assert len({s["matrix"].data_ptr() for s in state}) == 5 and all(s["conv"].dtype == torch.float32 for s in state)
    # a fork takes the states along
    for s in state:
        s["conv"][1], s["matrix"][1] = 1.5, 2.5
    e.copy_state([(1, 2)])
    assert all((s["conv"][2] == 1.5).all() and (s["matrix"][2] == 2.5).all() and not s["matrix"][0].any() for s in state)
    per_slot = sum(4 * (math.prod(s["conv"].shape[1:]) + math.prod(s["matrix"].shape[1:])) for s in state)
    assert CacheEngine.get_state_bytes(c, 7) == 7 * per_slot


def test_rows_in_another_order_turn_alike():
    """Pairs (i, i + dims / 2) as the pairs (2i, 2i + 1) of reordered rows: dot products stay."""
    from light_vllm_amd.engine.latent_config import RotationConfig
    from light_vllm_amd.engine.latent_layers import Rotation
    r = Rotation(RotationConfig(8, 100.0, halves=True), "cpu")
    x = torch.arange(11.0)[:, None]
    assert r.ordered(x)[:, 0].tolist() == [0, 4, 1, 5, 2, 6, 3, 7, 8, 9, 10]
    assert torch.equal(Rotation(RotationConfig(8, 100.0), "cpu").ordered(x), x)


# ---- the restatement ----
def test_rotation_pairs_halves_grows_and_depends_on_the_distance():
    r = sc.rot(8, 500.0, (4.0, 64, 8.0, 1.0))
    grow = 0.1 * math.log(4) + 1
    x = rand(5, 3, 8)
    y = susalorn.rotate(x, [0, 1, 7, 1000, 123456], r)
    assert torch.allclose(y[0], grow * x[0]) and torch.allclose(y.norm(dim=-1), grow * x.norm(dim=-1))
    e = susalorn.rotate(torch.eye(8, dtype=F64)[:1], [1], sc.rot(8, 500.0))  # entry 0 turns towards entry 4
    assert torch.allclose(e[0, [0, 4]], torch.tensor([math.cos(1), math.sin(1)], dtype=F64)) and e[0].count_nonzero() == 2
    a, b = rand(1, 8, seed=1), rand(1, 8, seed=2)

    def score(p, q):
        return (susalorn.rotate(a, [p], r) * susalorn.rotate(b, [q], r)).sum()
    assert torch.allclose(score(9, 4), score(1009, 1004))


def test_frequency_ramp():
    base = susalorn.frequencies(sc.rot(32, 1e4))
    got = susalorn.frequencies(sc.rot(32, 1e4, (8.0, 1000, 16.0, 2.0)))
    turns = [1000 * f / (2 * math.pi) for f in base]
    kinds = set()
    for i, (f, g, n) in enumerate(zip(base, got, turns)):
        if n >= 16 * 1e4 ** (2 / 32):  # (the ramp's ends are whole pairs)
            assert g == f
            kinds.add("kept")
        elif n <= 2 / 1e4 ** (2 / 32):
            assert math.isclose(g, f / 8)
            kinds.add("slowed")
        else:
            assert f / 8 <= g <= f
            kinds.add("between")
    assert kinds == {"kept", "slowed", "between"}
    # a ramp of no width at all is a step
    step = susalorn.frequencies(sc.rot(8, 1e4, (2.0, 1000, 1.0, 1.0)))
    assert all(g in (f, f / 2) for f, g in zip(susalorn.frequencies(sc.rot(8, 1e4)), step))


def test_attention_with_a_sink():
    q, k, v = rand(6, 3, 5), rand(6, 3, 5, seed=1), rand(6, 3, 4, seed=2)
    sink = torch.tensor([0.3, -50.0, 40.0], dtype=F64)
    got = susalorn.attend(q, k, v, 0.7, sink)
    for i in range(6):
        for h in range(3):
            e = torch.exp(torch.stack([q[i, h] @ k[j, h] * 0.7 for j in range(i + 1)]))
            assert torch.allclose(got[i, h], (e[:, None] * v[:i + 1, h]).sum(0) / (e.sum() + math.exp(sink[h])))


def test_short_convolution():
    x, w = rand(7, 3), rand(3, 4, seed=1)
    got = susalorn.short_conv(x, w)
    for t in range(7):
        z = sum(x[t - j] * w[:, 3 - j] for j in range(4) if t >= j)
        assert torch.allclose(got[t], z * torch.sigmoid(z))


def test_delta_rule_replaces_what_a_key_returns():
    """With unit keys, full writes and no decay, a key returns the value written for it last."""
    k = torch.zeros(4, 1, 3, dtype=F64)
    k[0, 0, 0] = k[1, 0, 1] = k[2, 0, 0] = k[3, 0, 2] = 1
    v, one = rand(4, 1, 5), torch.ones(4, 1, 3, dtype=F64)
    q = torch.tensor([[1.0, 0, 0], [1, 0, 0], [1, 0, 0], [1, 1, 0]], dtype=F64)[:, None]
    o = susalorn.delta_rule(q, k, v, one, torch.ones(4, 1, dtype=F64))
    assert torch.allclose(o[:, 0], torch.stack([v[0, 0], v[0, 0], v[2, 0], v[2, 0] + v[1, 0]]))
    # half a write, a decay of the key's channel
    o = susalorn.delta_rule(q[:2], k[:1].expand(2, 1, 3), v[:2], 0.5 * one[:2], torch.full((2, 1), 0.25, dtype=F64))
    s = 0.25 * v[0, 0]
    assert torch.allclose(o[1, 0], 0.5 * s + 0.25 * (v[1, 0] - 0.5 * s))


def test_router_of_groups():
    r = {"top": 2, "groups": {"count": 3, "keep": 2}, "scale": 2.5}
    z = torch.tensor([[9.0, 1.0, 7.0, 6.0, 8.0, 2.0], [0.0, 5.0, 4.9, 4.8, 1.0, 2.0]], dtype=F64)
    idx, w = susalorn.route(z, r)
    assert idx.tolist() == [[0, 4], [1, 2]]  # (expert 2 of the first row lies in the closed group)
    e = torch.exp(z.gather(1, idx))
    assert torch.allclose(w, 2.5 * e / e.sum(1, keepdim=True))


def test_streams():
    x, y = rand(3, 4, 5), rand(4, 5, seed=1)
    mix, out = rand(3, 3, seed=2), rand(3, seed=3)
    got = susalorn.write_streams(x, mix, out, y)
    assert torch.allclose(got[2], mix[0, 2] * x[0] + mix[1, 2] * x[1] + mix[2, 2] * x[2] + out[2] * y)
    assert torch.allclose(susalorn.read_streams(x, out), out[0] * x[0] + out[1] * x[1] + out[2] * x[2])


def test_order_of_passes():
    assert susalorn.passes(sc.model(1, 1, 1, 1, (1, 3, 2), [(("x", {}), None)] * 4)) == [0, 1, 2, 1, 2, 3]
    assert susalorn.passes(sc.model(1, 1, 1, 1, None, [(("x", {}), None)] * 2)) == [0, 1]


def changed(edit=None, patch=None, name="all", n=60):
    """Largest error of the restatement's logits after a planted change of the configuration or of a mechanism."""
    cfg, w = sc.case(name)
    t = tokens(cfg, n, 3)
    want = susalorn.forward(cfg, w, t)
    c = copy.deepcopy(cfg)
    if edit is not None:
        edit(c)
    with pytest.MonkeyPatch.context() as mp:
        if patch is not None:
            patch(mp)
        return error(susalorn.forward(c, w, t), want).max().item()


def test_planted_mistakes_show():
    def replace(name, make):
        def patch(mp):
            mp.setattr(susalorn, name, make(getattr(susalorn, name)))
        patch.__name__ = name
        return patch

    def interleaved(rotate):
        def f(x, p, r):
            perm = list(range(0, r["dims"], 2)) + list(range(1, r["dims"], 2)) + list(range(r["dims"], x.shape[-1]))
            out = torch.empty_like(x)
            out[..., perm] = rotate(x[..., perm], p, r)
            return out
        return f

    def before_the_write(rule):
        def f(q, k, v, g, beta):
            o = rule(q, k, v, g, beta)
            return torch.cat([torch.zeros_like(o[:1]), o[:-1]])
        return f

    def no_replacement(rule):
        def f(q, k, v, g, beta):  # a plain sum of outer products
            S, out = torch.zeros(*k.shape[1:], v.shape[2], dtype=v.dtype), []
            for t in range(len(k)):
                S = g[t][:, :, None] * S + beta[t][:, None, None] * k[t][:, :, None] * v[t][:, None]
                out.append((S * q[t][:, :, None]).sum(1))
            return torch.stack(out)
        return f

    def one_decay_per_head(decay):
        def f(*a):
            g = decay(*a)
            return g.mean(-1, keepdim=True).expand_as(g)
        return f

    def shifted(conv):
        return lambda x, taps: conv(x, taps.roll(1, 1))

    def any_group(route):
        return lambda z, r: route(z, dict(r, groups={"count": 1, "keep": 1}))

    def softmax_weights(route):  # over all experts, not over the chosen ones
        return lambda z, r: (route(z, r)[0], torch.softmax(z, -1).gather(1, route(z, r)[0]) * r["scale"])
    patches = [
        replace("attend", lambda f: lambda q, k, v, s, sink: f(q, k, v, s, torch.full_like(sink, -1e9))),
        replace("attend", lambda f: lambda q, k, v, s, sink: f(q, k, v, s, sink * s)),
        replace("rotate", interleaved), replace("rotate", lambda f: lambda x, p, r: x),
        replace("magnitude", lambda f: lambda r: 1.0), replace("delta_rule", before_the_write),
        replace("delta_rule", no_replacement), replace("channel_decay", one_decay_per_head), replace("short_conv", shifted),
        replace("unit", lambda f: lambda x: x), replace("route", any_group), replace("route", softmax_weights),
        replace("write_streams", lambda f: lambda x, mix, out, y: f(x, mix.T, out, y)),
        replace("read_streams", lambda f: lambda x, w: f(x, torch.full_like(w, 1 / len(w))))]
    for patch in patches:
        assert changed(patch=patch) > 1e-2, patch.__name__
    for edit in (lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling"), lambda c: c["loop"].update(times=3),
                 lambda c: c["loop"].update(stop=3), lambda c: c["norm"].update(eps=1e-2),
                 lambda c: c["layers"][0]["mlp"]["router"].update(scale=2.0), lambda c: c["layers"][2]["mixer"].update(scale=0.18)):
        assert changed(edit) > 3e-3, edit


def test_what_is_far_back_shows():
    """The first tokens of a sequence still matter at its end: keys, and what the states hold."""
    for name in ("all", "mfma"):
        cfg, w = sc.case(name)
        t = tokens(cfg, 150, 4)
        want = susalorn.forward(cfg, w, t)[-1:]
        other = [(x + 7) % cfg["vocab"] for x in t[:3]] + t[3:]
        assert error(susalorn.forward(cfg, w, other)[-1:], want).max() > 1e-3, name
