"""Lizazen on the CPU: configuration, cache and state sizes, and the plain restatement the GPU tests compare with (closed forms,
and planted mistakes that the tests' weights must make visible)."""
import copy
import math

import pytest
import torch

import lizazen_case as lc
from layered_case import error, tokens, write_model
from oracle import lizazen

F64 = torch.float64


def load(tmp_path, name, dtype=torch.float32):
    from light_vllm_amd.engine.registry import load_model_config
    return load_model_config(write_model(tmp_path / name, *lc.case(name)), dtype)


def rand(*shape, seed=0):
    return lc.rand(*shape, seed=seed).double()


@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_configuration_gives_every_size(tmp_path, name):
    from light_vllm_amd.engine.local_model import LocalModel
    cfg, w = lc.case(name)
    c = load(tmp_path, name)
    assert LocalModel.tensor_shapes(c) == {k: tuple(t.shape) for k, t in w.items()}
    b = cfg["embedding"]["bigram"]
    assert (c.norm_eps, c.vocab_size, c.pairs.buckets, c.pairs.mul_previous, c.pairs.mul_current) == (
        cfg["norm"]["eps"], cfg["vocab"], b["buckets"], b["mul_prev"], b["mul_cur"])
    assert c.num_hidden_layers == len(cfg["layers"])
    for spec, state, l, d in zip(c.kv_cache_specs(), c.state_specs(), c.layers, cfg["layers"]):
        a, m = c.attention_of(l), d["mixer"].get("left", d["mixer"])
        maps = 2 if d["type"] == "attention_2" else 1
        assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.maps) == (*(m[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale")), maps)
        size, keep = m["mask"]["size"], m["mask"].get("keep_first", 0)
        assert (a.sees.window, a.sees.chunk, a.sees.keep_first) == ((0, size, 0) if d["type"] == "parallel" else (size, 0, keep))
        assert (a.softcap, a.diff) == (m.get("softcap", 0.0), m.get("diff"))
        assert spec.kpad >= maps * a.dim and spec.kpad % (8 * maps) == 0 and spec.vpad >= a.vdim
        assert torch.allclose(torch.tensor(a.rot.frequencies(), dtype=F64), torch.tensor(lizazen.frequencies(m["rot"]), dtype=F64))
        if d["type"] == "parallel":
            r = d["mixer"]["right"]
            assert state == {"matrix": (r["heads"], r["dim"], r["vdim"])} and list(c.retention_of(l).decay) == r["decay"]
        else:
            assert state == {} and c.retention_of(l) is None
        if d["mlp"] is None:
            assert l.mlp is None
        elif d["mlp"]["kind"] == "dense":
            assert (l.mlp.ff, l.mlp.limit) == (d["mlp"]["ff"], d["mlp"]["limit"])
        else:
            assert (l.mlp.experts, l.mlp.top, l.mlp.expert.ff, l.mlp.shared.ff) == (
                d["mlp"]["router"]["experts"], d["mlp"]["router"]["top"], d["mlp"]["expert"]["ff"], d["mlp"]["shared"]["ff"])


def test_configuration_refuses_what_it_does_not_know():
    from light_vllm_amd.engine.local_config import LocalModelConfig
    good = lc.CONFIGS["all"]
    LocalModelConfig.from_dict(good)

    def broken(edit):
        c = copy.deepcopy(good)
        edit(c)
        with pytest.raises(ValueError):
            LocalModelConfig.from_dict(c)
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=2))             # three heads
    broken(lambda c: c["layers"][0]["mixer"].update(vdim=48))                # keys are the values
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1))
    broken(lambda c: c["layers"][2]["mixer"]["left"]["mask"].update(size=0))
    broken(lambda c: c["layers"][2]["mixer"]["right"].update(decay=[0.5]))   # three heads
    broken(lambda c: c["layers"][2]["mixer"]["right"].update(decay=[0.5, 1.1, 0.2]))
    broken(lambda c: c["layers"][2]["mixer"]["right"].update(dim=320))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=26))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=8))
    broken(lambda c: c["embedding"]["bigram"].update(buckets=0))
    with pytest.raises(ValueError):
        LocalModelConfig.from_dict(good, dtype=torch.float16)


def test_cache_and_states_of_a_sequence(tmp_path):
    from light_vllm_amd.attention.head_backend import HeadAttnBackend, HeadAttnImpl
    from light_vllm_amd.engine.cache_engine import CacheEngine
    from light_vllm_amd.engine.config import CacheConfig
    c = load(tmp_path, "all", torch.bfloat16)
    cc = CacheConfig(num_gpu_blocks=5, num_cpu_blocks=2, num_state_slots=3)
    e = CacheEngine(cc, c, HeadAttnBackend(), "cpu")
    caches = e.model_caches()
    assert [set(x.state) for x in caches.layers] == [set(), set(), {"matrix"}, set(), set()]
    previous = caches.sequence["previous_token"]
    assert previous.shape == (3,) and previous.dtype == torch.int32
    assert CacheEngine.get_state_bytes(c, 7) == 7 * 4 * (3 * 24 * 40 + 1)
    # a differential layer's keys: both maps of a kv head, each padded
    spec = c.kv_cache_specs()[1]
    assert (spec.maps, spec.kpad, spec.vpad) == (2, 64, 64)
    k, v = HeadAttnImpl.split_kv_cache(caches.layers[1].kv, spec, 16)
    assert k.shape == (5, 2, 8, 16, 8) and v.shape == (5, 2, 64, 16)
    # a fork takes the states and the last token along
    previous[1] = 123456
    caches.layers[2].state["matrix"][1] = 2.5
    e.copy_state([(1, 2)])
    assert previous.tolist() == [0, 123456, 123456] and (caches.layers[2].state["matrix"][2] == 2.5).all()


# ---- the restatement ----
def test_rows_of_the_pair_table():
    assert lizazen.bigram_rows([4, 9, 9, 0], {"buckets": 11, "mul_prev": 5, "mul_cur": 3}) == [11, (20 + 27) % 11, (45 + 27) % 11, 45 % 11]


def test_rotation_pairs_halves_and_depends_on_the_distance():
    r = lc.rot(8, 500.0)
    x = rand(5, 3, 12)
    y = lizazen.rotate(x, [0, 1, 7, 1000, 123456], r)
    assert torch.equal(y[..., 8:], x[..., 8:]) and torch.allclose(y[0], x[0]) and torch.allclose(y.norm(dim=-1), x.norm(dim=-1))
    e = lizazen.rotate(torch.eye(8, dtype=F64)[:1], [1], r)  # entry 0 turns towards entry 4
    assert torch.allclose(e[0, [0, 4]], torch.tensor([math.cos(1), math.sin(1)], dtype=F64)) and e[0].count_nonzero() == 2
    a, b = rand(1, 8, seed=1), rand(1, 8, seed=2)

    def score(p, q):
        return (lizazen.rotate(a, [p], r) * lizazen.rotate(b, [q], r)).sum()
    assert torch.allclose(score(9, 4), score(1009, 1004))


def test_frequency_scaling_regions():
    base = lizazen.frequencies(lc.rot(16, 1e4))
    got = lizazen.frequencies(lc.rot(16, 1e4, (8.0, 1.0, 4.0, 100)))
    turns = [100 * f / (2 * math.pi) for f in base]
    assert any(n > 4 for n in turns) and any(1 < n < 4 for n in turns) and any(n < 1 for n in turns)
    for f, g, n in zip(base, got, turns):
        if n > 4:
            assert g == f
        elif n < 1:
            assert g == f / 8
        else:
            assert f / 8 < g < f and math.isclose(g, f / 8 + (f - f / 8) * (n - 1) / 3)


def test_visible_keys():
    def seen(i, f, *a):
        return [j for j in range(12) if f(i, j, *a)]
    assert seen(9, lizazen.sees_window, 4) == [6, 7, 8, 9]
    assert seen(9, lizazen.sees_window, 3, 2) == [0, 1, 7, 8, 9] and seen(1, lizazen.sees_window, 1, 5) == [0, 1]
    assert seen(9, lizazen.sees_chunk, 4) == [8, 9] and seen(7, lizazen.sees_chunk, 4) == [4, 5, 6, 7] and seen(8, lizazen.sees_chunk, 4) == [8]


def test_attention_with_cap_and_sink():
    q, k, v = rand(6, 4, 5), rand(6, 2, 5, seed=1), rand(6, 2, 3, seed=2)
    sink = torch.tensor([0.3, -1.0, 2.0, 0.0], dtype=F64)
    got = lizazen.attend(q, k, v, 0.7, lambda i, j: lizazen.sees_window(i, j, 4), 1.5, sink)
    for i in range(6):
        for h in range(4):
            keys = range(max(0, i - 3), i + 1)
            e = torch.tensor([math.exp(1.5 * math.tanh(float(q[i, h] @ k[j, h // 2]) * 0.7 / 1.5)) for j in keys], dtype=F64)
            want = (e[:, None] * v[list(keys), h // 2]).sum(0) / (e.sum() + math.exp(sink[h]))
            assert torch.allclose(got[i, h], want)


def test_retention_is_a_decayed_sum():
    q, k, v = rand(7, 2, 3), rand(7, 2, 3, seed=1), rand(7, 2, 4, seed=2)
    got = lizazen.retain(q, k, v, [0.5, 1.0])
    for t in range(7):
        for h, w in enumerate((0.5, 1.0)):
            assert torch.allclose(got[t, h], sum(w ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1)))


def test_differential_weight_and_result():
    m = lc.diff(2, 1, 4, 6, 3, 1, lc.rot(4, 100.0), 0.5, 0.3)[1]
    w = {s: 0.5 * rand(4, seed=i) for i, s in enumerate(("lq1", "lk1", "lq2", "lk2"))}
    lam = lizazen.differential_weight(w.__getitem__, 0.3)
    assert torch.allclose(lam, (w["lq1"] @ w["lk1"]).exp() - (w["lq2"] @ w["lk2"]).exp() + 0.3)
    w.update(q=rand(16, 8, seed=5), k=rand(8, 8, seed=6), v=rand(6, 8, seed=7), o=torch.eye(12, dtype=F64))
    o = lizazen.differential_attention(rand(5, 8, seed=8), m, w.__getitem__, 1e-9).view(5, 2, 6)
    assert torch.allclose(o.pow(2).mean(-1), torch.full((5, 2), 0.49, dtype=F64))


def test_feed_forwards():
    g, u = torch.tensor([-9.0, 0.5, 9.0]), torch.tensor([0.3, -9.0, 9.0])
    a = lizazen.clamped_unit(g, u, 2.0)
    sig = torch.sigmoid
    assert torch.allclose(a, torch.stack([-9 * sig(torch.tensor(-9 * 1.702)) * 1.3, 0.5 * sig(torch.tensor(0.851)) * -1.0,
                                          2 * sig(torch.tensor(3.404)) * 3.0]))
    idx, s = lizazen.route(torch.tensor([[1.0, 5.0, 3.0, 4.0]], dtype=F64), 2)
    assert idx.tolist() == [[1, 3]] and torch.allclose(s, torch.sigmoid(torch.tensor([[5.0, 4.0]], dtype=F64)))


def changed(edit=None, patch=None, name="all", n=60):
    """Largest error of the restatement's logits after a planted change of the configuration or of a mechanism."""
    cfg, w = lc.case(name)
    t = tokens(cfg, n, 3)
    want = lizazen.forward(cfg, w, t)
    c = copy.deepcopy(cfg)
    if edit is not None:
        edit(c)
    with pytest.MonkeyPatch.context() as mp:
        if patch is not None:
            patch(mp)
        return error(lizazen.forward(c, w, t), want).max().item()


@pytest.mark.parametrize("name", ["all", "odd", "mfma"])
def test_an_edge_one_token_off_shows(name):
    for i, l in enumerate(lc.CONFIGS[name]["layers"]):
        for key in ("size", "keep_first"):
            m = l["mixer"].get("left", l["mixer"])["mask"]
            for by in (-1, 1):
                if key in m and m[key] + by > 0:
                    def edit(c):
                        c["layers"][i]["mixer"].get("left", c["layers"][i]["mixer"])["mask"][key] += by
                    assert changed(edit, name=name, n=150 if name == "mfma" else 90) > 2e-3, (i, key, by)


def test_planted_mistakes_show():
    def attend_with(**kw):
        def patch(mp):
            f = lizazen.attend
            mp.setattr(lizazen, "attend", lambda q, k, v, scale, sees, softcap=None, sink=None: f(
                q, k, v, scale, sees, **{**dict(softcap=softcap, sink=sink), **kw}))
        return patch

    def no_rotation(mp):
        mp.setattr(lizazen, "rotate", lambda x, p, r: x)

    def interleaved(mp):
        rotate = lizazen.rotate

        def f(x, p, r):
            perm = list(range(0, r["dims"], 2)) + list(range(1, r["dims"], 2)) + list(range(r["dims"], x.shape[-1]))
            out = torch.empty_like(x)
            out[..., perm] = rotate(x[..., perm], p, r)
            return out
        mp.setattr(lizazen, "rotate", f)

    def no_scaling(c):
        c["layers"][0]["mixer"]["rot"].pop("scaling")

    def one_softmax(mp):
        mp.setattr(lizazen, "differential_weight", lambda get, d: 0.0)

    def unclamped(mp):
        mp.setattr(lizazen, "clamped_unit", lambda g, u, limit: g * torch.sigmoid(1.702 * g) * (u + 1))

    def weights_on_the_output(mp):
        def f(h, mlp, get):
            idx, w = lizazen.route(h @ get("router").T, mlp["router"]["top"])
            out = lizazen.expert(h, get, "shared")
            for t in range(h.shape[0]):
                for e, s in zip(idx[t].tolist(), w[t]):
                    out[t] += s * lizazen.expert(h[t:t + 1], get, f"e{e}")[0]
            return out
        mp.setattr(lizazen, "mixture", f)

    def renormalised(mp):
        route = lizazen.route

        def f(z, top):
            i, w = route(z, top)
            return i, w / w.sum(-1, keepdim=True)
        mp.setattr(lizazen, "route", f)

    def no_start_row(mp):
        rows = lizazen.bigram_rows
        mp.setattr(lizazen, "bigram_rows", lambda t, b: [t[0] * b["mul_cur"] % b["buckets"]] + rows(t, b)[1:])

    def normed_values(mp):
        def f(h, m, get, eps):
            n, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
            q = lizazen.rms_norm(lizazen.project(h, get, "q", True), get("q.norm"), eps).view(n, H, d)
            k = lizazen.rms_norm(lizazen.project(h, get, "k", True), get("k.norm"), eps).view(n, G, d)
            o = lizazen.attend(lizazen.rotate(q, range(n), m["rot"]), lizazen.rotate(k, range(n), m["rot"]), k, m["scale"],
                               lambda i, j: lizazen.sees_window(i, j, m["mask"]["size"]), m["softcap"], get("sink"))
            return lizazen.project(o.reshape(n, -1), get, "o", True)
        mp.setattr(lizazen, "normed_attention", f)

    def no_bias(mp):
        mp.setattr(lizazen, "project", lambda h, get, name, bias: h @ get(name).T)

    def faster_decay(c):
        c["layers"][2]["mixer"]["right"]["decay"] = [0.8, 0.97, 0.997]
    for patch in (attend_with(softcap=None), attend_with(sink=None), no_rotation, interleaved, one_softmax, unclamped,
                  weights_on_the_output, renormalised, normed_values, no_bias):
        assert changed(patch=patch) > 1e-2, patch
    assert changed(patch=no_start_row, name="mfma") > 1e-2
    for edit in (no_scaling, faster_decay, lambda c: c["norm"].update(eps=1e-2), lambda c: c["layers"][1]["mixer"].update(diff=0.41)):
        assert changed(edit) > 1e-3, edit
