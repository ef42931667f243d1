"""Lepalorn on the CPU: configuration, cache sizes, the plan of long portions, and the plain restatement the GPU tests compare
with (closed forms, and planted mistakes that the tests' weights must make visible)."""
import copy

import pytest
import torch

import lepalorn_case as lc
from layered_case import error, tokens, write_model
from oracle import lepalorn


def load(tmp_path, name, dtype=torch.float32):
    from light_vllm_amd.engine.registry import load_model_config
    return load_model_config(write_model(tmp_path / name, *lc.case(name)), dtype)


@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_configuration_gives_every_size(tmp_path, name):
    from light_vllm_amd.engine.latent_model import LatentModel
    cfg, w = lc.case(name)
    c = load(tmp_path, name)
    assert LatentModel.tensor_shapes(c) == {k: tuple(t.shape) for k, t in w.items()}
    assert (c.norm_eps, c.embedding_scale, c.vocab_size) == (cfg["norm"]["eps"], cfg["embedding"]["scale"], cfg["vocab"])
    assert c.state_specs() is None and c.num_hidden_layers == len(cfg["layers"])
    for i, (spec, l, d) in enumerate(zip(c.kv_cache_specs(), c.layers, cfg["layers"])):
        m = d["mixer"]
        assert (l.mixer.window, l.mixer.scale, l.mixer.rot.base) == (m["mask"]["size"], m["scale"], m["rot"]["base"])
        if "kv_from" in m:
            assert spec is None and c.kv_layer(i) == m["kv_from"]
        else:
            assert (spec.kv_rank, spec.rot_dim) == (m["kv_rank"], m["rot_dim"]) and c.kv_layer(i) == i
            assert spec.cpad >= m["kv_rank"] and spec.rpad >= m["rot_dim"] and spec.block_elements(16) == 16 * (spec.cpad + spec.rpad)
        if d["mlp"] is not None:
            assert (l.mlp.top, l.mlp.expert.limit, l.mlp.shared.ff) == (
                d["mlp"]["router"]["top"], d["mlp"]["expert"]["limit"], d["mlp"]["shared"]["ff"])


def test_configuration_refuses_what_it_does_not_know():
    from light_vllm_amd.engine.latent_config import LatentModelConfig
    good = lc.CONFIGS["shared"]
    LatentModelConfig.from_dict(good)

    def broken(edit):
        c = copy.deepcopy(good)
        edit(c)
        with pytest.raises(ValueError):
            LatentModelConfig.from_dict(c)
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_from=1))            # itself
    broken(lambda c: c["layers"][1]["mixer"].update(kv_from=2))            # later
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=1))            # has no cache of its own
    broken(lambda c: c["layers"][1]["mixer"].update(kv_rank=40))           # another latent
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(base=6e3))      # another rotation
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18))
    with pytest.raises(ValueError):
        LatentModelConfig.from_dict(good, dtype=torch.float16)


def test_cache_has_a_buffer_per_layer_with_a_latent_of_its_own(tmp_path):
    from light_vllm_amd.attention.latent_backend import LatentAttnBackend, LatentAttnImpl
    from light_vllm_amd.engine.cache_engine import CacheEngine
    from light_vllm_amd.engine.config import CacheConfig
    c = load(tmp_path, "shared", torch.bfloat16)
    cc = CacheConfig(num_gpu_blocks=5, num_cpu_blocks=2)
    e = CacheEngine(cc, c, LatentAttnBackend(), "cpu")
    own = [s for s in c.kv_cache_specs() if s is not None]
    assert len(e.gpu_cache) == len(own) == 2
    assert CacheEngine.get_cache_block_size(cc, c) == sum(s.block_elements(16) * 2 for s in own)
    caches = e.model_caches()
    assert [x.kv is None for x in caches.layers] == [s is None for s in c.kv_cache_specs()]
    view = LatentAttnImpl.rows_view(e.gpu_cache[1], own[1], 16)
    view[3, 2, 1] = 7.0
    assert view.shape == (5, 16, own[1].row) and e.gpu_cache[1][3, 2 * own[1].row + 1] == 7.0


def test_plan_of_long_portions():
    from light_vllm_amd.engine.latent_layers import plan_long_portions
    assert plan_long_portions([1, 64, 2], [500, 0, 7], 100, 64, 16, "cpu") is None
    p = plan_long_portions([1, 100, 2, 65], [500, 210, 7, 0], 50, 64, 16, "cpu")
    # sequence 1 sees keys 161 .. 309, taken from 160 on; sequence 3 keys 0 .. 64
    assert p.starts.tolist() == [0, 0, 160, 160, 240] and p.n == 240
    assert p.first[1] == 160 and p.first[3] == 0
    assert p.seq_lens.tolist() == [1, 150, 2, 65] and p.max_seq_len == 150
    assert p.tables[1].tolist() == list(range(10)) and p.tables[3].tolist()[:5] == list(range(10, 15))
    assert p.tables.max() < p.n // 16


def test_interleaved_experts():
    from light_vllm_amd.engine.latent_layers import interleave_16
    g, u = torch.arange(40.)[:, None] + 1, -torch.arange(40.)[:, None] - 1
    w = interleave_16(g, u)[:, 0]
    assert w.shape == (128,)
    for n in range(64):
        t, r = divmod(n, 16)
        assert w[32 * t + r] == (n + 1 if n < 40 else 0) and w[32 * t + 16 + r] == (-n - 1 if n < 40 else 0)


# ---- the restatement ----
def test_rotation_is_a_rotation():
    gen = torch.Generator().manual_seed(0)
    x = torch.randn(5, 3, 12, generator=gen, dtype=torch.float64)
    y = lepalorn.rotate(x, [0, 1, 7, 1000, 123456], 8, 500.0)
    assert torch.equal(y[..., 8:], x[..., 8:]) and torch.equal(y[0], x[0])
    assert torch.allclose(y.norm(dim=-1), x.norm(dim=-1))
    # scores depend on the distance alone, and positive angles turn (1, 0) towards (0, 1)
    a, b = torch.randn(1, 8, generator=gen, dtype=torch.float64), torch.randn(1, 8, generator=gen, dtype=torch.float64)

    def score(p, q):
        return (lepalorn.rotate(a, [p], 8, 500.0) * lepalorn.rotate(b, [q], 8, 500.0)).sum()
    assert torch.allclose(score(9, 4), score(1009, 1004))
    e = lepalorn.rotate(torch.tensor([[1.0, 0.0]], dtype=torch.float64), [1], 2, 500.0)
    assert e[0, 1] > 0.8


def test_window_attention_is_masked_attention():
    gen = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(23, 2, d, generator=gen, dtype=torch.float64) for d in (6, 6, 4))
    i = torch.arange(23)
    seen = (i[:, None] >= i[None]) & (i[:, None] - i[None] < 7)
    s = torch.einsum("ihd,jhd->hij", q, k) * 0.4
    want = torch.einsum("hij,jhe->ihe", s.masked_fill(~seen, float("-inf")).softmax(-1), v)
    assert torch.allclose(lepalorn.window_attention(q, k, v, 0.4, 7), want)


def test_router_and_activation():
    z = torch.tensor([[1.0, 5.0, 3.0, 4.0]], dtype=torch.float64)
    idx, w = lepalorn.route(z, 2)
    assert idx.tolist() == [[1, 3]] and torch.allclose(w, torch.softmax(torch.tensor([[5.0, 4.0]], dtype=torch.float64), -1))
    g, u = torch.tensor([-9.0, 0.5, 9.0]), torch.tensor([0.3, -9.0, 9.0])
    a = lepalorn.clamped_gate(g, u, 2.0)
    sig = torch.sigmoid
    assert torch.allclose(a, torch.stack([-9 * sig(torch.tensor(-9 * 1.702)) * 1.3, 0.5 * sig(torch.tensor(0.851)) * -1.0,
                                          2 * sig(torch.tensor(3.404)) * 3.0]))


def test_depth_average_and_norm():
    xs = [torch.full((1, 2), float(i)) for i in range(3)]
    assert torch.equal(lepalorn.depth_average(xs, torch.tensor([5.0, 0.5, 2.0])), torch.full((1, 2), 4.5))
    x = torch.tensor([[3.0, 4.0]], dtype=torch.float64)
    assert torch.allclose(lepalorn.scalar_norm(x, 2.0, 0.5), x * 2 / 13.0 ** 0.5)


def changed(edit_cfg=None, patch=None, name="shared", n=60):
    """Largest error of the restatement's logits after a planted change."""
    cfg, w = lc.case(name)
    t = tokens(cfg, n, 3)
    want = lepalorn.forward(cfg, w, t)
    c = copy.deepcopy(cfg)
    if edit_cfg is not None:
        edit_cfg(c)
    with pytest.MonkeyPatch.context() as mp:
        if patch is not None:
            patch(mp)
        return error(lepalorn.forward(c, w, t), want).max().item()


@pytest.mark.parametrize("name", ["shared", "odd", "mfma"])
@pytest.mark.parametrize("by", [-1, 1])
def test_a_window_one_token_off_shows(name, by):
    for i in range(len(lc.CONFIGS[name]["layers"])):
        if name == "mfma" and i:
            continue
        assert changed(lambda c: c["layers"][i]["mixer"]["mask"].update(
            size=c["layers"][i]["mixer"]["mask"]["size"] + by), name=name, n=90) > 1e-3, i


def test_planted_mistakes_show():
    def no_rotation(mp):
        mp.setattr(lepalorn, "rotate", lambda x, p, d, b: x)

    def half_layout(mp):
        rotate = lepalorn.rotate

        def f(x, p, d, b):
            perm = [j // 2 + (j % 2) * (d // 2) for j in range(d)]
            y = rotate(x[..., perm], p, d, b)
            out = x.clone()
            out[..., perm] = y
            return out
        mp.setattr(lepalorn, "rotate", f)

    def unclamped(mp):
        mp.setattr(lepalorn, "clamped_gate", lambda g, u, limit: g * torch.sigmoid(1.702 * g) * (u + 1))

    def plain_silu(mp):
        mp.setattr(lepalorn, "clamped_gate", lambda g, u, limit: g.clamp(max=limit) * torch.sigmoid(g.clamp(max=limit)) *
                   (u.clamp(-limit, limit) + 1))

    def softmax_over_all(mp):
        def f(z, top):
            v, i = torch.topk(torch.softmax(z, -1), top, dim=-1)
            return i, v
        mp.setattr(lepalorn, "route", f)

    def last_stream_only(mp):
        mp.setattr(lepalorn, "depth_average", lambda xs, w: w[-1] * xs[-1])
    for patch in (no_rotation, half_layout, unclamped, plain_silu, softmax_over_all, last_stream_only):
        assert changed(patch=patch) > 1e-2, patch.__name__
    assert changed(lambda c: c["layers"][4]["mixer"].update(kv_from=2) or c["embedding"].update(scale=3.1)) > 1e-3
    assert changed(lambda c: c["norm"].update(eps=1e-2)) > 1e-4


@pytest.mark.parametrize("window", [1, 16, 50])
@pytest.mark.parametrize("sizes", [(3, 24, 16, 16, 40, 48), (16, 128, 64, 64, 128, 512)])
def test_edge_inputs_show_both_sides_of_a_window(sizes, window):
    """The inputs the operator tests use: a window one token longer or shorter changes the last row by far more than they
    allow."""
    cfg, w = lc.mixer_case(sizes)
    h = lc.edge_inputs(cfg, w, 90, window, 5).double()
    lat = lepalorn.latent_parts(h, cfg, lambda s: w[s].double(), 1e-5)
    want = lc.dense_mixer(h, cfg, w, lat, window)[-1]
    assert torch.allclose(want, lepalorn.latent_attention(h, dict(cfg, mask={"size": window}), lambda s: w[s].double(), lat)[-1])
    for other in (window - 1, window + 1):
        if other > 0:
            got = lc.dense_mixer(h, cfg, w, lat, other)[-1]
            assert (got - want).abs().max() > 0.12 * want.abs().max(), other
