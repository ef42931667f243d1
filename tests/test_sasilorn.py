"""Sasilorn on the CPU: configuration, checkpoint reader, cache and state sizes, state slots beside the block manager, and
the consistency of the plain restatement the GPU tests compare with (its recurrences against closed forms, and planted
mistakes that the tests' weights must make visible)."""
import copy

import pytest
import torch

import sasilorn_case as sc
from oracle import sasilorn


def load(tmp_path, name, dtype=torch.float32):
    from light_vllm_amd.engine.registry import load_model_config
    cfg, w = sc.case(name)
    return load_model_config(sc.write_model(tmp_path / name, cfg, w), dtype)


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_configuration_gives_every_size(tmp_path, name):
    from light_vllm_amd.engine.hybrid_model import tensor_shapes
    cfg, w = sc.case(name)
    c = load(tmp_path, name)
    c.random_rank = 12
    assert tensor_shapes(c) == {k: tuple(t.shape) for k, t in w.items()}
    assert c.norm_eps == cfg["norm"]["eps"] and c.num_hidden_layers == len(cfg["layers"])
    for spec, state, layer in zip(c.kv_cache_specs(), c.state_specs(), cfg["layers"]):
        m = layer["mixer"]
        if layer["type"] == "parallel":
            assert (spec.kv_heads, spec.dim, spec.vdim) == (m["left"]["kv_heads"], m["left"]["dim"], m["left"]["vdim"])
            assert spec.kpad >= spec.dim and spec.vpad >= spec.vdim
            assert state == {"matrix": (m["right"]["heads"], m["right"]["dim"], m["right"]["vdim"])}
        else:
            assert spec is None and state == {"matrix": (m["heads"], m["dim"], m["dim"]), "shift": (cfg["width"],)}


def test_configuration_refuses_what_it_does_not_know():
    from light_vllm_amd.engine.hybrid_config import HybridModelConfig
    from light_vllm_amd.engine.registry import model_entry
    good = sc.CONFIGS["tied"]

    def broken(edit):
        c = copy.deepcopy(good)
        edit(c)
        with pytest.raises(ValueError):
            HybridModelConfig.from_dict(c)
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][2].update(weights_of=1))       # differs from the layer it names
    broken(lambda c: c["layers"][2].update(weights_of=2))       # itself
    broken(lambda c: c["layers"][2].update(weights_of=40))
    with pytest.raises(ValueError):
        model_entry("Unheard")


def test_weights_of_may_name_a_tied_or_a_later_layer():
    from light_vllm_amd.engine.hybrid_config import HybridModelConfig
    a = sc.wkv(2, 16)
    c = HybridModelConfig.from_dict(sc.model(64, 32, 1e-5, [sc.tied(a, 2), a, sc.tied(a, 1)]))
    assert [c.weights_layer(i) for i in range(3)] == [1, 1, 1]


def test_checkpoint_reader(tmp_path):
    from light_vllm_amd.engine.weights import load_checkpoint
    cfg, w = sc.case("odd")
    folder = sc.write_model(tmp_path, cfg, w)
    ckpt = load_checkpoint(folder)
    assert set(ckpt.keys()) == set(w)
    for name, t in w.items():
        assert ckpt[name].dtype == torch.bfloat16 and torch.equal(ckpt[name].float(), t)
    raw = (tmp_path / "model.safetensors").read_bytes()
    (tmp_path / "model.safetensors").write_bytes(raw[:-2])
    with pytest.raises(ValueError):
        load_checkpoint(folder)


def test_state_slots_are_given_back_and_forks_reserved():
    from light_vllm_amd.block_manager.state_slots import StateSlotManager
    m = StateSlotManager(3)
    a = m.allocate(1, 2)
    assert m.num_free() == 1 and m.can_allocate(1) and not m.can_allocate(2)
    m.allocate(2)
    with pytest.raises(RuntimeError):
        m.allocate(3)
    m.fork(1, 9)  # the reserved one
    assert m.take_copies() == [(a, m.slot_of(9))] and m.take_copies() == []
    m.free(1)
    m.free(1)
    assert m.num_free() == 1 and m.allocate(4) == a


def test_scheduler_admits_by_state_slots():
    """Plenty of blocks, two slots: the third request waits until one is given back."""
    from light_vllm_amd.engine.config import CacheConfig, SchedulerConfig
    from light_vllm_amd.engine.scheduler import DecodingScheduler
    from light_vllm_amd.engine.sequence import Sequence, SequenceGroup
    s = DecodingScheduler(SchedulerConfig(max_num_batched_tokens=256, max_num_seqs=8, max_model_len=256),
                          CacheConfig(num_gpu_blocks=64, num_cpu_blocks=0, num_state_slots=2))
    groups = [SequenceGroup(str(i), [Sequence(i, [1, 2, 3], 16)]) for i in range(3)]
    for g in groups:
        s.add_request(g)
    out = s.schedule()
    metas = out.seq_group_metadata_list
    assert [m.request_id for m in metas] == ["0", "1"]
    assert sorted(next(iter(m.state_slots.values())) for m in metas) == [0, 1]
    assert s.state_slots.num_free() == 0
    s.free_seq(groups[0].seqs[0])
    assert s.state_slots.num_free() == 1


# ---- the restatement itself ----
def test_gated_linear_attention_closed_form():
    g = torch.Generator().manual_seed(0)
    n, heads, d, e = 9, 2, 5, 3
    q, k, v = (torch.randn(n, heads, x, generator=g, dtype=torch.float64) for x in (d, d, e))
    alpha = torch.rand(n, heads, d, generator=g, dtype=torch.float64)
    o, s = sasilorn.gated_linear_attention(q, k, v, alpha)
    lp = torch.log(alpha).cumsum(0)
    for t in range(n):
        want = sum(((q[t] * k[j] * torch.exp(lp[t] - lp[j])).sum(-1, keepdim=True) * v[j]) for j in range(t + 1))
        assert torch.allclose(o[t], want)
    o2, s2 = sasilorn.gated_linear_attention(q[:4], k[:4], v[:4], alpha[:4])
    o3, s3 = sasilorn.gated_linear_attention(q[4:], k[4:], v[4:], alpha[4:], s2)
    assert torch.allclose(torch.cat([o2, o3]), o) and torch.allclose(s3, s)


def test_wkv_closed_form():
    g = torch.Generator().manual_seed(1)
    n, heads, d = 8, 2, 4
    r, k, v = (torch.randn(n, heads, d, generator=g, dtype=torch.float64) for _ in range(3))
    w = torch.rand(n, heads, d, generator=g, dtype=torch.float64)
    u = torch.randn(heads, d, generator=g, dtype=torch.float64)
    o, _ = sasilorn.wkv(r, k, v, w, u)
    lp = torch.log(w).cumsum(0)
    for t in range(n):
        want = (r[t] * u * k[t]).sum(-1, keepdim=True) * v[t]
        for j in range(t):  # decayed by the tokens strictly between
            want = want + (r[t] * k[j] * torch.exp(lp[t - 1] - lp[j])).sum(-1, keepdim=True) * v[j]
        assert torch.allclose(o[t], want)


def test_softmax_heads_against_torch():
    g = torch.Generator().manual_seed(2)
    q = torch.randn(7, 6, 5, generator=g, dtype=torch.float64)
    k, v = torch.randn(7, 2, 5, generator=g, dtype=torch.float64), torch.randn(7, 2, 3, generator=g, dtype=torch.float64)
    want = torch.nn.functional.scaled_dot_product_attention(
        q.transpose(0, 1), k.repeat_interleave(3, 1).transpose(0, 1), v.repeat_interleave(3, 1).transpose(0, 1),
        is_causal=True, scale=0.4).transpose(0, 1)
    assert torch.allclose(sasilorn.softmax_heads(q, k, v, 0.4), want)


MISTAKES = {
    "query heads interleaved over kv heads": ("softmax_heads", lambda f: lambda q, k, v, s: f(
        q.view(q.shape[0], -1, k.shape[1], q.shape[2]).transpose(1, 2).reshape(q.shape), k, v, s)),
    "first token unseen": ("softmax_heads", lambda f: lambda q, k, v, s: torch.cat(
        [f(q, k, v, s)[:1], f(q[1:], k[1:], v[1:], s)])),
    "bonus left out": ("wkv", lambda f: lambda r, k, v, w, u, state=None: f(r, k, v, w, torch.zeros_like(u), state)),
    "state lost at token 20": ("wkv", lambda f: lambda r, k, v, w, u, state=None: (
        torch.cat([f(r[:20], k[:20], v[:20], w[:20], u)[0], f(r[20:], k[20:], v[20:], w[20:], u)[0]]), None)),
    "linear state lost at token 20": ("gated_linear_attention", lambda f: lambda q, k, v, a, state=None: (
        torch.cat([f(q[:20], k[:20], v[:20], a[:20])[0], f(q[20:], k[20:], v[20:], a[20:])[0]]), None)),
    "shift lost at token 20": ("token_shift", lambda f: lambda h, mu, before=None: torch.cat([f(h[:20], mu), f(h[20:], mu)])),
    "tau ignored": ("gated_linear_decay", lambda f: lambda z, tau: f(z, 1.0)),
    "decay without its sign": ("wkv_decay", lambda f: lambda z: f(-z)),
    "relu not squared": ("squared_relu", lambda f: lambda x: torch.clamp(x, min=0)),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_mistakes_show_in_the_logits(monkeypatch, mistake):
    """What the GPU tests' tolerances (5e-5 in 32-bit, 0.1 in bfloat16 for the typical row) would catch."""
    name, wrap = MISTAKES[mistake]
    cfg, w = sc.case("tied")
    t, want = sc.expected("tied", 40, 3)
    monkeypatch.setattr(sasilorn, name, wrap(getattr(sasilorn, name)))
    assert sc.error(sasilorn.forward(cfg, w, t), want).max() > 0.05
