"""Sasilorn on the GPU: every operator and whole models against the plain float64 restatement (oracle/sasilorn.py) --
prompts, portions, single tokens, mixed batches over reused pages and slots, and generation through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

import layered_case
import sasilorn_case as sc
from layered_case import engine, generate
from oracle import sasilorn

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]


@pytest.fixture(scope="module")
def amd():
    import light_vllm_amd  # noqa: F401
    from light_vllm_amd import _custom_ops  # noqa: F401
    return torch.ops._C_amd


def i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def layout(seqs):
    """seqs: (new tokens, context) -> query_start_loc, seq_lens on the device."""
    qsl = [0]
    for n, _ in seqs:
        qsl.append(qsl[-1] + n)
    return i32(qsl), i32([n + c for n, c in seqs])


def rand(*shape, seed=0, dtype=F32):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


def close(got, want, rtol, what=""):
    """Worst difference against the largest expected value."""
    want = want.double()
    err = (got.double().cpu() - want).abs().max().item() / (want.abs().max().item() + 1e-30)
    assert err <= rtol, (what, err)


# ---- row-wise operators ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 4), (3, 7), (33, 96), (70, 250), (5, 1024)])
@pytest.mark.parametrize("addend", ["none", "rows", "slabs"])
def test_dynamic_tanh(amd, dtype, rows, width, addend):
    x, w, b, alpha = rand(rows, width), rand(width, seed=1), rand(width, seed=2), torch.tensor([0.63])
    y = {"none": None, "rows": rand(rows, width, seed=3, dtype=dtype), "slabs": rand(3, rows, width, seed=4)}[addend]
    total = x.double()
    if y is not None:
        total = total + (y.double() if addend == "rows" else y.sum(0).to(dtype).double())
    xd = x.to(DEV)
    h = amd.add_dyt(xd, None if y is None else y.to(DEV), alpha.to(DEV), w.to(DEV), b.to(DEV), dtype)
    close(xd, total, 1e-6 if addend != "slabs" or dtype == F32 else 4e-3)
    close(h, sasilorn.dynamic_tanh(total, 0.63, w.double(), b.double()), 1e-6 if dtype == F32 else 8e-3)


LAYOUTS = {
    "prompt": [(37, 0)],
    "singles": [(1, 5), (1, 0), (1, 900)],
    "portions": [(2, 3), (16, 16), (17, 31), (3, 0)],
    "mixed": [(50, 7), (33, 0), (1, 64), (1, 1), (2, 1)],
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(LAYOUTS))
@pytest.mark.parametrize("width", [96, 90])
def test_token_shift(amd, dtype, name, width):
    seqs = LAYOUTS[name]
    qsl, lens = layout(seqs)
    rows = sum(n for n, _ in seqs)
    x, y, mu = rand(rows, width), rand(rows, width, seed=1, dtype=dtype), torch.rand(5, width)
    w, b, alpha = rand(width, seed=2), rand(width, seed=3), torch.tensor([0.8])
    carried = rand(9, width, seed=4)
    slots = [7, 2, 5, 0, 8][:len(seqs)]
    cd = carried.to(DEV)
    x_out, mix = amd.add_dyt_shift_mix(x.to(DEV), y.to(DEV), mu.to(DEV), alpha.to(DEV), w.to(DEV), b.to(DEV), cd, i32(slots),
                                       qsl, lens, dtype)
    total = x.double() + y.double()
    h = sasilorn.dynamic_tanh(total, 0.8, w.double(), b.double())
    close(x_out, total, 1e-6)
    at = 0
    after = carried.double().clone()
    for (n, ctx), slot in zip(seqs, slots):
        before = carried[slot].double() if ctx else None
        for m in range(5):
            close(mix[m, at:at + n], sasilorn.token_shift(h[at:at + n], mu[m].double(), before), 2e-6 if dtype == F32 else 8e-3)
        after[slot] = h[at + n - 1]
        at += n
    close(cd, after, 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 24, 1000])
def test_relu_squared(amd, dtype, n):
    x = rand(n, dtype=dtype)
    out = torch.empty_like(x, device=DEV)
    amd.relu_squared(out, x.to(DEV))
    close(out, sasilorn.squared_relu(x.double()), 1e-6 if dtype == F32 else 8e-3)


@pytest.mark.parametrize("m,n,k", [(1, 64, 96), (33, 160, 256), (64, 4096, 1024), (32, 512, 14336)])
def test_relu_squared_in_the_projection(amd, m, n, k):
    """Bit for bit the projection followed by the activation, with K inside a workgroup and split over several."""
    x, w = rand(m, k, dtype=BF16).to(DEV), (rand(n, k, seed=1) * k ** -0.5).bfloat16().to(DEV)
    packed = amd.pack_weight(w)
    want = amd.skinny_linear_packed(x, packed, None, n, k)
    amd.relu_squared(want, want)
    assert torch.equal(amd.skinny_linear_packed_relu_squared(x, packed, n, k), want)


# ---- recurrences ----
def recurrence_case(kind, seqs, heads, dk, dv, rank, spread, dtype, seed=0):
    rows = sum(n for n, _ in seqs)
    c = dict(q=rand(rows, heads * dk, seed=seed, dtype=dtype), k=rand(rows, heads * dk, seed=seed + 1, dtype=dtype),
             v=rand(rows, heads * dv, seed=seed + 2, dtype=dtype), u=rand(rows, rank, seed=seed + 3, dtype=dtype),
             gate=rand(rows, heads * dv, seed=seed + 4, dtype=dtype), a=rand(heads * dk, rank, seed=seed + 5) * 0.3,
             bias=rand(heads * dk, seed=seed + 6) * spread + (-2.0 if kind == 1 else 1.0),
             bonus=rand(heads, dk, seed=seed + 7) if kind == 1 else None,
             norm=rand(dv if kind == 0 else heads * dv, seed=seed + 8), state=rand(6, heads, dk, dv, seed=seed + 9))
    return c, rows


def recurrence_expected(c, kind, tau, q_scale, eps, out_scale, seqs, slots, heads, dk, dv):
    d = {k: (v.double() if torch.is_tensor(v) else v) for k, v in c.items()}
    state, outs, decays, at = d["state"].clone(), [], [], 0
    for (n, ctx), slot in zip(seqs, slots):
        s = slice(at, at + n)
        at += n
        u = d["u"][s]
        z = (torch.tanh(u) if kind == 1 else u) @ d["a"].T + d["bias"]
        w = (sasilorn.wkv_decay(z) if kind == 1 else sasilorn.gated_linear_decay(z, tau)).view(n, heads, dk)
        q, k, v = d["q"][s].view(n, heads, dk) * q_scale, d["k"][s].view(n, heads, dk), d["v"][s].view(n, heads, dv)
        s0 = state[slot] if ctx else None
        o, state[slot] = (sasilorn.wkv(q, k, v, w, d["bonus"], s0) if kind == 1
                          else sasilorn.gated_linear_attention(q, k, v, w, s0))
        o = sasilorn.rms_norm(o, eps)
        o = o * d["norm"] if kind == 0 else (o.reshape(n, -1) * d["norm"]).view(n, heads, dv)
        outs.append(o.reshape(n, -1) * sasilorn.silu(d["gate"][s]) * out_scale)
    return torch.cat(outs), state


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", [0, 1])
@pytest.mark.parametrize("name", sorted(LAYOUTS))
@pytest.mark.parametrize("heads,dk,dv,rank,spread", [(3, 24, 40, 12, 1.0), (1, 10, 7, 5, 2.0), (2, 64, 64, 16, 2.0),
                                                     (2, 128, 128, 33, 4.0), (1, 200, 50, 16, 1.0), (2, 256, 16, 64, 3.0)])
def test_recurrence(amd, dtype, kind, name, heads, dk, dv, rank, spread):
    """Both decays, read-outs with and without a bonus, states read from and written to scattered slots; `spread` up to
    channels that forget within a token next to ones that never do."""
    from light_vllm_amd.engine.mixers import LowRankDecay, Recurrence, StepLayout
    seqs, tau, eps = LAYOUTS[name], 3.0, 1e-4
    c, rows = recurrence_case(kind, seqs, heads, dk, dv, rank, spread, dtype)
    slots = [4, 1, 5, 0, 3][:len(seqs)]
    qsl, lens = layout(seqs)
    step = StepLayout(qsl, lens, None, None, i32(slots), max(n for n, _ in seqs), max(sum(s) for s in seqs), 16)
    want, want_state = recurrence_expected(c, kind, tau, dk ** -0.5, eps, 0.7, seqs, slots, heads, dk, dv)
    dev = {k: (v.to(DEV) if torch.is_tensor(v) else v) for k, v in c.items()}
    decay = LowRankDecay(dev["a"], dev["bias"], kind, 1.0 / tau if kind == 0 else 1.0)
    for fused in (True, False):
        rec = Recurrence(decay, dev["bonus"], eps)
        rec.fused = fused
        state, out = dev["state"].clone(), torch.empty(rows, heads * dv, dtype=dtype, device=DEV)
        rec(out, dev["q"], dev["k"], dev["v"], dev["u"], dev["gate"], dev["norm"], 0.7, dk ** -0.5, state, step)
        close(out, want, 3e-5 if dtype == F32 else 8e-3, ("out", fused))
        close(state, want_state, 5e-6, ("state", fused))


def test_slow_decays_beside_fast_ones(amd):
    """A token that wipes a channel out must not disturb the decays of the tokens around it."""
    from light_vllm_amd.engine.mixers import LowRankDecay, Recurrence, StepLayout
    n, dk = 40, 64
    c, _ = recurrence_case(1, [(n, 0)], 1, dk, dk, 1, 0.0, F32)
    c["u"].zero_()
    c["u"][5], c["u"][22] = 20.0, 20.0     # tanh = 1: these tokens decay by exp(-exp(bias + a))
    c["a"].fill_(14.0)
    c["bias"].fill_(-6.0)
    want, want_state = recurrence_expected(c, 1, 1.0, 1.0, 1e-5, 1.0, [(n, 0)], [2], 1, dk, dk)
    dev = {k: v.to(DEV) for k, v in c.items()}
    qsl, lens = layout([(n, 0)])
    out = torch.empty(n, dk, device=DEV)
    Recurrence(LowRankDecay(dev["a"], dev["bias"], 1), dev["bonus"], 1e-5)(
        out, dev["q"], dev["k"], dev["v"], dev["u"], dev["gate"], dev["norm"], 1.0, 1.0, dev["state"],
        StepLayout(qsl, lens, None, None, i32([2]), n, n, 16))
    close(out, want, 3e-5)
    close(dev["state"][2], want_state[2], 5e-6)


def test_a_sequence_without_a_slot_leaves_the_states_alone(amd):
    from light_vllm_amd.engine.mixers import LowRankDecay, Recurrence, StepLayout
    for seqs in ([(20, 0)], [(1, 0)]):
        c, n = recurrence_case(0, seqs, 2, 16, 16, 4, 1.0, F32)
        want, _ = recurrence_expected(c, 0, 1.0, 1.0, 1e-5, 1.0, seqs, [0], 2, 16, 16)
        dev = {k: (v.to(DEV) if torch.is_tensor(v) else v) for k, v in c.items()}
        qsl, lens = layout(seqs)
        out = torch.empty(n, 32, device=DEV)
        Recurrence(LowRankDecay(dev["a"], dev["bias"], 0), None, 1e-5)(
            out, dev["q"], dev["k"], dev["v"], dev["u"], dev["gate"], dev["norm"], 1.0, 1.0, dev["state"],
            StepLayout(qsl, lens, None, None, i32([-1]), n, n, 16))
        close(out, want, 3e-5)
        assert torch.equal(dev["state"].cpu(), c["state"])


# ---- softmax heads over the paged cache ----
ATTENTION_LAYOUTS = {
    "prompts": [(150, 0), (64, 0), (1, 0), (17, 0)],
    "singles": [(1, 300), (1, 15), (1, 16), (1, 0), (1, 63)],
    "short portions": [(2, 47), (3, 16), (5, 200), (2, 0)],
    "mixed": [(100, 37), (40, 129), (2, 31), (1, 255), (1, 64)],
    "long": [(1, 3000), (2, 1500)],
}


def attention_inputs(seqs, heads, kv_heads, dim, vdim, seed=0):
    """Each query row points at one key: a page's first or last, the sequence's first, its own, the one before it, or the
    next one (which it must not see)."""
    g = torch.Generator().manual_seed(seed)
    out = []
    for n, ctx in seqs:
        total = n + ctx
        k = torch.randn(total, kv_heads, dim, generator=g)
        v = torch.randn(total, kv_heads, vdim, generator=g)
        q = 0.3 * torch.randn(total, heads, dim, generator=g)
        for i in range(total):
            for h in range(heads):
                page = i // 16 * 16
                targets = (0, i, max(i - 1, 0), page, max(page - 1, 0), min(i + 1, total - 1), max(page - 17, 0),
                           int(torch.randint(0, i + 1, (1,), generator=g)))
                q[i, h] += k[targets[(i + 3 * h) % 8], h // (heads // kv_heads)]
        out.append((q, k, v))
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(ATTENTION_LAYOUTS))
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(6, 2, 40, 24), (3, 3, 20, 33), (20, 1, 128, 64), (4, 1, 72, 200),
                                                     (2, 1, 300, 48), (2, 2, 64, 256)])
def test_softmax_heads(amd, dtype, name, heads, kv_heads, dim, vdim):
    from light_vllm_amd.attention.head_backend import HeadAttnImpl
    from light_vllm_amd.engine.hybrid_config import KVSpec
    seqs = ATTENTION_LAYOUTS[name]
    if name == "long" and heads * dim > 256:
        pytest.skip("covered by the narrower sizes")
    ins = attention_inputs(seqs, heads, kv_heads, dim, vdim)
    ins = [tuple(t.to(dtype).float() for t in x) for x in ins]
    scale, eps, out_scale = 1.2 * dim ** -0.5, 1e-5, 0.6
    qw, kw = 1.6 + 0.1 * rand(dim, seed=5), 1.6 + 0.1 * rand(dim, seed=6)
    spec = KVSpec(kv_heads, dim, vdim)
    n_blocks = sum((n + c + 15) // 16 for n, c in seqs) + 3
    perm = torch.randperm(n_blocks, generator=torch.Generator().manual_seed(1)).tolist()
    stride = spec.block_elements(16) + 256
    cache = torch.randn(n_blocks, stride, device=DEV).to(dtype)[:, :spec.block_elements(16)]  # what freed pages may hold
    kc, vc = HeadAttnImpl.split_kv_cache(cache, spec, 16)
    tables = [[perm.pop() for _ in range((n + c + 15) // 16)] for n, c in seqs]
    width = max(map(len, tables))
    bt = i32([t + [0] * (width - len(t)) for t in tables])

    def put(rows_q, rows_k, rows_v, slots):
        r = len(slots)
        flat = torch.cat([x.reshape(r, -1) for x in (rows_q, rows_k, rows_v)], 1).to(dtype).to(DEV)
        a, b = heads * dim, heads * dim + kv_heads * dim
        return amd.qk_norm_cache(flat[:, :a], flat[:, a:b], flat[:, b:], qw.to(DEV), kw.to(DEV), eps, heads, kv_heads, kc, vc,
                                 torch.tensor(slots, dtype=torch.int64, device=DEV))
    new_q = [[], [], [], []]
    for (n, ctx), (q, k, v), table in zip(seqs, ins, tables):
        slots = [table[p // 16] * 16 + p % 16 for p in range(n + ctx)]
        if ctx:
            put(q[:ctx], k[:ctx], v[:ctx], slots[:ctx])
        for lst, t in zip(new_q, (q[ctx:], k[ctx:], v[ctx:], slots[ctx:])):
            lst.append(t)
    q = put(torch.cat(new_q[0]), torch.cat(new_q[1]), torch.cat(new_q[2]), sum(new_q[3], []))
    rows = q.shape[0]
    gate = rand(rows, heads + 8, seed=7, dtype=dtype)
    qsl, lens = layout(seqs)
    out = torch.zeros(rows, heads * vdim + 16, dtype=dtype, device=DEV)
    amd.head_attention(out[:, :heads * vdim], q, kc, vc, bt, lens, qsl, gate.to(DEV)[:, :heads], vdim, scale, out_scale,
                       max(n for n, _ in seqs), max(sum(s) for s in seqs))
    assert not out[:, heads * vdim:].any()
    at = 0
    for (n, ctx), (q, k, v) in zip(seqs, ins):
        qn = sasilorn.rms_norm(q.double(), eps, qw.double())
        kn = sasilorn.rms_norm(k.double(), eps, kw.double())
        if dtype == BF16:  # (stored in 16 bits)
            qn, kn = qn.bfloat16().double(), kn.bfloat16().double()
        want = dense_rows(qn, kn, v.double(), scale, ctx) * torch.sigmoid(gate[at:at + n, :heads].double())[:, :, None] * out_scale
        close(out[at:at + n, :heads * vdim], want.reshape(n, -1), 1e-5 if dtype == F32 else 1e-2, (n, ctx))
        at += n


def dense_rows(q, k, v, scale, first):
    """The restatement's softmax heads for rows first .. (its own loop takes every row)."""
    if first == 0 and q.shape[0] < 40:
        return sasilorn.softmax_heads(q, k, v, scale)
    n, heads, group = q.shape[0], q.shape[1], q.shape[1] // k.shape[1]
    kk, vv = k.repeat_interleave(group, 1).transpose(0, 1), v.repeat_interleave(group, 1).transpose(0, 1)
    s = q[first:].transpose(0, 1) @ kk.transpose(1, 2) * scale
    s.masked_fill_(torch.arange(n)[None, :] > torch.arange(first, n)[:, None], float("-inf"))
    return (s.softmax(-1) @ vv).transpose(0, 1)


# ---- whole models ----
LIMIT = {F32: 5e-5, BF16: 0.3}  # (these weights' gains make bfloat16 rounding 0.03 to 0.2 of the logits' spread)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {n: sc.write_model(tmp_path_factory.mktemp(n), *sc.case(n)) for n in sc.CONFIGS}


def check_rows(got, want, dtype, what):
    e = sc.error(got, want)
    if dtype == F32:
        assert e.max() < LIMIT[F32], (what, e.argmax().item(), e.max().item())
    else:  # a row may be sensitive (two keys of nearly equal score); most are not
        assert e.median() < LIMIT[BF16] / 3 and (e > LIMIT[BF16]).double().mean() <= 0.04, (what, e.median(), e.max())


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_residual_stream_layer_by_layer(folders, name):
    """32-bit: the stream after every layer, and with the unfused recurrence as well."""
    cfg, w = sc.case(name)
    t = sc.tokens(cfg, 37, 7)
    want = []
    sasilorn.forward(cfg, w, t, on_layer=lambda i, x: want.append(x))
    for fused in (True, False):
        rp = sc.replay(folders[name], F32, 64)
        model, got = rp.engine.worker.model, []
        for _, mixer, _ in model.layers:
            mixer.recurrence.fused = fused
        forward = model.forward
        model.forward = lambda *a: forward(*a, on_layer=lambda i, x: got.append(x.cpu()))
        rp.step([("a", t, [])])
        assert len(got) == len(want)
        for i, (a, b) in enumerate(zip(got, want)):
            close(a, b, 2e-5, (name, "layer", i, fused))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_prompts_portions_and_single_tokens(folders, dtype, name):
    """One sequence, cut in many ways: whole, token by token, portions of two and other sizes.  The pages and the slot of
    each run are the ones the run before gave back."""
    t, want = sc.expected(name, 170, 1)
    rp = sc.replay(folders[name], dtype, 192)
    cuts = {"whole": [170], "tokens": [1] * 170, "most, then tokens": [129] + [1] * 41, "twos": sc.portions(170, [2]),
            "threes": sc.portions(170, [3, 1, 16]), "mixed": sc.portions(170, [15, 2, 33, 1, 1, 64, 7])}
    for cut, sizes in cuts.items():
        got = sc.play(rp, {cut: t}, [[(cut, n)] for n in sizes])[cut]
        check_rows(got, want, dtype, (name, cut))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_batches_of_unequal_requests(folders, dtype, name):
    """Portions beside single tokens, requests that pause, end and leave their pages and slots to others; each against the
    sequence alone, in a pool with no page to spare."""
    lens = {"a": 140, "b": 33, "c": 90, "d": 1, "e": 60, "f": 17}
    seqs = {r: sc.expected(name, n, 10 + i) for i, (r, n) in enumerate(lens.items())}
    steps = [[("a", 100)], [("b", 30), ("a", 1)], [("c", 2), ("a", 1), ("b", 1)], [("d", 1), ("c", 60)],
             [("b", 1), ("a", 20), ("c", 1)], [("a", 18), ("b", 1)],            # a and b end
             [("e", 37), ("c", 2), ("f", 16)], [("e", 1), ("c", 1)], [("f", 1), ("e", 1), ("c", 23)], [("e", 19), ("c", 1)],
             [("e", 2)]]
    rp = sc.replay(folders[name], dtype, 384)
    got = sc.play(rp, {r: t for r, (t, _) in seqs.items()}, steps)
    for r, (_, want) in seqs.items():
        check_rows(got[r], want, dtype, (name, r))
    assert not rp.groups and rp.engine.scheduler.state_slots.num_free() == 4


def test_long_decoding(folders):
    t, want = sc.expected("tied", 700, 2)
    rp = sc.replay(folders["tied"], F32, 704)
    got = sc.play(rp, {"a": t}, [[("a", 20)]] + [[("a", 1)]] * 680)["a"]
    check_rows(got, want, F32, "long")


def greedy(cfg, w, prompt, n):
    return layered_case.greedy(lambda t: sasilorn.forward(cfg, w, t), prompt, n)


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_greedy_generation(folders, name):
    """The engine's own scheduler and captured decode steps, 32-bit, against the restatement's arg-max: whole prompts,
    portions of prompts beside decoded tokens, recomputed and swapped sequences in a pool too small for all, several steps
    in flight."""
    cfg, w = sc.case(name)
    prompts = [sc.tokens(cfg, n, 50 + n) for n in (5, 31, 1, 48, 16)]
    want = [greedy(cfg, w, p, 10) for p in prompts]
    folder = folders[name]
    assert generate(engine(folder, F32), prompts, 10) == want
    assert generate(engine(folder, F32, graph=False, chunked=True, budget=24), prompts, 10) == want
    assert generate(engine(folder, F32, chunked=True, budget=24, max_seqs=3), prompts, 10) == want
    assert generate(engine(folder, F32, num_blocks=11, preemption_mode="recompute"), prompts, 10) == want
    assert generate(engine(folder, F32, num_blocks=11, preemption_mode="swap"), prompts, 10) == want
    assert generate(engine(folder, F32, scheduling="async", max_seqs=3), prompts, 10, use_async=True) == want


def test_bfloat16_steps_captured_and_not(folders):
    cfg, _ = sc.case("mfma")
    prompts = [sc.tokens(cfg, n, 80 + n) for n in (5, 31, 1, 48, 16)]
    a = generate(engine(folders["mfma"], BF16, graph=False), prompts, 24)
    assert generate(engine(folders["mfma"], BF16), prompts, 24) == a
    assert generate(engine(folders["mfma"], BF16, use_v2_block_manager=True, num_scheduler_steps=4), prompts, 24) == a


def test_several_sequences_per_prompt(folders):
    """Forked sequences take copies of the prompt's state: their log-probabilities are the restatement's for their own
    tokens."""
    from light_vllm_amd.engine.sampling_params import SamplingParams
    cfg, w = sc.case("tied")
    p = sc.tokens(cfg, 21, 90)
    eng = engine(folders["tied"], F32, graph=False)
    eng.add_request("0", p, sampling_params=SamplingParams(n=3, temperature=1.0, seed=3, max_tokens=6, logprobs=1))
    outs = []
    while eng.has_unfinished_requests():
        outs += [o for o in eng.step() if o.finished]
    eng.shutdown()
    seqs = outs[-1].outputs
    assert len(seqs) == 3 and len({tuple(s) for s in seqs}) > 1
    sums = []
    for ids in seqs:
        lp = sasilorn.forward(cfg, w, p + list(ids)).log_softmax(-1)
        sums.append(sum(lp[len(p) - 1 + j, tok].item() for j, tok in enumerate(ids)))
        if list(ids) == list(outs[-1].token_ids):
            for j, (tok, d) in enumerate(zip(ids, outs[-1].logprobs)):
                assert abs(d[tok][0] - lp[len(p) - 1 + j, tok].item()) < 1e-3
    assert all(x >= y - 1e-3 for x, y in zip(sums, sums[1:]))  # ranked by what each sequence's own state said


def test_programs(folders, tmp_path):
    """bin/generate and bin/trace_run as a user starts them."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg, w = sc.case("odd")
    t, want = sc.expected("odd", 30, 5)
    r = subprocess.run([sys.executable, f"{root}/bin/generate", "--model", folders["odd"], "--dtype", "float32",
                        "--max-tokens", "4", "--num-gpu-blocks", "16", ",".join(map(str, t[:9]))],
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert json.loads(r.stdout.splitlines()[-1])["token_ids"] == greedy(cfg, w, t[:9], 4)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:25], "want": [3, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": t[25:27], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": t[27:], "want": [2, 0]}], "end": ["x"]}]
    r = subprocess.run([f"{root}/bin/trace_run", "--model", folders["odd"], "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", "64"], input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True,
                       timeout=100)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "2.f32"]
    for step, places in ((0, [3, 24]), (2, [29, 27])):
        got = torch.frombuffer(bytearray((tmp_path / f"{step}.f32").read_bytes()), dtype=F32).view(len(places), -1)
        check_rows(got, want[places], F32, step)
