"""Lepalorn on the GPU: every operator and whole models against the plain float64 restatement (oracle/lepalorn.py) -- prompts,
portions, single tokens, mixed batches over reused pages, and generation through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

import layered_case
import lepalorn_case as lc
from lepalorn_case import dense_mixer, edge_inputs, mixer_case
from layered_case import engine, generate, play, portions, replay, tokens, write_model
from oracle import lepalorn

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
@pytest.mark.parametrize("rows,width", [(1, 4), (3, 7), (33, 96), (70, 250), (5, 1030), (2, 4096), (3, 1500), (2, 9000)])
@pytest.mark.parametrize("addend", ["rows", "slabs", "slots"])
def test_output_norm_and_depth_average(amd, dtype, rows, width, addend):
    x, gain, eps = rand(rows, width), torch.tensor([1.3]), 1e-3
    slots = weights = None
    if addend == "rows":
        y = rand(rows, width, seed=3, dtype=dtype)
        total = y.double()
    elif addend == "slabs":
        y = rand(3, rows, width, seed=4)
        total = y.double().sum(0)
    else:
        y = rand(3 * rows, width, seed=5, dtype=dtype)
        slots = torch.randperm(3 * rows, generator=torch.Generator().manual_seed(6)).view(rows, 3).int()
        weights = rand(rows, 3, seed=7)
        total = (y.double()[slots.long()] * weights.double()[:, :, None]).sum(1)
    v = x.double() + lepalorn.scalar_norm(total, 1.3, eps)
    dev = [t.to(DEV) if t is not None else None for t in (y, slots, weights)]
    tol = 2e-6 if dtype == F32 else 1e-2
    # in place, without a depth average
    xd = x.to(DEV)
    h = amd.norm_add_mix(xd, None, xd, *dev, gain.to(DEV), eps, None, None, None, dtype)
    close(xd, v, 3e-6, "x")
    close(h, v, tol, "h")
    # average over four streams and the new one, kept beside them; then the final norm
    streams, depth = torch.zeros(6, rows, width, device=DEV), rand(5, seed=8)
    streams[:4] = rand(4, rows, width, seed=9).to(DEV)
    avg = lepalorn.depth_average([*streams[:4].double().cpu(), v], depth.double())
    for final in (None, torch.tensor([0.7])):
        out = torch.zeros(rows, width, device=DEV)
        h = amd.norm_add_mix(out, streams[4], x.to(DEV), *dev, gain.to(DEV), eps, streams[:4], depth.to(DEV),
                             final.to(DEV) if final is not None else None, dtype)
        close(streams[4], v, 3e-6, "stream")
        close(out, avg, 3e-6, "average")
        close(h, avg if final is None else lepalorn.scalar_norm(avg, 0.7, eps), tol, "h")
        assert not streams[5].any()


@pytest.mark.parametrize("dtype", DTYPES)
def test_scaled_embedding(amd, dtype):
    table = rand(11, 37, dtype=dtype)
    ids = torch.tensor([3, 0, 10, 3])
    x = torch.zeros(4, 37, device=DEV)
    h = amd.embed_scale(x, table.to(DEV), ids.to(DEV), 7.3)
    close(x, table.double()[ids] * 7.3, 1e-6)
    assert torch.equal(h, x.to(dtype))


# ---- latent attention ----
SIZES = {  # heads, dim, rot_dim, rot_dims, vdim, kv_rank
    "small": (4, 24, 16, 16, 40, 48), "odd": (3, 13, 6, 4, 21, 35), "one head": (1, 32, 64, 64, 16, 128),
    "many heads": (33, 32, 32, 32, 64, 256), "large": (16, 128, 64, 64, 128, 512), "no class": (2, 40, 80, 80, 272, 544),
}
# (new tokens, context): portions of two and more, single tokens, both sides of the longest absorbed portion, page edges
LAYOUTS = {"decode": [(1, 0), (1, 15), (1, 16), (1, 90), (1, 333)], "short": [(2, 0), (2, 31), (16, 0), (5, 200), (64, 17)],
           "long": [(65, 0), (130, 3), (66, 150)], "mixed": [(1, 77), (100, 40), (2, 14), (64, 0), (97, 0), (1, 0)]}


def run_mixer(mixer, rows_by_seq, seqs, cache_blocks, dtype, seed, absorb_all=False):
    """The mixer over sequences whose contexts are put into the cache first; returns its output rows per sequence."""
    from light_vllm_amd.attention.latent_backend import LatentAttnImpl
    from light_vllm_amd.engine.latent_layers import LatentStep
    from light_vllm_amd.engine.mixers import StepLayout
    spec = mixer.spec
    perm = torch.randperm(cache_blocks, generator=torch.Generator().manual_seed(seed)).tolist()
    stride = spec.block_elements(16) + 256
    kv = torch.randn(cache_blocks, stride, device=DEV).to(dtype)[:, :spec.block_elements(16)]  # what freed pages may hold
    tables = [[perm.pop() for _ in range((n + c + 15) // 16)] for n, c in seqs]
    width = max(map(len, tables))
    bt = i32([t + [0] * (width - len(t)) for t in tables])

    def step(parts):  # (sequence, first, last)
        qlens = [b - a for _, a, b in parts]
        qsl, lens = layout([(b - a, a) for _, a, b in parts])
        slots = [tables[s][p // 16] * 16 + p % 16 for s, a, b in parts for p in range(a, b)]
        pos = torch.tensor([p for _, a, b in parts for p in range(a, b)], device=DEV)
        host = None if absorb_all else qlens
        l = StepLayout(qsl, lens, bt[[s for s, _, _ in parts]].contiguous(), torch.tensor(slots, device=DEV), None, max(qlens),
                       max(b for _, _, b in parts), 16, pos, host, None if absorb_all else [a for _, a, _ in parts])
        h = torch.cat([rows_by_seq[s][a:b] for s, a, b in parts]).to(dtype).to(DEV)
        out = mixer(h, kv, 0, LatentStep(l), LatentAttnImpl)
        y = (out.y.sum(0) if out.y.dim() == 3 else out.y).float().cpu()
        return list(y.split(qlens))
    for i, (n, c) in enumerate(seqs):
        if c:
            step([(i, 0, c)])
    return step([(i, c, c + n) for i, (n, c) in enumerate(seqs)])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", sorted(SIZES))
@pytest.mark.parametrize("name", sorted(LAYOUTS))
def test_latent_attention(amd, dtype, sizes, name):
    from light_vllm_amd.engine.latent_config import LatentAttentionConfig, RotationConfig
    from light_vllm_amd.engine.latent_layers import LatentAttention
    seqs, eps = LAYOUTS[name], 1e-5
    cfg, w = mixer_case(SIZES[sizes])
    for window in (1, 16, 50, 1000) if name != "mixed" else (33,):
        m = dict(cfg, mask={"size": window})
        c = LatentAttentionConfig(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"],
                                  RotationConfig(m["rot"]["dims"], m["rot"]["base"]), m["scale"], window)
        mixer = LatentAttention(lambda s: w[s[1:]].to(dtype).to(DEV), "", c, eps, True)
        assert mixer.expands == (dtype == BF16 and sizes != "no class")
        rows = [edge_inputs(m, w, n + ctx, window, 20 + i) for i, (n, ctx) in enumerate(seqs)]
        blocks = sum((n + ctx + 15) // 16 for n, ctx in seqs) + 2
        outs = {"": run_mixer(mixer, rows, seqs, blocks, dtype, 1)}
        if mixer.expands and name in ("long", "mixed"):
            outs["absorbed"] = run_mixer(mixer, rows, seqs, blocks, dtype, 2, absorb_all=True)
        for i, (n, ctx) in enumerate(seqs):
            h = rows[i].double()
            lat = lepalorn.latent_parts(h, m, lambda s: w[s].double(), eps)
            want = dense_mixer(h, m, w, lat, window)[ctx:]
            for way, got in outs.items():
                # (the last row's scores are the largest, and bfloat16 rounds queries and keys)
                close(got[i], want, 2e-5 if dtype == F32 else 1e-1, (window, n, ctx, way))
                if n > 1:
                    close(got[i][:-1], want[:-1], 2e-5 if dtype == F32 else 4e-2, (window, n, ctx, way))


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_from_the_start(amd, dtype):
    """Cached key parts and queries at positions up to a million."""
    from light_vllm_amd.engine.latent_config import RotationConfig
    from light_vllm_amd.engine.latent_layers import Rotation
    pos = [0, 1, 17, 4095, 131071, 1000003]
    heads, dim, rot, rank, dims, base = 3, 16, 24, 40, 20, 5e4
    inv = Rotation(RotationConfig(dims, base), DEV).turns
    kv, q = rand(6, rank + rot, seed=1, dtype=dtype), rand(6, heads * (dim + rot), seed=2, dtype=dtype)
    cache = torch.zeros(2, 16, 96, dtype=dtype, device=DEV)
    p = torch.tensor(pos, device=DEV)
    amd.latent_cache(cache, kv.to(DEV), torch.ones(rank, device=DEV), 1e-5, 64, p, inv, torch.tensor([3, -1, 20, 0, 31, 9], device=DEV))
    want = lepalorn.rotate(kv.double()[:, rank:], pos, dims, base)
    got = cache.view(32, 96)
    tol = 3e-7 if dtype == F32 else 5e-3
    for i, s in enumerate([3, None, 20, 0, 31, 9]):
        if s is not None:
            close(got[s, 64:64 + rot], want[i], tol, i)
            close(got[s, :rank], lepalorn.rms_norm(kv.double()[i, :rank], 1.0, 1e-5), tol, i)
    assert not got[:, rank:64].any() and not got[:, 64 + rot:].any()
    assert not got[[s for s in range(32) if s not in (3, 20, 0, 31, 9)]].any()
    out = amd.latent_rotate_query(q.to(DEV), heads, dim, 64, p, inv)
    qh = q.double().view(6, heads, dim + rot)
    close(out[..., dim:dim + rot], lepalorn.rotate(qh[..., dim:], pos, dims, base), tol)
    assert torch.equal(out[..., :dim].cpu(), q.view(6, heads, -1)[..., :dim]) and not out[..., dim + rot:].any()


@pytest.mark.parametrize("window", [1, 7, 16, 64, 200])
def test_windows_of_head_attention(amd, window):
    """Both matrix-core bodies and the plain one, a key at each side of the window's edge standing out."""
    from light_vllm_amd.attention.head_backend import HeadAttnImpl
    from light_vllm_amd.engine.hybrid_config import KVSpec
    seqs, scale = [(1, 0), (1, 250), (3, 61), (40, 5), (150, 130), (129, 0)], 0.125
    for dtype, heads, kv_heads, dim, vdim in ((BF16, 4, 2, 64, 64), (BF16, 3, 3, 128, 96), (F32, 4, 2, 20, 33)):
        spec = KVSpec(kv_heads, dim, vdim)
        blocks = sum((n + c + 15) // 16 for n, c in seqs)
        cache = torch.randn(blocks, spec.block_elements(16), device=DEV).to(dtype)
        kc, vc = HeadAttnImpl.split_kv_cache(cache, spec, 16)
        qs, wants, tables, at = [], [], [], 0
        for s, (n, c) in enumerate(seqs):
            t = n + c
            q, k, v = (rand(t, h, d, seed=10 * s + j, dtype=dtype) for j, (h, d) in
                       enumerate(((heads, dim), (kv_heads, dim), (kv_heads, vdim))))
            for j in (t - window, t - 1 - window):
                if 0 <= j < t - 1:
                    k[j, 0] = 3 * q[-1, 0]
            table = list(range(at, at + (t + 15) // 16))
            at += len(table)
            for p in range(t):
                kc[table[p // 16], :, :, p % 16] = F_pad(k[p], spec.kpad).view(kv_heads, -1, kc.shape[4]).to(DEV)
                vc[table[p // 16], :, :vdim, p % 16] = v[p].to(DEV)
            tables.append(table)
            qs.append(F_pad(q[c:], spec.kpad))
            g = heads // kv_heads
            i = torch.arange(t)
            seen = (i[:, None] >= i[None]) & (i[:, None] - i[None] < window)
            sc = (q.double().transpose(0, 1) @ k.double().repeat_interleave(g, 1).permute(1, 2, 0) * scale)
            o = sc.masked_fill(~seen, float("-inf")).softmax(-1) @ v.double().repeat_interleave(g, 1).transpose(0, 1)
            wants.append(o.transpose(0, 1)[c:].reshape(n, -1))
        qsl, lens = layout(seqs)
        w = max(map(len, tables))
        out = torch.full((int(qsl[-1]), heads * vdim), 9.0, dtype=dtype, device=DEV)
        amd.head_attention(out, torch.cat(qs).to(DEV).contiguous(), kc, vc, i32([t + [0] * (w - len(t)) for t in tables]), lens, qsl,
                           None, vdim, scale, 1.0, 150, 280, window, 3)
        row = 0
        for (n, c), want in zip(seqs, wants):
            if n < 3:
                assert (out[row:row + n] == 9.0).all()
            else:
                close(out[row:row + n], want, 1e-5 if dtype == F32 else 1.5e-2, (dtype, n, c))
            row += n


def F_pad(t, n):
    return torch.nn.functional.pad(t, (0, n - t.shape[-1]))


def F_rows(t, n):
    return torch.nn.functional.pad(t, (0, 0, 0, -t.shape[0] % n))


# ---- mixture of experts ----
def mixture_case(experts, top, width, ff, shared_ff, seed=0, bias=1.0):
    mlp = lc.moe(experts, top, ff, 1.3, shared_ff, 0.8)
    w = {"router": rand(experts, width, seed=seed + 1) * 2 * width ** -0.5, "router.b": bias * rand(experts, seed=seed + 2),
         "shared.sg": rand(1, width, seed=seed + 3) * 2 * width ** -0.5}
    for i, e in enumerate([f"e{j}" for j in range(experts)] + ["shared"]):
        n = shared_ff if e == "shared" else ff
        w[e + ".gate"], w[e + ".up"] = (rand(n, width, seed=seed + 10 + 3 * i + j) * 1.5 * width ** -0.5 for j in (0, 1))
        w[e + ".down"] = rand(width, n, seed=seed + 12 + 3 * i) * n ** -0.5
    return mlp, {k: t.bfloat16().float() for k, t in w.items()}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,width,ff,shared_ff", [(6, 1, 96, 40, 72), (5, 2, 90, 33, 90), (70, 7, 128, 64, 160), (3, 3, 64, 256, 16),
                                                          (16, 4, 320, 32, 32)])
def test_mixture_of_experts(amd, dtype, experts, top, width, ff, shared_ff):
    from light_vllm_amd.engine.latent_config import ExpertConfig, MixtureConfig
    from light_vllm_amd.engine.latent_layers import MixtureOfExperts
    for skew in (0.0, 30.0):  # 30: nearly every token takes the same experts
        mlp, w = mixture_case(experts, top, width, ff, shared_ff)
        w["router.b"] = (w["router.b"] + skew * (torch.arange(experts) < top)).bfloat16().float()
        moe = MixtureOfExperts(lambda s: w[s[1:]].to(dtype).to(DEV), "",
                               MixtureConfig(experts, top, ExpertConfig(ff, 1.3), ExpertConfig(shared_ff, 0.8)), True)
        assert moe.packed == (dtype == BF16 and width % 32 == 0)
        for rows in (1, 2, 17, 64, 65, 300):
            h = (1.5 * rand(rows, width, seed=50 + rows)).to(dtype)
            y, slots, weights = moe(h.to(DEV))
            y, slots, weights = y.double().cpu(), slots.long().cpu(), weights.double().cpu()
            assert sorted(slots.reshape(-1).tolist()) == list(range(rows * (top + 1)))
            got = (y[slots] * weights[:, :, None]).sum(1)
            close(got, lepalorn.mixture(h.double(), mlp, lambda s: w[s].double()), 1e-5 if dtype == F32 else 2e-2, (rows, skew))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,width", [(5, 24), (64, 256), (130, 90), (256, 128)])
def test_router(amd, dtype, experts, width):
    for rows in (1, 33, 200):
        h, w, b = rand(rows, width, seed=1, dtype=dtype), rand(experts + 1, width, seed=2, dtype=dtype), rand(experts, seed=3)
        z = h.double() @ w.double().T
        packed = dtype == BF16 and width % 32 == 0
        wd = amd.pack_weight(F_rows(w, 16).to(DEV)) if packed else w.to(DEV)
        for top in (1, 3, 5):
            ids, weights, *_ = amd.moe_route(h.to(DEV), wd, b.to(DEV), top, True, packed)
            want_ids, want_w = lepalorn.route(z[:, :experts] + b.double(), top)
            assert torch.equal(ids[:, :top].long().cpu(), want_ids) and (ids[:, top] == experts).all()
            close(weights[:, :top], want_w, 1e-5)
            close(weights[:, top], torch.sigmoid(z[:, experts]), 1e-5)
    # equal logits: the smaller numbers
    ids, weights, *_ = amd.moe_route(torch.zeros(2, width, dtype=dtype, device=DEV), wd, torch.zeros(experts, device=DEV), 4, True, packed)
    assert ids[:, :4].tolist() == [[0, 1, 2, 3]] * 2 and (weights == torch.tensor([0.25] * 4 + [0.5], device=DEV)).all()


# ---- whole models ----
LIMIT = {F32: 5e-5, BF16: 0.3}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {n: write_model(tmp_path_factory.mktemp(n), *lc.case(n)) for n in lc.CONFIGS}


def check_rows(got, want, dtype, what):
    e = layered_case.error(got, want)
    if dtype == F32:
        assert e.max() < LIMIT[F32], (what, e.argmax().item(), e.max().item())
    else:  # a row may be sensitive (two keys or experts of nearly equal score); most are not
        assert e.median() < LIMIT[BF16] / 3 and (e > LIMIT[BF16]).double().mean() <= 0.1, (what, e.median(), e.max(), (e > LIMIT[BF16]).double().mean())


@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_residual_stream_layer_by_layer(folders, name):
    cfg, w = lc.case(name)
    t = tokens(cfg, 37, 7)
    want, got = [], []
    lepalorn.forward(cfg, w, t, on_layer=lambda i, x: want.append(x))
    rp = replay(folders[name], F32, 64)
    forward = rp.engine.worker.model.forward
    rp.engine.worker.model.forward = lambda *a: forward(*a, on_layer=lambda i, x: got.append(x.cpu()))
    rp.step([("a", t, [])])
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        close(a, b, 2e-5, (name, "layer", i))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_prompts_portions_and_single_tokens(folders, dtype, name):
    """One sequence, cut in many ways.  The pages of each run are the ones the run before gave back."""
    t, want = lc.expected(name, 170, 1)
    rp = replay(folders[name], dtype, 192)
    cuts = {"whole": [170], "tokens": [1] * 170, "most, then tokens": [129] + [1] * 41, "twos": portions(170, [2]),
            "threes": portions(170, [3, 1, 16]), "mixed": portions(170, [15, 2, 33, 1, 1, 64, 7]), "long": [2, 66, 80, 22]}
    for cut, sizes in cuts.items():
        got = play(rp, {cut: t}, [[(cut, n)] for n in sizes])[cut]
        check_rows(got, want, dtype, (name, cut))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_batches_of_unequal_requests(folders, dtype, name):
    """Portions beside single tokens, requests that pause, end and leave their pages to others; each against the sequence
    alone, in a pool with no page to spare."""
    lens = {"a": 140, "b": 33, "c": 90, "d": 1, "e": 60, "f": 17}
    seqs = {r: lc.expected(name, n, 10 + i) for i, (r, n) in enumerate(lens.items())}
    steps = [[("a", 100)], [("b", 30), ("a", 1)], [("c", 2), ("a", 1), ("b", 1)], [("d", 1), ("c", 66)],
             [("b", 1), ("a", 20), ("c", 1)], [("a", 18), ("b", 1)],            # a and b end
             [("e", 37), ("c", 2), ("f", 16)], [("e", 1), ("c", 1)], [("f", 1), ("e", 1), ("c", 17)], [("e", 19), ("c", 1)],
             [("e", 2)]]
    rp = replay(folders[name], dtype, 384)
    got = play(rp, {r: t for r, (t, _) in seqs.items()}, steps)
    for r, (_, want) in seqs.items():
        check_rows(got[r], want, dtype, (name, r))
    assert not rp.groups


def test_long_decoding(folders):
    t, want = lc.expected("shared", 400, 2)
    rp = replay(folders["shared"], F32, 448)
    got = play(rp, {"a": t}, [[("a", 20)]] + [[("a", 1)]] * 380)["a"]
    check_rows(got, want, F32, "long")


def greedy(cfg, w, prompt, n):
    return layered_case.greedy(lambda t: lepalorn.forward(cfg, w, t), prompt, n)


@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_greedy_generation(folders, name):
    """The engine's own scheduler and captured steps, 32-bit, against the restatement's arg-max: whole prompts, portions of
    prompts beside decoded tokens (captured together, and not), recomputed and swapped sequences in a pool too small for
    all, several steps in flight, blocks shared through the prefix cache."""
    cfg, w = lc.case(name)
    prompts = [tokens(cfg, n, 50 + n) for n in (5, 31, 1, 48, 16)]
    prompts.append(prompts[3][:40] + prompts[0])
    want = [greedy(cfg, w, p, 8) for p in prompts]
    folder = folders[name]
    assert generate(engine(folder, F32), prompts, 8) == want
    assert generate(engine(folder, F32, graph=False, chunked=True, budget=24), prompts, 8) == want
    assert generate(engine(folder, F32, chunked=True, budget=24, max_seqs=3), prompts, 8) == want
    assert generate(engine(folder, F32, num_blocks=13, preemption_mode="recompute"), prompts, 8) == want
    assert generate(engine(folder, F32, num_blocks=13, preemption_mode="swap"), prompts, 8) == want
    assert generate(engine(folder, F32, scheduling="async", max_seqs=3), prompts, 8, use_async=True) == want
    assert generate(engine(folder, F32, max_seqs=1, cache=dict(enable_prefix_caching=True)), prompts, 8) == want


def test_bfloat16_steps_captured_and_not(folders):
    cfg, _ = lc.case("mfma")
    prompts = [tokens(cfg, n, 80 + n) for n in (5, 31, 1, 48, 16)]
    a = generate(engine(folders["mfma"], BF16, graph=False), prompts, 24)
    assert generate(engine(folders["mfma"], BF16), prompts, 24) == a
    assert generate(engine(folders["mfma"], BF16, use_v2_block_manager=True, num_scheduler_steps=4), prompts, 24) == a


def test_several_sequences_per_prompt(folders):
    """Forked sequences: their log-probabilities are the restatement's for their own tokens."""
    from light_vllm_amd.engine.sampling_params import SamplingParams
    cfg, w = lc.case("shared")
    p = tokens(cfg, 21, 90)
    eng = engine(folders["shared"], F32, graph=False)
    eng.add_request("0", p, sampling_params=SamplingParams(n=3, temperature=1.0, seed=3, max_tokens=6, logprobs=1))
    outs = []
    while eng.has_unfinished_requests():
        outs += [o for o in eng.step() if o.finished]
    eng.shutdown()
    seqs = outs[-1].outputs
    assert len(seqs) == 3 and len({tuple(s) for s in seqs}) > 1
    sums = []
    for ids in seqs:
        lp = lepalorn.forward(cfg, w, p + list(ids)).log_softmax(-1)
        sums.append(sum(lp[len(p) - 1 + j, tok].item() for j, tok in enumerate(ids)))
        if list(ids) == list(outs[-1].token_ids):
            for j, (tok, d) in enumerate(zip(ids, outs[-1].logprobs)):
                assert abs(d[tok][0] - lp[len(p) - 1 + j, tok].item()) < 1e-3
    assert all(x >= y - 1e-3 for x, y in zip(sums, sums[1:]))


def test_refuses_a_quantised_cache(folders):
    with pytest.raises(ValueError):
        engine(folders["odd"], BF16, cache=dict(cache_dtype="fp8"))


def test_programs(folders, tmp_path):
    """bin/generate and bin/trace_run as a user starts them."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg, w = lc.case("odd")
    t, want = lc.expected("odd", 30, 5)
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
