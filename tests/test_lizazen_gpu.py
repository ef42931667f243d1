"""Lizazen on the GPU: every operator and whole models against the plain float64 restatement (oracle/lizazen.py) -- prompts,
portions, single tokens, mixed batches over reused pages and slots, and generation through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

import layered_case
import lizazen_case as lc
from layered_case import engine, generate, play, portions, replay, tokens, write_model
from oracle import lizazen

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64
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
    return lc.rand(*shape, seed=seed).to(dtype)


def close(got, want, rtol, what=""):
    """Worst difference against the largest expected value."""
    want = want.double()
    err = (got.double().cpu() - want).abs().max().item() / (want.abs().max().item() + 1e-30)
    assert err <= rtol, (what, err)


def pad(t, n):
    return torch.nn.functional.pad(t, (0, n - t.shape[-1]))


# ---- row-wise operators ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 4), (3, 7), (33, 96), (70, 250), (5, 1030), (2, 4096), (300, 1500), (2, 9000)])
@pytest.mark.parametrize("kind", ["rows", "slabs", "slots", "two", "two slabs"])
def test_norms_around_a_sublayer(amd, dtype, rows, width, kind):
    eps, x = 1e-3, rand(rows, width)
    w, nw, b0, w0, w1 = (1 + 0.3 * rand(width, seed=20 + i) for i in range(5))
    slabs = "slabs" in kind
    y = rand(3, rows, width, seed=3) if slabs else rand(rows, width, seed=3, dtype=dtype)
    total, slots = y.double().sum(0) if slabs else y.double(), None
    if kind == "slots":
        y = rand(3 * rows, width, seed=5, dtype=dtype)
        slots = torch.randperm(3 * rows, generator=torch.Generator().manual_seed(6)).view(rows, 3).int()
        total = y.double()[slots.long()].sum(1)
    bias = b0 if kind in ("slabs", "two") else None
    if bias is not None:
        total = total + b0.double()
    other, other_w, own_w = None, None, None
    if kind.startswith("two"):
        other = (30 * rand(2, rows, width, seed=8)) if slabs else (30 * rand(rows, width, seed=8)).to(dtype)
        other_w, own_w = w1, w0
        o = other.double().sum(0) if slabs else other.double()
        total = (lizazen.rms_norm(total, w0.double(), eps) + lizazen.rms_norm(o, w1.double(), eps)) / 2
    want = x.double() + lizazen.rms_norm(total, w.double(), eps)
    dev = [t.to(DEV) if t is not None else None for t in (y, slots, bias, own_w, other, None, other_w, w, nw)]
    xd = x.to(DEV)
    h = amd.sandwich_norm(xd, *dev, eps, dtype)
    close(xd, want, 3e-6, "x")
    close(h, lizazen.rms_norm(want, nw.double(), eps), 3e-6 if dtype == F32 else 1e-2, "h")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [37, 96])
def test_embedding_of_token_pairs(amd, dtype, width):
    """Portions of several sequences: the token before a portion comes from the slot, which then holds its last one."""
    vocab, eps, bigram = 61, 1e-4, {"buckets": 29, "mul_prev": 5, "mul_cur": 3}
    table, pairs, w = rand(vocab, width, dtype=dtype), rand(30, width, seed=1, dtype=dtype), 1 + 0.2 * rand(width, seed=2)
    seqs = [torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (9, 1, 14, 6)]
    previous = i32([60, 59, 58, 57, 56])
    slots, at = [3, 0, 4, 1], [0] * 4
    for step in ([(0, 4), (2, 1)], [(1, 1), (0, 1), (2, 9)], [(3, 2), (0, 4)], [(2, 4), (3, 1)], [(3, 3)]):
        ids = [t for s, n in step for t in seqs[s][at[s]:at[s] + n]]
        qsl, lens = layout([(n, at[s]) for s, n in step])
        x = torch.full((len(ids), width), 7.0, device=DEV)
        h = amd.pair_embed(x, table.to(DEV), pairs.to(DEV), torch.tensor(ids, device=DEV), previous, i32([slots[s] for s, _ in step]),
                           qsl, lens, 5, 3, w.to(DEV), eps)
        want = torch.cat([table.double()[seqs[s]][at[s]:at[s] + n]
                          + pairs.double()[lizazen.bigram_rows(seqs[s], bigram)][at[s]:at[s] + n] for s, n in step])
        close(x, want, 1e-6)
        close(h, lizazen.rms_norm(want, w.double(), eps), 2e-6 if dtype == F32 else 1e-2)
        for s, n in step:
            at[s] += n
            assert previous[slots[s]] == seqs[s][at[s] - 1]
    assert previous[2] == 58  # nobody's
    # rows of a captured step without a sequence: nothing is read or kept
    before = previous.clone()
    x = torch.zeros(2, width, device=DEV)
    amd.pair_embed(x, table.to(DEV), pairs.to(DEV), torch.tensor([4, 5], device=DEV), previous, i32([-1, -1]), i32([0, 1, 2]),
                   i32([5, 1]), 5, 3, w.to(DEV), eps)
    assert torch.equal(before, previous)
    close(x, table.double()[[4, 5]] + pairs.double()[29], 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,limit", [(96, 72, 0.8), (90, 33, 2.0), (2048, 160, 1.2), (64, 4096, 0.5), (512, 512, 1e9)])
def test_clamped_feed_forward(amd, dtype, width, ff, limit):
    from light_vllm_amd.engine.local_config import ClampedMlpConfig
    from light_vllm_amd.engine.local_layers import ClampedMlp
    w = {"gate": rand(ff, width, seed=1) * 1.5 * width ** -0.5, "up": rand(ff, width, seed=2) * 1.5 * width ** -0.5,
         "down": rand(width, ff, seed=3) * ff ** -0.5}
    w = {k: t.bfloat16().float() for k, t in w.items()}
    mlp = ClampedMlp(lambda s: w[s[1:]].to(dtype).to(DEV), "", ClampedMlpConfig(ff, limit), True)
    for rows in (1, 5, 33, 64, 65, 300):
        h = rand(rows, width, seed=rows, dtype=dtype)
        y = mlp(h.to(DEV)).y
        want = lizazen.dense(h.double(), {"limit": limit}, lambda s: w[s].double())
        close(y.sum(0) if y.dim() == 3 else y, want, 1e-5 if dtype == F32 else 1.5e-2, rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,width,ff,shared_ff", [(6, 1, 96, 40, 72), (5, 2, 90, 33, 90), (70, 7, 128, 64, 160), (3, 3, 64, 256, 16),
                                                          (130, 4, 320, 32, 0)])
def test_mixture_of_experts(amd, dtype, experts, top, width, ff, shared_ff):
    """Sigmoid scores on what the experts read; a plain shared expert, or none."""
    from light_vllm_amd.engine.local_layers import MixtureMlp
    from light_vllm_amd.engine.moe import ExpertConfig, MixtureConfig
    w = {"router": rand(experts, width, seed=1) * 2 * width ** -0.5}
    for i, e in enumerate([f"e{j}" for j in range(experts)] + ["shared"] * (shared_ff > 0)):
        n = shared_ff if e == "shared" else ff
        w[e + ".gate"], w[e + ".up"] = (rand(n, width, seed=10 + 3 * i + j) * 1.5 * width ** -0.5 for j in (0, 1))
        w[e + ".down"] = rand(width, n, seed=12 + 3 * i) * n ** -0.5
    w = {k: t.bfloat16().float() for k, t in w.items()}
    cfg = MixtureConfig(experts, top, ExpertConfig(ff), ExpertConfig(shared_ff) if shared_ff else None, "sigmoid", "silu", False,
                        False, True)
    moe = MixtureMlp(lambda s: w[s[1:]].to(dtype).to(DEV), "", cfg, True)
    assert moe.packed == (dtype == BF16 and width % 32 == 0)
    n = top + (shared_ff > 0)
    for rows in (1, 2, 17, 64, 65, 300):
        h = (1.5 * rand(rows, width, seed=50 + rows)).to(dtype)
        y, _, slots = moe(h.to(DEV))
        y, slots = y.double().cpu(), slots.long().cpu()
        assert sorted(slots.reshape(-1).tolist()) == list(range(rows * n))
        mlp = lc.moe(experts, top, ff, shared_ff)
        with pytest.MonkeyPatch.context() as mp:
            if not shared_ff:
                expert = lizazen.expert
                mp.setattr(lizazen, "expert", lambda x, get, e: torch.zeros_like(x) if e == "shared" else expert(x, get, e))
            want = lizazen.mixture(h.double(), mlp, lambda s: w[s].double())
        close(y[slots].sum(1), want, 1e-5 if dtype == F32 else 2e-2, rows)


def test_router_scores(amd):
    for dtype, experts, width in ((F32, 5, 24), (BF16, 64, 256), (BF16, 130, 90), (BF16, 256, 128)):
        for rows in (1, 33, 200):
            h, w = rand(rows, width, seed=1, dtype=dtype), rand(experts, width, seed=2, dtype=dtype) * width ** -0.5
            w = w.to(dtype)
            packed = dtype == BF16 and width % 32 == 0
            wd = amd.pack_weight(torch.nn.functional.pad(w, (0, 0, 0, -experts % 16)).to(DEV)) if packed else w.to(DEV)
            for top in (1, 5):
                ids, weights, _, token, slots, _, by_slot = amd.moe_route(h.to(DEV), wd, None, top, True, packed, experts, False, 1, True)
                want_ids, want = lizazen.route(h.double() @ w.double().T, top)
                assert torch.equal(ids[:, :top].long().cpu(), want_ids) and (ids[:, top] == experts).all()
                close(weights[:, :top], want, 1e-5)
                assert (weights[:, top] == 1).all()
                assert torch.equal(by_slot[slots.long()], weights)
                assert torch.equal(token[slots.long()], torch.arange(rows, device=DEV, dtype=torch.int32)[:, None].expand(-1, top + 1))


# ---- what goes into the cache ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,maps,dims,norm,own_v", [
    (4, 2, 64, 96, 1, 64, False, True), (3, 1, 13, 21, 1, 6, False, True), (6, 3, 40, 40, 1, 24, True, False), (5, 5, 10, 10, 1, 2, True, False),
    (4, 2, 24, 40, 2, 24, False, True), (3, 1, 7, 11, 2, 6, False, True), (8, 1, 128, 128, 1, 32, True, False), (2, 2, 96, 64, 2, 0, False, True)])
@pytest.mark.parametrize("scaled", [False, True])
def test_rotated_queries_keys_and_cached_values(amd, dtype, heads, kv_heads, dim, vdim, maps, dims, norm, own_v, scaled):
    """At positions up to a million; rows without a slot, padding and everything else in the cache."""
    from light_vllm_amd.attention.head_backend import HeadAttnImpl
    from light_vllm_amd.engine.hybrid_config import KVSpec
    from light_vllm_amd.engine.local_config import FrequencyScaling, RotaryConfig
    from light_vllm_amd.engine.local_layers import turns_of
    s = (8.0, 1.0, 4.0, 200.0)
    r = lc.rot(dims, 5e4, s if scaled else None)
    turns = turns_of(RotaryConfig(dims, 5e4, FrequencyScaling(*s) if scaled else None), DEV)
    for rows in (6, 130):
        pos = [0, 1, 17, 4095, 131071, 1000003] + list(range(40, 40 + rows - 6))
        slots = [3, -1, 20, 0, 31, 9] + list(range(48, 48 + rows - 6))
        qkv = rand(rows, (heads + kv_heads) * maps * dim + kv_heads * vdim + 5, seed=1, dtype=dtype).to(DEV)
        a, b = heads * maps * dim, (heads + kv_heads) * maps * dim
        q, k = qkv[:, :a], qkv[:, a:b]
        v = qkv[:, b:b + kv_heads * vdim] if own_v else k
        spec = KVSpec(kv_heads, dim, vdim, maps)
        cache = torch.full((12, spec.block_elements(16)), 7.0, dtype=dtype, device=DEV)
        kc, vc = HeadAttnImpl.split_kv_cache(cache, spec, 16)
        wq, wk = ((1 + 0.3 * rand(t.shape[1], seed=9 + i)) for i, t in enumerate((q, k)))
        out = amd.rotary_cache(q, k, v, wq.to(DEV) if norm else None, wk.to(DEV) if norm else None, 1e-3, heads, kv_heads, maps,
                               torch.tensor(pos, device=DEV), turns, kc, vc, torch.tensor(slots, device=DEV))
        qh, kh, vh = (t.double().cpu() for t in (q, k, v))
        if norm:
            qh, kh = lizazen.rms_norm(qh, wq.double(), 1e-3), lizazen.rms_norm(kh, wk.double(), 1e-3)
        qh, kh = (lizazen.rotate(t.view(rows, -1, dim), pos, r) for t in (qh, kh))
        tol, mpad = 4e-7 if dtype == F32 else 5e-3, spec.kpad // maps
        got = out.view(rows, heads * maps, mpad)
        close(got[..., :dim], qh, tol, "q")
        assert not got[..., dim:].any()
        # [slots, kv head, map, entry]
        ks = kc.permute(0, 3, 1, 2, 4).reshape(192, kv_heads * maps, mpad)
        vs = vc.permute(0, 3, 1, 2).reshape(192, kv_heads, spec.vpad)
        used = [i for i in slots if i >= 0]
        rows_used = [i for i, s_ in enumerate(slots) if s_ >= 0]
        close(ks[used][..., :dim], kh[rows_used], tol, "k")
        assert torch.equal(vs[used][..., :vdim].double().cpu(), vh.view(rows, kv_heads, vdim)[rows_used])
        assert not ks[used][..., dim:].any() and not vs[used][..., vdim:].any()
        rest = [i for i in range(192) if i not in used]
        assert (ks[rest] == 7).all() and (vs[rest] == 7).all()


# ---- attention ----
def put_keys(kc, vc, table, k, v, spec):
    """k [n, kv_heads * maps, dim], v [n, kv_heads, vdim] of one sequence into its pages."""
    n, G = k.shape[0], spec.kv_heads
    for p in range(n):
        row = pad(k[p], spec.kpad // spec.maps).reshape(G, -1)
        kc[table[p // 16], :, :, p % 16] = row.view(G, -1, kc.shape[4]).to(DEV)
        vc[table[p // 16], :, :, p % 16] = pad(v[p], spec.vpad).to(DEV)


# heads, kv heads, dim, vdim
HEADS = {"mfma": (8, 2, 64, 64), "group of one": (3, 3, 96, 128), "many heads": (33, 1, 32, 32), "wide": (4, 2, 128, 256), "odd": (5, 1, 13, 21),
         "no class": (2, 2, 272, 48)}
SEQS = [(1, 0), (1, 250), (2, 61), (3, 0), (40, 5), (150, 130), (129, 0), (1, 16), (17, 47)]


@pytest.mark.parametrize("maps", [1, 2])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", sorted(HEADS))
@pytest.mark.parametrize("window,chunk,keep,softcap,sink", [(1, 0, 0, 0.0, False), (16, 0, 0, 0.0, True), (50, 0, 6, 0.0, False),
                                                            (64, 0, 70, 0.0, False), (0, 64, 0, 0.0, False), (0, 19, 0, 5.0, False),
                                                            (200, 0, 0, 8.0, True), (0, 1, 0, 0.0, True), (33, 100, 17, 3.0, True)])
def test_attention_over_what_a_query_sees(amd, maps, dtype, sizes, window, chunk, keep, softcap, sink):
    """All bodies; the last token of every sequence looks for the keys at both sides of every edge, each in a head of its own."""
    from light_vllm_amd.attention.head_backend import HeadAttnImpl
    from light_vllm_amd.engine.hybrid_config import KVSpec
    H, G, dim, vdim = HEADS[sizes]
    scale, spec = 2.0 * dim ** -0.5, KVSpec(G, dim, vdim, maps)
    gen = torch.Generator().manual_seed(5)
    blocks = sum((n + c + 15) // 16 for n, c in SEQS) + 3
    cache = (5 * torch.randn(blocks, spec.block_elements(16), generator=gen)).to(dtype).to(DEV)  # what freed pages may hold
    kc, vc = HeadAttnImpl.split_kv_cache(cache, spec, 16)
    perm = torch.randperm(blocks, generator=gen).tolist()
    sinks = rand(H, seed=3) + 1.5 if sink else None

    def sees(i, j):
        low = max(i - window + 1 if window else 0, i - i % chunk if chunk else 0)
        return j <= i and (j >= low or j < keep)
    qs, wants, tables = [], [], []
    for s, (n, c) in enumerate(SEQS):
        t = n + c
        q, k = rand(t, H * maps, dim, seed=10 * s, dtype=dtype), rand(t, G * maps, dim, seed=10 * s + 1, dtype=dtype)
        v = rand(t, G, vdim, seed=10 * s + 2, dtype=dtype)
        edges = [t - 1 - window, t - window] if window else []
        edges += [(t - 1) - (t - 1) % chunk, (t - 1) - (t - 1) % chunk - 1] if chunk else []
        edges += [0, keep - 1, keep] if keep else []
        for e, j in enumerate(j for j in edges if 0 <= j < t - 1):
            k[j, e % (G * maps)] = (1.5 * q[-1, e % (G * maps) * (H // G)].float()).to(dtype) if maps == 1 else k[j, 0] + 1
        table = [perm.pop() for _ in range((t + 15) // 16)]
        put_keys(kc, vc, table, k, v, spec)
        tables.append(table)
        qs.append(pad(q[c:], spec.kpad // maps).reshape(n, H, spec.kpad))
        qd, kd = q.double().view(t, H, maps, dim), k.double().view(t, G, maps, dim)
        o = [lizazen.attend(qd[:, :, i], kd[:, :, i], v.double(), scale, sees, softcap or None,
                            sinks.double() if sink else None) for i in range(maps)]
        o = o[0] if maps == 1 else lizazen.rms(o[0] - 0.37 * o[1], 1e-2) * 0.6
        wants.append(o[c:].reshape(n, -1))
    qsl, lens = layout(SEQS)
    w = max(map(len, tables))
    out = torch.full((int(qsl[-1]), H * vdim), 9.0, dtype=dtype, device=DEV)
    amd.head_attention(out, torch.cat(qs).to(DEV).contiguous(), kc, vc, i32([t + [0] * (w - len(t)) for t in tables]), lens, qsl, None,
                       vdim, scale, 1.0 if maps == 1 else 0.6, 150, 280, window, 0, chunk, keep, softcap,
                       sinks.to(DEV) if sink else None, maps, 0.37, 1e-2)
    tol = 1e-5 if dtype == F32 else 2e-2 if maps == 1 else 4e-2
    row = 0
    for (n, c), want in zip(SEQS, wants):
        close(out[row:row + n], want, tol, (n, c))
        row += n


@pytest.mark.parametrize("maps", [1, 2])
def test_many_single_tokens_cut_into_shares(amd, maps):
    """Long contexts: shares of the keys, kept tokens in the first of them."""
    from light_vllm_amd.attention.head_backend import HeadAttnImpl
    from light_vllm_amd.engine.hybrid_config import KVSpec
    H, G, dim, vdim, t = 4, 2, 32, 64, 3000
    spec = KVSpec(G, dim, vdim, maps)
    q, k, v = rand(3, H * maps, dim, dtype=BF16), rand(t, G * maps, dim, seed=1, dtype=BF16), rand(t, G, vdim, seed=2, dtype=BF16)
    lens = [3000, 2999, 1700]
    cache = torch.zeros((t + 15) // 16, spec.block_elements(16), dtype=BF16, device=DEV)
    kc, vc = HeadAttnImpl.split_kv_cache(cache, spec, 16)
    n = (t + 15) // 16 * 16
    kp = torch.nn.functional.pad(pad(k, spec.kpad // maps).reshape(t, G, -1), (0, 0, 0, 0, 0, n - t))
    kc.copy_(kp.view(-1, 16, G, spec.kpad // 8, 8).permute(0, 2, 3, 1, 4).to(DEV))
    vp = torch.nn.functional.pad(pad(v, spec.vpad), (0, 0, 0, 0, 0, n - t))
    vc.copy_(vp.view(-1, 16, G, spec.vpad).permute(0, 2, 3, 1).to(DEV))
    table = i32([list(range((t + 15) // 16))] * 3)
    for window, chunk, keep in ((0, 0, 0), (1500, 0, 40), (0, 1024, 0), (2000, 0, 1)):
        out = torch.zeros(3, H * vdim, dtype=BF16, device=DEV)
        amd.head_attention(out, pad(q, spec.kpad // maps).reshape(3, H, spec.kpad).contiguous().to(DEV), kc, vc, table, i32(lens),
                           i32([0, 1, 2, 3]), None, vdim, 0.3, 1.0, 1, t, window, 0, chunk, keep, 0.0, None, maps, 0.5, 1e-3)
        for i, L in enumerate(lens):
            low = max(L - window if window else 0, (L - 1) - (L - 1) % chunk if chunk else 0)
            keys = [j for j in range(L) if j >= low or j < keep]
            a = []
            for m in range(maps):
                s = torch.einsum("hd,jhd->hj", q[i].double().view(H, maps, dim)[:, m],
                                 k[keys].double().view(-1, G, maps, dim)[:, :, m].repeat_interleave(H // G, 1)) * 0.3
                a.append(torch.einsum("hj,jhe->he", s.softmax(-1), v[keys].double().repeat_interleave(H // G, 1)))
            want = a[0] if maps == 1 else lizazen.rms(a[0] - 0.5 * a[1], 1e-3)
            close(out[i], want.reshape(-1), 2e-2 if maps == 1 else 5e-2, (window, chunk, keep, L))


# ---- retention ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,dims", [(3, 24, 40, 16), (2, 11, 9, 10), (4, 64, 64, 64), (2, 128, 128, 128), (2, 144, 200, 0), (1, 256, 72, 6),
                                                (5, 64, 136, 32)])
def test_retention(amd, dtype, heads, dim, vdim, dims):
    """Sequences cut into portions and single tokens over slots that hold what others left; strong and no decay."""
    decay = [0.999, 0.5, 1.0, 0.9, 1e-6][:heads]
    r, eps = lc.rot(dims, 3e3), 1e-4
    lens, slots = [70, 300, 5, 1, 33], [4, 2, 0, 5, 1]
    data, wants = [], []
    for s, n in enumerate(lens):
        q, k = (rand(n, heads * dim, seed=10 * s + i, dtype=dtype) for i in (0, 1))
        v, g = (rand(n, heads * vdim, seed=10 * s + i, dtype=dtype) for i in (2, 3))
        data.append((q, k, v, g))
        qd, kd = (lizazen.rotate(t.double().view(n, heads, dim), range(n), r) for t in (q, k))
        o = lizazen.rms(lizazen.retain(qd, kd * dim ** -0.5, v.double().view(n, heads, vdim), decay), eps).reshape(n, -1)
        wants.append(o * g.double() * torch.sigmoid(g.double()))
    turns = torch.tensor([f / (2 * torch.pi) for f in lizazen.frequencies(r)], dtype=F64, device=DEV)
    d = torch.tensor(decay, dtype=F64)
    d = torch.stack([d, d.log()]).float().to(DEV)
    state = 1e4 * torch.randn(6, heads, dim, vdim, device=DEV)
    untouched = state[3].clone()
    at = [0] * len(lens)
    for step in ([(0, 16), (1, 250)], [(2, 2), (0, 1), (3, 1)], [(1, 1), (2, 1), (0, 1), (4, 1)], [(0, 17), (1, 2)], [(2, 1), (4, 1)],
                 [(4, 31), (0, 34), (1, 47)], [(0, 1), (2, 1)]):
        cols = [torch.cat([data[s][i][at[s]:at[s] + n] for s, n in step]).to(DEV) for i in range(4)]
        qsl, sl = layout([(n, at[s]) for s, n in step])
        pos = torch.tensor([p for s, n in step for p in range(at[s], at[s] + n)], device=DEV)
        out = torch.zeros(len(pos), heads * vdim + 3, dtype=dtype, device=DEV)
        amd.retention(out[:, :heads * vdim], *cols[:3], pos, turns, d, dim ** -0.5, cols[3], None, eps, 1.0, state,
                      i32([slots[s] for s, _ in step]), qsl, sl, max(n for _, n in step))
        row = 0
        for s, n in step:
            close(out[row:row + n, :heads * vdim], wants[s][at[s]:at[s] + n], 5e-5 if dtype == F32 else 1e-2, (s, at[s], n))
            at[s] += n
            row += n
        assert not out[:, heads * vdim:].any()
    assert at == lens and torch.equal(untouched, state[3])


# ---- whole models ----
LIMIT = {F32: 5e-5, BF16: 0.25}


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
    t = tokens(cfg, 75, 7)
    want, got = [], []
    lizazen.forward(cfg, w, t, on_layer=lambda i, x: want.append(x))
    rp = replay(folders[name], F32, 128)
    forward = rp.engine.worker.model.forward
    rp.engine.worker.model.forward = lambda *a: forward(*a, on_layer=lambda i, x: got.append(x.cpu()))
    rp.step([("a", t, [])])
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        close(a, b, 2e-5, (name, "layer", i))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_prompts_portions_and_single_tokens(folders, dtype, name):
    """One sequence, cut in many ways.  The pages and the slot of each run are the ones the run before gave back."""
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
    """Portions beside single tokens, requests that pause, end and leave their pages and slots to others; each against the
    sequence alone, in a pool with no page to spare."""
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
    t, want = lc.expected("all", 500, 2)
    rp = replay(folders["all"], F32, 512)
    got = play(rp, {"a": t}, [[("a", 20)]] + [[("a", 1)]] * 480)["a"]
    check_rows(got, want, F32, "long")


def greedy(cfg, w, prompt, n):
    return layered_case.greedy(lambda t: lizazen.forward(cfg, w, t), prompt, n)


@pytest.mark.parametrize("name", sorted(lc.CONFIGS))
def test_greedy_generation(folders, name):
    """The engine's own scheduler and captured steps, 32-bit, against the restatement's arg-max: whole prompts, portions of
    prompts beside decoded tokens, recomputed and swapped sequences in a pool too small for all, several steps in flight,
    several decoded tokens a step."""
    cfg, w = lc.case(name)
    prompts = [tokens(cfg, n, 50 + n) for n in (5, 31, 1, 48, 16)]
    want = [greedy(cfg, w, p, 8) for p in prompts]
    folder = folders[name]
    assert generate(engine(folder, F32), prompts, 8) == want
    assert generate(engine(folder, F32, graph=False, chunked=True, budget=24), prompts, 8) == want
    assert generate(engine(folder, F32, chunked=True, budget=24, max_seqs=3), prompts, 8) == want
    assert generate(engine(folder, F32, num_blocks=11, preemption_mode="recompute"), prompts, 8) == want
    assert generate(engine(folder, F32, num_blocks=11, preemption_mode="swap"), prompts, 8) == want
    assert generate(engine(folder, F32, scheduling="async", max_seqs=3), prompts, 8, use_async=True) == want
    assert generate(engine(folder, F32, use_v2_block_manager=True, num_scheduler_steps=4), prompts, 8) == want


def test_bfloat16_steps_captured_and_not(folders):
    cfg, _ = lc.case("mfma")
    prompts = [tokens(cfg, n, 80 + n) for n in (5, 31, 1, 48, 16)]
    a = generate(engine(folders["mfma"], BF16, graph=False), prompts, 24)
    assert generate(engine(folders["mfma"], BF16), prompts, 24) == a
    assert generate(engine(folders["mfma"], BF16, use_v2_block_manager=True, num_scheduler_steps=4), prompts, 24) == a


def test_several_sequences_per_prompt(folders):
    """Forked sequences: their log-probabilities are the restatement's for their own tokens."""
    from light_vllm_amd.engine.sampling_params import SamplingParams
    cfg, w = lc.case("all")
    p = tokens(cfg, 21, 90)
    eng = engine(folders["all"], F32, graph=False)
    eng.add_request("0", p, sampling_params=SamplingParams(n=3, temperature=1.0, seed=3, max_tokens=6, logprobs=1))
    outs = []
    while eng.has_unfinished_requests():
        outs += [o for o in eng.step() if o.finished]
    eng.shutdown()
    seqs = outs[-1].outputs
    assert len(seqs) == 3 and len({tuple(s) for s in seqs}) > 1
    sums = []
    for ids in seqs:
        lp = lizazen.forward(cfg, w, p + list(ids)).log_softmax(-1)
        sums.append(sum(lp[len(p) - 1 + j, tok].item() for j, tok in enumerate(ids)))
        if list(ids) == list(outs[-1].token_ids):
            for j, (tok, d) in enumerate(zip(ids, outs[-1].logprobs)):
                assert abs(d[tok][0] - lp[len(p) - 1 + j, tok].item()) < 1e-3
    assert all(x >= y - 1e-3 for x, y in zip(sums, sums[1:]))


def test_refuses_what_it_does_not_keep(folders):
    with pytest.raises(ValueError):
        engine(folders["odd"], BF16, cache=dict(cache_dtype="fp8"))
    with pytest.raises(ValueError):
        engine(folders["odd"], BF16, cache=dict(enable_prefix_caching=True))


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
