"""Susalorn on the GPU: every operator and whole models against the plain float64 restatement (oracle/susalorn.py) -- prompts,
portions, single tokens, mixed batches over reused pages and slots, and generation through the engine."""
import json
import os
import subprocess
import sys

import pytest
import torch

import layered_case
import susalorn_case as sc
from layered_case import engine, generate, play, portions, replay, tokens, write_model
from oracle import susalorn

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
    return sc.rand(*shape, seed=seed).to(dtype)


def close(got, want, rtol, what=""):
    """Worst difference against the largest expected value."""
    want = want.double()
    err = (got.double().cpu() - want).abs().max().item() / (want.abs().max().item() + 1e-30)
    assert err <= rtol, (what, err)


# ---- residual streams ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 4), (3, 7), (33, 96), (70, 250), (5, 1030), (2, 4096), (300, 2500), (2, 9000)])
@pytest.mark.parametrize("streams,kind", [(1, "rows"), (2, "slabs"), (3, "slots"), (4, "rows"), (5, "slots"), (16, "slabs")])
def test_streams_between_two_sublayers(amd, dtype, rows, width, streams, kind):
    eps, x = 1e-3, rand(streams, rows, width)
    mix, out, reads = rand(streams, streams, seed=20), rand(streams, seed=21), rand(streams, seed=22)
    w = 1 + 0.3 * rand(width, seed=23)
    slots = weights = None
    if kind == "slots":
        y, weights = rand(3 * rows, width, seed=5, dtype=dtype), rand(rows, 3, seed=7)
        slots = torch.randperm(3 * rows, generator=torch.Generator().manual_seed(6)).view(rows, 3).int()
        total = (y.double()[slots.long()] * weights.double()[..., None]).sum(1)
    elif kind == "slabs":
        y = rand(5, rows, width, seed=3)
        total = y.double().sum(0)
    else:
        y = rand(rows, width, seed=3, dtype=dtype)
        total = y.double()
    dev = [t.to(DEV) if t is not None else None for t in (y, slots, weights, mix, out, reads, w)]
    for same in (False, True):  # streams of their own, or one row for all of them
        xd = x.double() if not same else x[:1].double().expand(streams, rows, width)
        want = susalorn.write_streams(xd, mix.double(), out.double(), total)
        h_want = susalorn.rms_norm(susalorn.read_streams(want, reads.double()), w.double(), eps)
        x_in = x[0].to(DEV).expand(streams, rows, width) if same else x.to(DEV)
        for x_out in (None, torch.empty(streams, rows, width, device=DEV), x_in):
            if same and x_out is x_in:
                continue
            h = amd.stream_mix(x_out, x_in, *dev, eps, dtype)
            close(h, h_want, 4e-6 if dtype == F32 else 1e-2, ("h", same))
            if x_out is not None:
                close(x_out, want, 2e-6, ("x", same))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,streams", [(37, 1), (96, 3), (2048, 4)])
def test_embedding_of_all_streams(amd, dtype, width, streams):
    table, ids, reads, w = rand(61, width, dtype=dtype), [4, 60, 0, 4], rand(streams, seed=2), 1 + 0.2 * rand(width, seed=3)
    x = torch.full((4, width), 7.0, device=DEV)
    h = amd.stream_embed(x, table.to(DEV), torch.tensor(ids, device=DEV), reads.to(DEV), w.to(DEV), 1e-4)
    e = table.double()[ids]
    assert torch.equal(x.double().cpu(), e)
    close(h, susalorn.rms_norm(e * reads.double().sum(), w.double(), 1e-4), 3e-6 if dtype == F32 else 1e-2)


# ---- feed-forwards ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff", [(96, 72), (90, 33), (2048, 160), (64, 4096)])
def test_dense_feed_forward(amd, dtype, width, ff):
    from light_vllm_amd.engine.mixers import SiluMlp
    w = {"gate": rand(ff, width, seed=1) * 1.5 * width ** -0.5, "up": rand(ff, width, seed=2) * 1.5 * width ** -0.5,
         "down": rand(width, ff, seed=3) * ff ** -0.5}
    w = {k: t.bfloat16().float() for k, t in w.items()}
    mlp = SiluMlp(lambda s: w[s[1:]].to(dtype).to(DEV), "", True)
    for rows in (1, 5, 33, 64, 65, 300):
        h = rand(rows, width, seed=rows, dtype=dtype)
        y = mlp(h.to(DEV))
        close(y.sum(0) if y.dim() == 3 else y, susalorn.dense(h.double(), lambda s: w[s].double()), 1e-5 if dtype == F32 else 1.5e-2, rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,width,ff,count,keep", [(6, 1, 96, 40, 3, 1), (5, 2, 90, 33, 1, 1), (72, 7, 128, 64, 9, 4), (3, 3, 64, 256, 3, 3),
                                                           (128, 4, 320, 32, 64, 5), (16, 4, 512, 96, 4, 3)])
def test_mixture_of_ungated_experts(amd, dtype, experts, top, width, ff, count, keep):
    """Squared-ReLU experts without gates, chosen within the best groups."""
    from light_vllm_amd.engine.moe import ExpertConfig, MixtureConfig, MixtureOfExperts
    w = {"router": rand(experts, width, seed=1) * 2 * width ** -0.5}
    for i in range(experts):
        w[f"e{i}.up"] = rand(ff, width, seed=10 + 3 * i) * 1.5 * width ** -0.5
        w[f"e{i}.down"] = rand(width, ff, seed=12 + 3 * i) * ff ** -0.5
    w = {k: t.bfloat16().float() for k, t in w.items()}
    cfg = MixtureConfig(experts, top, ExpertConfig(ff), None, activation="relu_squared", router_bias=False, groups=count, keep=keep,
                        weight_scale=1.7)
    moe = MixtureOfExperts(lambda s: w[s[1:]].to(dtype).to(DEV), "", cfg, True)
    assert moe.packed == (dtype == BF16 and width % 32 == 0)
    mlp = sc.moe(experts, top, ff, count, keep, 1.7)
    for rows in (1, 2, 17, 64, 65, 300):
        h = (1.5 * rand(rows, width, seed=50 + rows)).to(dtype)
        y, slots, weights = moe(h.to(DEV))
        y, slots = y.double().cpu(), slots.long().cpu()
        assert sorted(slots.reshape(-1).tolist()) == list(range(rows * top))
        got = (y[slots] * weights.double().cpu()[..., None]).sum(1)
        close(got, susalorn.mixture(h.double(), mlp, lambda s: w[s].double()), 1e-5 if dtype == F32 else 2e-2, rows)


def test_router_of_groups(amd):
    for dtype, experts, width, count in ((F32, 6, 24, 3), (BF16, 64, 256, 8), (BF16, 130, 90, 13), (BF16, 256, 128, 64), (BF16, 63, 64, 9)):
        for rows in (1, 33, 200):
            h, w = rand(rows, width, seed=1, dtype=dtype), (rand(experts, width, seed=2) * width ** -0.5).to(dtype)
            packed = dtype == BF16 and width % 32 == 0
            wd = amd.pack_weight(torch.nn.functional.pad(w, (0, 0, 0, -experts % 16)).to(DEV)) if packed else w.to(DEV)
            for top, keep in ((1, 1), (2, 1), (4, 2), (5, count)):
                ids, weights, _, token, slots, _, _ = amd.moe_route(h.to(DEV), wd, None, top, False, packed, experts, False, 0, False,
                                                                    count, keep, 0.6)
                r = {"top": top, "groups": {"count": count, "keep": keep}, "scale": 0.6}
                want_ids, want = susalorn.route(h.double() @ w.double().T, r)
                assert torch.equal(ids.long().cpu(), want_ids)
                close(weights, want, 1e-5)
                assert torch.equal(token[slots.long()], torch.arange(rows, device=DEV, dtype=torch.int32)[:, None].expand(-1, top))


# ---- latent attention ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot_dim,q_rank", [(48, 16, 40), (35, 6, 19), (128, 32, 1536), (512, 64, 2100), (256, 64, 96)])
def test_query_latents_and_cache_rows(amd, dtype, rank, rot_dim, q_rank):
    """Norms and rotated rows at positions up to a million, in the kernels' order of pairs; rows without a slot, padding and
    everything else in the cache."""
    from light_vllm_amd.engine.latent_config import LatentKVSpec, RampScaling, RotationConfig
    from light_vllm_amd.engine.latent_layers import Rotation
    scaling = (4.0, 4096, 32.0, 1.0)
    r, spec = sc.rot(rot_dim, 5e4, scaling), LatentKVSpec(rank, rot_dim)
    rotation = Rotation(RotationConfig(rot_dim, 5e4, True, RampScaling(*scaling)), DEV)
    order = rotation.ordered(torch.arange(rot_dim, device=DEV)[:, None])[:, 0].cpu()
    q_pad = (q_rank + 31) // 32 * 32
    for rows in (6, 70):
        pos = [0, 1, 17, 4095, 131071, 1000003] + list(range(40, 40 + rows - 6))
        slots = [3, -1, 20, 0, 31, 9] + list(range(48, 48 + rows - 6))
        z = rand(rows, q_rank + rank + rot_dim + 3, seed=1, dtype=dtype)
        q, kv = z[:, :q_rank], z[:, q_rank:q_rank + rank + rot_dim]
        wq, wc = 1 + 0.3 * rand(q_rank, seed=2), 1 + 0.3 * rand(rank, seed=3)
        cache = torch.full((8, 16, spec.row), 7.0, dtype=dtype, device=DEV)
        zd = z.to(DEV)
        kvd = torch.cat([zd[:, q_rank:q_rank + rank], zd[:, q_rank + rank:q_rank + rank + rot_dim][:, order.to(DEV)]], 1)
        got = amd.latent_down(zd[:, :q_rank], wq.to(DEV), q_pad, cache, kvd, wc.to(DEV), 1e-3, spec.cpad, torch.tensor(pos, device=DEV),
                              rotation.turns, torch.tensor(slots, device=DEV), rotation.grow)
        tol = 1e-6 if dtype == F32 else 5e-3
        close(got[:, :q_rank], susalorn.rms_norm(q.double(), wq.double(), 1e-3), tol)
        assert not got[:, q_rank:].any()
        flat = cache.view(-1, spec.row)
        used, which = [s for s in slots if s >= 0], [i for i, s in enumerate(slots) if s >= 0]
        close(flat[used][:, :rank], susalorn.rms_norm(kv[:, :rank].double(), wc.double(), 1e-3)[which], tol)
        close(flat[used][:, spec.cpad:spec.cpad + rot_dim], susalorn.rotate(kv[:, rank:].double(), pos, r)[which][:, order], tol)
        assert not flat[used][:, rank:spec.cpad].any() and not flat[used][:, spec.cpad + rot_dim:].any()
        rest = [i for i in range(128) if i not in used]
        assert (flat[rest] == 7).all()


# heads, dim, rot, vdim, kv rank, q rank
LATENT = {"mfma": (16, 64, 32, 64, 128, 96), "many heads": (33, 32, 32, 32, 64, 40), "odd": (3, 13, 6, 21, 35, 19),
          "large": (8, 128, 64, 128, 512, 384), "no class": (2, 48, 80, 40, 600, 64)}
SEQS = [(1, 0), (1, 250), (2, 61), (3, 0), (40, 5), (150, 130), (129, 0), (1, 16), (17, 47), (66, 500), (64, 100), (65, 33)]


def far_inputs(m, w, n, width, back, seed):
    """Rows of one sequence whose last token's first head looks for one key, `back` tokens before it: that key's latent points along
    the query and would carry most of the softmax."""
    x = sc.rand(n, width, seed=seed).double()
    j = n - 1 - back
    if j < 0 or back == 0:
        return x.bfloat16().float()
    q = susalorn.rms_norm(x[-1:] @ w["dq"].double().T, w["dq.norm"].double(), 1e-4) @ w["uq"].double().T
    latent = (w["uk"][:m["dim"]].double() * w["dkv.norm"].double()).T @ q[0, :m["dim"]]
    want = torch.linalg.lstsq(w["dkv"][:m["kv_rank"]].double(), latent[:, None]).solution[:, 0]
    x[j] = want / want.norm() * width ** 0.5 + 0.1 * x[j]
    return x.bfloat16().float()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", sorted(LATENT))
def test_latent_attention_over_all_keys(amd, dtype, sizes):
    """Single tokens, short and long portions in one step, over pages that hold what others left; every sequence's last token looks
    for a key at the start, at a page's edge or just before it."""
    from light_vllm_amd.attention.latent_backend import LatentAttnImpl
    from light_vllm_amd.engine.latent_config import LatentAttentionConfig, RampScaling, RotationConfig
    from light_vllm_amd.engine.latent_layers import LatentAttention, LatentStep
    from light_vllm_amd.engine.mixers import StepLayout
    H, dim, rot_dim, vdim, rank, q_rank = LATENT[sizes]
    width, eps, scaling = 96, 1e-4, (4.0, 128, 16.0, 1.0)
    _, m = sc.latent(H, dim, rot_dim, vdim, rank, q_rank, 2.0 * (dim + rot_dim) ** -0.5, 3e3, scaling)
    w = sc.mixer_weights("latent_attention", m, width)
    cfg = LatentAttentionConfig(H, dim, rot_dim, vdim, rank, RotationConfig(rot_dim, 3e3, True, RampScaling(*scaling)), m["scale"], 0,
                                q_rank=q_rank, gate=False, sink=True)
    mixer = LatentAttention(lambda s: w[s[1:]].to(dtype).to(DEV), "", cfg, eps, True)
    blocks = sum((n + c + 15) // 16 for n, c in SEQS) + 3
    cache = (5 * torch.randn(blocks, 16 * cfg.spec.row, generator=torch.Generator().manual_seed(5))).to(dtype).to(DEV)
    perm = torch.randperm(blocks, generator=torch.Generator().manual_seed(6)).tolist()
    rows, wants, tables, slots, pos, before = [], [], [], [], [], []
    for s, (n, c) in enumerate(SEQS):
        t = n + c
        x = far_inputs(m, w, t, width, (t - 1, (t - 1) % 16 + 1, 15, 16, 63, 64)[s % 6], 10 * s)
        table = [perm.pop() for _ in range((t + 15) // 16)]
        tables.append(table)
        wants.append(susalorn.latent_attention(x.double(), m, lambda k: w[k].double(), eps)[c:])
        rows.append(x[c:])
        before.append(x[:c])
        slots += [table[p // 16] * 16 + p % 16 for p in range(c, t)]
        pos += range(c, t)
    wide = max(map(len, tables))
    bt = i32([t + [0] * (wide - len(t)) for t in tables])

    def step(seqs, at, where):
        qsl, lens = layout(seqs)
        return LatentStep(StepLayout(qsl, lens, bt, torch.tensor(where, device=DEV), None, max(n for n, _ in seqs),
                                     max(n + c for n, c in seqs), 16, torch.tensor(at, device=DEV), [n for n, _ in seqs], [c for _, c in seqs]))
    # what came before goes to the cache first
    old = [(len(b), 0) for b in before]
    where = [t[p // 16] * 16 + p % 16 for t, b in zip(tables, before) for p in range(len(b))]
    mixer(torch.cat(before).to(dtype).to(DEV), cache, 0, step(old, [p for b in before for p in range(len(b))], where), LatentAttnImpl())
    y = mixer(torch.cat(rows).to(dtype).to(DEV), cache, 0, step(SEQS, pos, slots), LatentAttnImpl()).y
    y = y.sum(0) if y.dim() == 3 else y
    row = 0
    for (n, c), want in zip(SEQS, wants):
        close(y[row:row + n], want, 2e-5 if dtype == F32 else 3e-2, (n, c))
        row += n
    # single tokens alone (the split over shares)
    single = [i for i, (n, _) in enumerate(SEQS) if n == 1]
    bt = bt[single].contiguous()
    ends = [SEQS[i][1] for i in single]
    z = mixer(torch.cat([rows[i] for i in single]).to(dtype).to(DEV), cache, 0,
              step([(1, c) for c in ends], ends, [tables[i][c // 16] * 16 + c % 16 for i, c in zip(single, ends)]), LatentAttnImpl()).y
    close(z.sum(0) if z.dim() == 3 else z, torch.cat([wants[i] for i in single]), 2e-5 if dtype == F32 else 3e-2, "single")


def test_long_contexts_cut_into_shares(amd):
    """A far key and a sink, thousands of keys a token."""
    H, rank, rot_dim, vdim, t = 20, 100, 24, 48, 5000
    cpad, rpad = 128, 32
    rows = torch.zeros((t + 15) // 16 * 16, cpad + rpad)
    rows[:t, :rank], rows[:t, cpad:cpad + rot_dim] = rand(t, rank), rand(t, rot_dim, seed=1)
    lens = [5000, 4999, 1700]
    q = torch.zeros(3, H, cpad + rpad)
    q[:, :, :rank], q[:, :, cpad:cpad + rot_dim] = 0.3 * rand(3, H, rank, seed=2), 0.3 * rand(3, H, rot_dim, seed=3)
    rows[0, :rank] = 2.0 * q[0, 4, :rank]
    rows[1, :rank] = 2.0 * q[1, 7, :rank]
    rows, q = rows.bfloat16(), q.bfloat16()
    uv = torch.zeros(H, 48, cpad)
    uv[..., :rank] = rand(H, vdim, rank, seed=4) / 10
    uv = uv.bfloat16()
    sink = 1 + rand(H, seed=5)
    out = torch.zeros(3, H * vdim, dtype=BF16, device=DEV)
    cache, table = rows.view(-1, 16, cpad + rpad).to(DEV), i32([list(range((t + 15) // 16))] * 3)
    for with_sink in (True, False):
        amd.latent_attention(out, q.to(DEV), cache, uv.to(DEV), None, vdim, table, i32(lens), i32([0, 1, 2, 3]), 0.8, 0, 1 << 30, 1, t,
                             sink.to(DEV) if with_sink else None)
        for i, n in enumerate(lens):
            s = q[i].double() @ rows[:n].double().T * 0.8
            e = torch.exp(s - s.max())
            total = e.sum(1) + (torch.exp(sink.double() - s.max()) if with_sink else 0)
            o = (e @ rows[:n, :cpad].double()) / total[:, None]
            close(out[i], torch.bmm(uv.double(), o[..., None])[..., 0].reshape(-1), 2e-2, (with_sink, n))


# ---- short convolutions and the delta rule ----
STEPS = ([(0, 16), (1, 250)], [(2, 2), (0, 1), (3, 1)], [(1, 1), (2, 1), (0, 1), (4, 1)], [(0, 17), (1, 2)], [(2, 1), (4, 1)],
         [(4, 31), (0, 34), (1, 47)], [(0, 1), (2, 1)])
LENS, SLOTS = [70, 300, 5, 1, 33], [4, 2, 0, 5, 1]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels,taps", [(96, 4), (37, 3), (2048, 2), (20, 1), (64, 16), (19, 7)])
def test_short_convolution(amd, dtype, channels, taps):
    x = [rand(n, channels, seed=s, dtype=dtype) for s, n in enumerate(LENS)]
    w = 0.5 * rand(channels, taps, seed=9)
    wants = [susalorn.short_conv(v.double(), w.double()) for v in x]
    state, at = 1e4 * torch.randn(6, taps, channels, device=DEV), [0] * 5
    untouched = state[3].clone()
    for step in STEPS:
        qsl, lens = layout([(n, at[s]) for s, n in step])
        rows = torch.cat([x[s][at[s]:at[s] + n] for s, n in step]).to(DEV)
        y = amd.short_conv(rows, w.t().contiguous().to(DEV), state, i32([SLOTS[s] for s, _ in step]), qsl, lens, max(n for _, n in step))
        row = 0
        for s, n in step:
            close(y[row:row + n], wants[s][at[s]:at[s] + n], 1e-6 if dtype == F32 else 8e-3, (s, at[s], n))
            at[s] += n
            row += n
    assert at == LENS and torch.equal(state[3], untouched)


def run_delta(mixer, dtype, xs, steps, slots, state):
    """Rows of several sequences through the mixer, step by step; one result per sequence."""
    from light_vllm_amd.engine.mixers import LayerCache, StepLayout
    at, out = [0] * len(xs), [[] for _ in xs]
    for step in steps:
        qsl, lens = layout([(n, at[s]) for s, n in step])
        rows = torch.cat([xs[s][at[s]:at[s] + n] for s, n in step]).to(dtype).to(DEV)
        y = mixer(rows, LayerCache(None, state), StepLayout(qsl, lens, None, None, i32([slots[s] for s, _ in step]),
                                                            max(n for _, n in step), int(lens.max()), 16)).y
        y = (y.sum(0) if y.dim() == 3 else y).cpu()
        row = 0
        for s, n in step:
            out[s].append(y[row:row + n])
            at[s] += n
            row += n
    return [torch.cat(o) if o else None for o in out]


def delta_mixer(m, w, dtype, eps, fused=True):
    from light_vllm_amd.engine.stream_config import DeltaRuleConfig
    from light_vllm_amd.engine.stream_layers import DeltaRule
    cfg = DeltaRuleConfig(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"])
    mixer = DeltaRule(lambda s: w[s[1:]].to(dtype).to(DEV), "", cfg, eps, True)
    mixer.fused = fused
    state = {"matrix": 1e4 * torch.randn(6, cfg.heads, cfg.dim, cfg.vdim, device=DEV),
             "conv": 1e4 * torch.randn(6, cfg.taps, sum(cfg.columns), device=DEV)}
    return mixer, state


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,taps,rank", [
    (4, 2, 24, 40, 4, 24), (3, 1, 11, 9, 5, 7), (2, 2, 64, 64, 4, 64), (4, 4, 128, 128, 4, 128), (2, 1, 144, 200, 3, 33), (1, 1, 256, 72, 1, 16),
    (5, 5, 64, 136, 2, 200), (1, 1, 32, 600, 4, 9), (6, 2, 100, 30, 16, 40), (2, 2, 256, 256, 4, 130)])
def test_delta_rule(amd, dtype, heads, kv_heads, dim, vdim, taps, rank):
    """Sequences cut into portions and single tokens over slots that hold what others left; channels that keep and that forget at
    once."""
    _, m = sc.delta(heads, kv_heads, dim, vdim, taps)
    width, eps = 64, 1e-4
    w = sc.mixer_weights("channel_delta", m, width, rank, seed=heads)
    xs = [rand(n, width, seed=s) for s, n in enumerate(LENS)]
    xs = [x.bfloat16().float() for x in xs]
    wants = [susalorn.channel_delta(x.double(), m, lambda k: w[k].double(), eps) for x in xs]
    for fused in (True, False):
        mixer, state = delta_mixer(m, w, dtype, eps, fused)
        untouched = [t[3].clone() for t in state.values()]
        got = run_delta(mixer, dtype, xs, STEPS, SLOTS, state)
        for s, (a, b) in enumerate(zip(got, wants)):
            close(a, b, 3e-5 if dtype == F32 else 4e-2, (fused, s))
        assert all(torch.equal(t[3], u) for t, u in zip(state.values(), untouched))


def test_delta_rule_of_equal_keys():
    """One token over and over: keys that are all the same, full writes, hardly a decay -- the system of a chunk at its worst."""
    _, m = sc.delta(2, 2, 32, 48, 2)
    w = sc.mixer_weights("channel_delta", m, 64, seed=3)
    w["b"][:], w["dt_bias"][:] = 0.0, -12.0
    w["a2"][:] = 0.0
    x = rand(1, 64, seed=1).expand(200, 64).clone()
    x[100:] = rand(1, 64, seed=2)
    w["b"][0], w["b"][1] = 0.5 * x[0], 0.5 * x[150]
    w["b"] = w["b"].bfloat16().float()
    x = x.bfloat16().float()
    want = susalorn.channel_delta(x.double(), m, lambda k: w[k].double(), 1e-4)
    for cut in ([200], [1] * 200, [33, 1, 100, 66]):
        mixer, state = delta_mixer(m, w, F32, 1e-4)
        got = run_delta(mixer, F32, [x], [[(0, n)] for n in cut], [2], state)[0]
        close(got, want, 3e-5, cut)


def test_delta_rule_keeps_what_is_far_back():
    """A state that forgets nothing: the first token's value is read out hundreds of tokens later."""
    _, m = sc.delta(2, 2, 64, 32, 4)
    w = sc.mixer_weights("channel_delta", m, 64, seed=5)
    w["dt_bias"][:], w["a2"][:] = -20.0, 0.0
    xs = [rand(700, 64, seed=7).bfloat16().float()]
    other = xs[0].clone()
    other[0] = -other[0]
    want, changed = (susalorn.channel_delta(x.double(), m, lambda k: w[k].double(), 1e-4) for x in (xs[0], other))
    assert (want - changed)[600:].abs().max() > 1e-3 * want.abs().max()
    for cut in ([700], [500] + [1] * 200, portions(700, [64, 2, 1, 130])):
        mixer, state = delta_mixer(m, w, F32, 1e-4)
        close(run_delta(mixer, F32, xs, [[(0, n)] for n in cut], [0], state)[0], want, 3e-5, cut[:4])


def test_rows_of_a_captured_step_without_a_sequence():
    _, m = sc.delta(4, 2, 24, 40, 4)
    w = sc.mixer_weights("channel_delta", m, 64)
    mixer, state = delta_mixer(m, w, F32, 1e-4)
    before = [t.clone() for t in state.values()]
    got = run_delta(mixer, F32, [rand(1, 64)] * 2, [[(0, 1), (1, 1)]], [-1, -1], state)
    assert all(torch.equal(a, b) for a, b in zip(state.values(), before)) and all(g.isfinite().all() for g in got)


# ---- whole models ----
LIMIT = {F32: 5e-5, BF16: 0.25}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {n: write_model(tmp_path_factory.mktemp(n), *sc.case(n)) for n in sc.CONFIGS}


def check_rows(got, want, dtype, what):
    e = layered_case.error(got, want)
    if dtype == F32:
        assert e.max() < LIMIT[F32], (what, e.argmax().item(), e.max().item())
    else:  # a row may be sensitive (two keys or experts of nearly equal score); most are not
        assert e.median() < LIMIT[BF16] / 3 and (e > LIMIT[BF16]).double().mean() <= 0.1, (what, e.median(), e.max(), (e > LIMIT[BF16]).double().mean())


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_residual_stream_layer_by_layer(folders, name):
    cfg, w = sc.case(name)
    t = tokens(cfg, 75, 7)
    want, got = [], []
    susalorn.forward(cfg, w, t, on_layer=lambda i, x: want.append(x))
    rp = replay(folders[name], F32, 128)
    forward = rp.engine.worker.model.forward
    rp.engine.worker.model.forward = lambda *a: forward(*a, on_layer=lambda i, x: got.append(x.cpu()))
    rp.step([("a", t, [])])
    assert len(got) == len(want) == len(susalorn.passes(cfg))
    for i, (a, b) in enumerate(zip(got, want)):
        close(a, b, 2e-5, (name, "layer", i))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_prompts_portions_and_single_tokens(folders, dtype, name):
    """One sequence, cut in many ways.  The pages and the slot of each run are the ones the run before gave back."""
    t, want = sc.expected(name, 170, 1)
    rp = replay(folders[name], dtype, 192)
    cuts = {"whole": [170], "tokens": [1] * 170, "most, then tokens": [129] + [1] * 41, "twos": portions(170, [2]),
            "threes": portions(170, [3, 1, 16]), "mixed": portions(170, [15, 2, 33, 1, 1, 64, 7]), "long": [2, 66, 80, 22]}
    for cut, sizes in cuts.items():
        got = play(rp, {cut: t}, [[(cut, n)] for n in sizes])[cut]
        check_rows(got, want, dtype, (name, cut))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_batches_of_unequal_requests(folders, dtype, name):
    """Portions beside single tokens, requests that pause, end and leave their pages and slots to others; each against the
    sequence alone, in a pool with no page to spare."""
    lens = {"a": 140, "b": 33, "c": 90, "d": 1, "e": 60, "f": 17}
    seqs = {r: sc.expected(name, n, 10 + i) for i, (r, n) in enumerate(lens.items())}
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
    t, want = sc.expected("all", 500, 2)
    rp = replay(folders["all"], F32, 512)
    got = play(rp, {"a": t}, [[("a", 20)]] + [[("a", 1)]] * 480)["a"]
    check_rows(got, want, F32, "long")


def greedy(cfg, w, prompt, n):
    return layered_case.greedy(lambda t: susalorn.forward(cfg, w, t), prompt, n)


@pytest.mark.parametrize("name", sorted(sc.CONFIGS))
def test_greedy_generation(folders, name):
    """The engine's own scheduler and captured steps, 32-bit, against the restatement's arg-max: whole prompts, portions of
    prompts beside decoded tokens, recomputed and swapped sequences in a pool too small for all, several steps in flight,
    several decoded tokens a step."""
    cfg, w = sc.case(name)
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
    cfg, _ = sc.case("mfma")
    prompts = [tokens(cfg, n, 80 + n) for n in (5, 31, 1, 48, 16)]
    a = generate(engine(folders["mfma"], BF16, graph=False), prompts, 24)
    assert generate(engine(folders["mfma"], BF16), prompts, 24) == a
    assert generate(engine(folders["mfma"], BF16, use_v2_block_manager=True, num_scheduler_steps=4), prompts, 24) == a


def test_several_sequences_per_prompt(folders):
    """Forked sequences: their log-probabilities are the restatement's for their own tokens."""
    from light_vllm_amd.engine.sampling_params import SamplingParams
    cfg, w = sc.case("all")
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
        lp = susalorn.forward(cfg, w, p + list(ids)).log_softmax(-1)
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


def test_sizing_without_a_cache(folders):
    """Blocks cost nothing where no layer has a cache: the engine still finds a number of them."""
    cfg, w = sc.case("states")
    p = tokens(cfg, 20, 3)
    assert generate(engine(folders["states"], F32, num_blocks=None), [p], 6) == [greedy(cfg, w, p, 6)]


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
