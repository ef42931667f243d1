"""Sublayers of hybrid decoders on the gfx950 operators: a Dynamic-Tanh norm fused with the residual add, the two mixers
(softmax heads beside gated linear attention; token-shift time mixing) and the squared-ReLU feed-forward.

The residual stream is fp32 and travels as (x, y): x the stream, y the projection result of the sublayer before, which the
next norm's launch adds.  y is [rows, width] in the compute dtype or, for decode-size steps, the fp32 split-K slabs of a
weight-streaming GEMM.  Constants come from the configuration; nothing here knows a model's sizes."""
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn.functional as F

from .hybrid_config import KVSpec, LinearHeadsConfig, ParallelMixerConfig, SoftmaxHeadsConfig, TimeMixerConfig
from .model import Weight, linear

amd = torch.ops._C_amd
DECAY_LOGSIGMOID, DECAY_NEGEXP = 0, 1
DECODE_ROWS = 64  # steps of up to this many rows take the weight-streaming GEMMs


@dataclass
class StepLayout:
    """Where a step's rows belong (device tensors): the new tokens of num_seqs sequences, back to back."""
    query_start_loc: torch.Tensor   # int32 [num_seqs + 1]
    seq_lens: torch.Tensor          # int32 [num_seqs], the new tokens included
    block_tables: torch.Tensor      # int32 [num_seqs, blocks]
    slot_mapping: torch.Tensor      # int64 [rows]
    state_slots: torch.Tensor       # int32 [num_seqs]
    max_query_len: int
    max_seq_len: int
    block_size: int
    positions: Optional[torch.Tensor] = None    # int64 [rows]
    # host copies of the sequences' new tokens and of what came before (None: a captured step)
    query_lens: Optional[List[int]] = None
    context_lens: Optional[List[int]] = None


@dataclass
class LayerCache:
    """What one layer keeps between steps: its paged keys / values (None: no softmax heads) and its recurrent state."""
    kv: Optional[torch.Tensor]
    state: Dict[str, torch.Tensor]


def ceil_to(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def stack_rows(parts: List[torch.Tensor], align: int = 16) -> Tuple[torch.Tensor, List[int]]:
    """Weights of projections that read the same input, one under the other, each padded with zero rows to a multiple of
    `align` (vector loads of its columns stay aligned); returns the stack and the first row of each part."""
    offsets, rows, at = [], [], 0
    for p in parts:
        offsets.append(at)
        rows.append(p)
        pad = ceil_to(p.shape[0], align) - p.shape[0]
        if pad:
            rows.append(p.new_zeros(pad, p.shape[1]))
        at += p.shape[0] + pad
    return torch.cat(rows), offsets


def pad_columns(w: torch.Tensor, align: int = 32) -> torch.Tensor:
    pad = ceil_to(w.shape[1], align) - w.shape[1]
    return F.pad(w, (0, pad)) if pad else w


def make_weight(w: torch.Tensor, pack: bool) -> Weight:
    return Weight(w.contiguous(), pack and w.dtype != torch.float32)


def project_to_residual(x: torch.Tensor, w: Weight) -> torch.Tensor:
    """A projection whose only reader is the next residual add: split-K slabs where that launch sums them."""
    if 0 < x.shape[0] <= DECODE_ROWS and w.packed is not None:
        return amd.skinny_linear_packed_partials(x, w.packed, w.N, w.K, False)
    return linear(x, w)


class DynTanhNorm:
    """tanh(alpha x) * weight + bias in fp32, the residual add in the same launch."""

    def __init__(self, get, name: str):
        self.weight, self.bias, self.alpha = get(name).float(), get(name + ".b").float(), get(name + ".alpha").float().reshape(1)

    def __call__(self, x: torch.Tensor, y: Optional[torch.Tensor], dtype: torch.dtype) -> torch.Tensor:
        """x += y in place; returns the normed rows in `dtype`."""
        return amd.add_dyt(x, y, self.alpha, self.weight, self.bias, dtype)

    def shift_mix(self, x, y, mu: torch.Tensor, carried: torch.Tensor, step: StepLayout, dtype) -> Tuple[torch.Tensor, torch.Tensor]:
        """(x + y, the token-shift mixes [mixes, rows, width]); `carried` is read and updated."""
        x_new, mix = amd.add_dyt_shift_mix(x, y, mu, self.alpha, self.weight, self.bias, carried, step.state_slots,
                                           step.query_start_loc, step.seq_lens, dtype)
        return (x if y is None else x_new), mix


class LowRankDecay:
    """ln w per channel from a low-rank projection: z = A f(u) + bias (csrc/recurrent.hip)."""

    def __init__(self, a: torch.Tensor, bias: torch.Tensor, kind: int, inv_tau: float = 1.0):
        self.a_t, self.bias = a.float().t().contiguous(), bias.float().reshape(-1).contiguous()
        self.kind, self.inv_tau = kind, inv_tau

    def __call__(self, u: torch.Tensor) -> torch.Tensor:
        return amd.log_decay(u, self.a_t, self.bias, self.kind, self.inv_tau)


class Recurrence:
    """A decayed matrix state with its read-out, per-head RMS norm and SiLU gate: out = norm(o) * weight * silu(g) * scale.
    `fused`: one operator (a single launch for steps of single tokens); else decays, token-by-token recurrence, norm and
    gate as launches of their own."""

    def __init__(self, decay: LowRankDecay, bonus: Optional[torch.Tensor], eps: float):
        self.decay, self.bonus, self.eps, self.fused = decay, bonus, eps, True

    def __call__(self, out, q, k, v, u, gate, weight, out_scale: float, q_scale: float, state, step: StepLayout) -> None:
        d = self.decay
        if self.fused:
            amd.recurrent_mix(out, q, k, v, u, d.a_t, d.bias, d.kind, d.inv_tau, self.bonus, q_scale, gate, weight, self.eps,
                              out_scale, state, step.state_slots, step.query_start_loc, step.seq_lens, step.max_query_len)
        else:
            o = amd.recurrent_scan(q, k, v, d(u), self.bonus, q_scale, state, step.state_slots, step.query_start_loc,
                                   step.seq_lens)
            amd.head_norm_gate(out, o, gate, weight, self.eps, out_scale)


class ParallelMixer:
    """left_scale * softmax heads + right_scale * gated linear attention, both reading the same normed input: ONE input
    projection (all ten weights stacked) and ONE output projection over the two concatenated results; the scales are
    applied with the gates in front of it."""

    def __init__(self, get, name: str, cfg: ParallelMixerConfig, eps: float, pack: bool):
        self.cfg, self.eps = cfg, eps
        a, r = cfg.left, cfg.right
        l, rt = name + ".left", name + ".right"
        a1 = get(rt + ".a1")
        parts = [get(l + ".q"), get(l + ".k"), get(l + ".v"), get(rt + ".q"), get(rt + ".k"), get(rt + ".v"),
                 get(rt + ".g"), get(l + ".g"), a1]
        stack, self.at = stack_rows(parts)
        self.sizes = [p.shape[0] for p in parts]
        self.proj = make_weight(stack, pack)
        self.q_norm, self.k_norm = get(l + ".q.norm").float(), get(l + ".k.norm").float()
        self.decay = LowRankDecay(get(rt + ".a2"), get(rt + ".a2.b"), DECAY_LOGSIGMOID, 1.0 / r.tau)
        self.out_norm = get(rt + ".norm").float()
        self.recurrence = Recurrence(self.decay, None, eps)
        self.left_cols, self.right_cols = a.heads * a.vdim, r.heads * r.vdim
        self.out = make_weight(pad_columns(torch.cat([get(l + ".o"), get(rt + ".o")], dim=1)), pack)
        self.kv_spec = KVSpec(a.kv_heads, a.dim, a.vdim)

    def __call__(self, x, y, norm: DynTanhNorm, cache: LayerCache, step: StepLayout, attn, dtype):
        a, r = self.cfg.left, self.cfg.right
        h = norm(x, y, dtype)
        proj = linear(h, self.proj)
        lq, lk, lv, rq, rk, rv, rg, lg, u = (proj[:, o:o + n] for o, n in zip(self.at, self.sizes))
        rows = proj.shape[0]
        cols = self.left_cols + self.right_cols
        both = (torch.empty if self.out.K == cols else torch.zeros)(rows, self.out.K, dtype=dtype, device=proj.device)
        # softmax heads
        kc, vc = attn.split_kv_cache(cache.kv, self.kv_spec, step.block_size)
        q = amd.qk_norm_cache(lq, lk, lv, self.q_norm, self.k_norm, self.eps, a.heads, a.kv_heads, kc, vc, step.slot_mapping)
        amd.head_attention(both[:, :self.left_cols], q, kc, vc, step.block_tables, step.seq_lens, step.query_start_loc, lg,
                           a.vdim, a.scale, self.cfg.left_scale, step.max_query_len, step.max_seq_len)
        # gated linear attention
        self.recurrence(both[:, self.left_cols:cols], rq, rk, rv, u, rg, self.out_norm, self.cfg.right_scale,
                        r.dim ** -0.5, cache.state["matrix"], step)
        return x, project_to_residual(both, self.out)


class TimeMixer:
    """Token shift, five mixes, four projections of one size (one batched product), a low-rank decay, the bonus read-out."""

    MIXES = "rkvgw"

    def __init__(self, get, name: str, cfg: TimeMixerConfig, eps: float, pack: bool):
        self.cfg = cfg
        self.mu = torch.stack([get(f"{name}.mu.{s}").float() for s in self.MIXES]).contiguous()
        self.rkvg = [make_weight(get(f"{name}.{s}"), pack) for s in "rkvg"]
        # the library's batched product takes the weights as [4, width, heads * dim]
        self.rkvg_t = torch.stack([get(f"{name}.{s}").t() for s in "rkvg"]).contiguous()
        w1 = get(name + ".w1")
        self.rank = w1.shape[0]
        self.w1 = make_weight(stack_rows([w1])[0], pack)
        self.decay = LowRankDecay(get(name + ".w2"), get(name + ".w0"), DECAY_NEGEXP)
        self.recurrence = Recurrence(self.decay, get(name + ".u").float().contiguous(), eps)
        self.norm = get(name + ".norm").float()
        self.out = make_weight(pad_columns(get(name + ".o")), pack)

    def __call__(self, x, y, norm: DynTanhNorm, cache: LayerCache, step: StepLayout, attn, dtype):
        x, mix = norm.shift_mix(x, y, self.mu, cache.state["shift"], step, dtype)
        rows = x.shape[0]
        if 0 < rows <= DECODE_ROWS and self.rkvg[0].packed is not None:
            r, k, v, g = (linear(mix[i], w) for i, w in enumerate(self.rkvg))
        else:
            r, k, v, g = torch.bmm(mix[:4], self.rkvg_t)
        u = linear(mix[4], self.w1)[:, :self.rank]
        cols = self.cfg.heads * self.cfg.dim
        out = (torch.empty if self.out.K == cols else torch.zeros)(rows, self.out.K, dtype=dtype, device=x.device)
        self.recurrence(out[:, :cols], r, k, v, u, g, self.norm, 1.0, 1.0, cache.state["matrix"], step)
        return x, project_to_residual(out, self.out)


class SiluMlp:
    """W_down (silu(W_gate h) * (W_up h))."""

    def __init__(self, get, name: str, pack: bool):
        # zero rows of gate and up give zero activations: all sizes may be padded for the weight-streaming kernel
        self.up = make_weight(stack_rows([get(name + ".gate"), get(name + ".up")], 32)[0], pack)
        self.down = make_weight(pad_columns(get(name + ".down")), pack)

    def numel(self) -> int:
        return self.up.numel() + self.down.numel()

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        if 0 < h.shape[0] <= DECODE_ROWS and self.up.packed is not None:
            a = amd.skinny_linear_packed_swiglu(h, self.up.packed, None, self.up.N, self.up.K)
        else:
            a = amd.silu_unit(linear(h, self.up))
        return project_to_residual(a, self.down)


class SquaredReluMlp:

    def __init__(self, get, name: str, pack: bool):
        up = get(name + ".up")
        # zero rows of `up` give zero activations: both sizes may be padded for the weight-streaming kernel
        self.up = make_weight(stack_rows([up], 32)[0], pack)
        self.down = make_weight(pad_columns(get(name + ".down")), pack)

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        if 0 < h.shape[0] <= DECODE_ROWS and self.up.packed is not None:
            a = amd.skinny_linear_packed_relu_squared(h, self.up.packed, self.up.N, self.up.K)
        else:
            a = linear(h, self.up)
            amd.relu_squared(a, a)
        return project_to_residual(a, self.down)
