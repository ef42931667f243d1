"""Sublayers of latent decoders on the gfx950 operators: latent attention, and the norm on a sublayer's output with the
residual add and the average over the depth (the mixture of experts: engine/moe.py).

A mixer takes the rows h it reads (compute dtype) and returns its projection: [rows, width], or the fp32 split-K slabs of a
decode-size step; the mixture returns its assignments' rows, which the norm's launch sums.  Constants come from the
configuration; nothing here knows a model's sizes."""
from dataclasses import dataclass
from typing import Dict, List, Optional

import numpy as np
import torch
import torch.nn.functional as F

from .hybrid_config import KVSpec
from .latent_config import LatentAttentionConfig, RotationConfig
from .mixers import StepLayout, ceil_to, make_weight, pad_columns, project_to_residual, stack_rows
from .model import linear
from .moe import MixtureOfExperts, SublayerOutput, interleave_16  # noqa: F401

amd = torch.ops._C_amd
ABSORBED_MAX = 64      # portions of up to this many tokens attend in latent space (csrc/latent_attention.h)
UNBOUNDED = 1 << 30


class OutputNorm:
    """RMS norm of a sublayer's output with one gain for all coordinates, added to the stream; then, after a layer, the
    average over the depth, and after the last one the model's norm."""

    def __init__(self, get, name: str, eps: float):
        self.gain, self.eps = get(name).float().reshape(1), eps

    def __call__(self, out: SublayerOutput, x: torch.Tensor, dtype, *, x_out=None, v_out=None, streams=None, depth=None,
                 final: Optional["OutputNorm"] = None) -> torch.Tensor:
        return amd.norm_add_mix(x_out, v_out, x, out.y, out.slots, out.weights, self.gain, self.eps, streams, depth,
                                final.gain if final is not None else None, dtype)


class Rotation:
    """Full turns per position of every pair, in double: angles are reduced in double before the fp32 sine and cosine.

    The kernels turn entries 2i and 2i + 1.  Rotated entries meet in a dot product only, so that other pairs are an order of the
    rows that project queries and keys (`ordered`)."""

    def __init__(self, cfg: RotationConfig, device):
        self.cfg, self.grow = cfg, cfg.grow
        self.turns = torch.tensor(np.asarray(cfg.frequencies(), np.float64) / (2 * np.pi), dtype=torch.float64, device=device)

    def ordered(self, rows: torch.Tensor) -> torch.Tensor:
        """rows [..., rot_dim, k], of the rotated entries."""
        if not self.cfg.halves:
            return rows
        half = self.cfg.dims // 2
        at = [j for i in range(half) for j in (i, i + half)] + list(range(self.cfg.dims, rows.shape[-2]))
        return rows.index_select(-2, torch.tensor(at, device=rows.device))


@dataclass
class LongPortions:
    """A step's sequences that attend over expanded keys, for one window: where their keys lie, back to back."""
    n: int                       # gathered rows, every sequence from a multiple of 16
    starts: torch.Tensor         # int32 [num_seqs + 1]
    first: torch.Tensor          # int32 [num_seqs]: the first key taken (a multiple of the page size)
    seq_lens: torch.Tensor       # int32 [num_seqs], counted from the first key taken
    tables: torch.Tensor         # int32 [num_seqs, pages]
    max_seq_len: int


def plan_long_portions(query_lens: List[int], context_lens: List[int], window: int, longest_short: int, page: int, device):
    """None when every sequence is short."""
    q, c = np.asarray(query_lens, np.int64), np.asarray(context_lens, np.int64)
    long = q > longest_short
    if not long.any():
        return None
    first = np.maximum(c - (window or UNBOUNDED) + 1, 0) // page * page
    keys = np.where(long, c + q - first, 0)
    starts = np.zeros(len(q) + 1, np.int64)
    np.cumsum(-(-keys // page) * page, out=starts[1:])
    pages = int(-(-keys.max() // page))
    tables = starts[:-1, None] // page + np.arange(pages)[None]
    tables = np.minimum(tables, starts[-1] // page - 1)
    seq_lens = np.where(long, keys, q)
    flat = torch.from_numpy(np.concatenate([starts, first, seq_lens, tables.reshape(-1)]).astype(np.int32))
    if torch.device(device).type == "cuda":
        flat = flat.pin_memory().to(device, non_blocking=True)
    ns = len(q)
    # (pieces begin anywhere: the kernels read single int32s)
    return LongPortions(int(starts[-1]), flat[:ns + 1], flat[ns + 1:2 * ns + 1], flat[2 * ns + 1:3 * ns + 1],
                        flat[3 * ns + 1:].view(ns, pages), int(keys.max()))


class LatentStep:
    """A step's layout and what its layers share: the plans of long portions per window, gathered latents per cache."""

    def __init__(self, layout: StepLayout):
        self.layout = layout
        self._plans: Dict[int, Optional[LongPortions]] = {}
        self._gathered: Dict[tuple, torch.Tensor] = {}

    def long_portions(self, window: int) -> Optional[LongPortions]:
        l = self.layout
        if l.query_lens is None or l.max_query_len <= ABSORBED_MAX:
            return None
        if window not in self._plans:
            self._plans[window] = plan_long_portions(l.query_lens, l.context_lens, window, ABSORBED_MAX, l.block_size,
                                                     l.seq_lens.device)
        return self._plans[window]

    def gathered(self, layer: int, window: int, rows_view: torch.Tensor, plan: LongPortions) -> torch.Tensor:
        key = (layer, window)
        if key not in self._gathered:
            l = self.layout
            self._gathered[key] = amd.latent_gather(rows_view, plan.starts, plan.first, l.seq_lens, l.block_tables, plan.n)
        return self._gathered[key]


class LatentAttention:

    def __init__(self, get, name: str, cfg: LatentAttentionConfig, eps: float, pack: bool):
        self.cfg, self.eps, self.spec = cfg, eps, cfg.spec
        H = cfg.heads
        uk, uv = get(name + ".uk"), get(name + ".uv")
        self.rotation = Rotation(cfg.rot, uk.device)

        def queries(w):
            w = w.view(H, cfg.dim + cfg.rot_dim, -1)
            return torch.cat([w[:, :cfg.dim], self.rotation.ordered(w[:, cfg.dim:])], 1).reshape(H * w.shape[1], -1)
        parts = {}
        if cfg.q_rank is None:
            parts["q"], self.up = queries(get(name + ".q")), None
        else:
            parts["q"], self.q_norm = get(name + ".dq"), get(name + ".dq.norm").float()
            self.up = make_weight(stack_rows([pad_columns(queries(get(name + ".uq")))])[0], pack)
        if cfg.gate:
            parts["gate"] = get(name + ".g")
        if cfg.kv_from is None:
            dkv = get(name + ".dkv")
            parts["dkv"] = torch.cat([dkv[:cfg.kv_rank], self.rotation.ordered(dkv[cfg.kv_rank:])])
            self.norm = get(name + ".dkv.norm").float()
        stack, at = stack_rows(list(parts.values()))
        self.columns = {s: slice(o, o + p.shape[0]) for (s, p), o in zip(parts.items(), at)}
        self.proj = make_weight(stack, pack)
        self.sink = get(name + ".sink").float().contiguous() if cfg.sink else None
        dpad, vpad, cpad = ceil_to(cfg.dim, 32), ceil_to(cfg.vdim, 16), self.spec.cpad
        self.uk_t = uk.new_zeros(H, cpad, dpad)
        self.uk_t[:, :cfg.kv_rank, :cfg.dim] = uk.view(H, cfg.dim, cfg.kv_rank).transpose(1, 2)
        self.uv = uv.new_zeros(H, vpad, cpad)
        self.uv[:, :cfg.vdim, :cfg.kv_rank] = uv.view(H, cfg.vdim, cfg.kv_rank)
        self.pages = KVSpec(H, cfg.dim + cfg.rot_dim, cfg.vdim)  # of expanded keys and values
        # long portions take the expanded way where head_attention has a matrix-core body
        self.expands = uk.dtype == torch.bfloat16 and uk.is_cuda and self.pages.kpad <= 256 and self.pages.vpad <= 256
        self.expand = F.pad(torch.cat([uk, uv]), (0, cpad - cfg.kv_rank)).contiguous() if self.expands else None
        self.out_cols = H * cfg.vdim
        self.out = make_weight(pad_columns(get(name + ".o")), pack)

    def weights(self):
        return [self.proj, self.out] + ([self.up] if self.up is not None else [])

    def numel(self) -> int:
        """What a decode step reads of them."""
        return sum(w.numel() for w in self.weights()) + self.uk_t.numel() + self.uv.numel()

    def __call__(self, h: torch.Tensor, kv: torch.Tensor, layer: int, step: LatentStep, attn) -> SublayerOutput:
        """`kv`: the cache of layer number `layer`, this one's own or the one it reads."""
        c, l, spec, turns, grow = self.cfg, step.layout, self.spec, self.rotation.turns, self.rotation.grow
        proj = linear(h, self.proj)
        q, gate, dkv = (proj[:, self.columns[s]] if s in self.columns else None for s in ("q", "gate", "dkv"))
        cache = attn.rows_view(kv, spec, l.block_size)
        rows = h.shape[0]
        heads_out = (torch.empty if self.out.K == self.out_cols else torch.zeros)(rows, self.out.K, dtype=h.dtype, device=h.device)
        out = heads_out[:, :self.out_cols]
        plan = step.long_portions(c.window) if self.expands and l.block_size == 16 else None
        if self.up is not None:  # the query latents' norm; the rows' own latents go to the cache beside it
            q = amd.latent_down(q, self.q_norm, self.up.K, cache, dkv, self.norm, self.eps, spec.cpad, l.positions, turns,
                                l.slot_mapping, grow)
            q, dkv = linear(q, self.up)[:, :c.heads * (c.dim + c.rot_dim)], None
        elif plan is not None and dkv is not None:
            amd.latent_cache(cache, dkv, self.norm, self.eps, spec.cpad, l.positions, turns, l.slot_mapping, grow)
            dkv = None
        if plan is None or min(l.query_lens) <= ABSORBED_MAX:
            longest = ABSORBED_MAX if plan is not None else UNBOUNDED
            own = (dkv, self.norm) if dkv is not None else (None, None)  # (written by the same launch)
            qa = amd.latent_query(q, self.uk_t, c.dim, l.positions, turns, l.query_start_loc, longest, cache, *own, self.eps,
                                  l.slot_mapping, grow)
            amd.latent_attention(out, qa, cache, self.uv, gate, c.vdim, l.block_tables, l.seq_lens, l.query_start_loc, c.scale,
                                 c.window, longest, l.max_query_len, l.max_seq_len, self.sink)
        if plan is not None:
            self._long(out, q, gate, cache, layer, plan, step)
        return SublayerOutput(project_to_residual(heads_out, self.out))

    def _long(self, out, q, gate, cache, layer: int, plan: LongPortions, step: LatentStep) -> None:
        c, l, spec, p = self.cfg, step.layout, self.spec, self.pages
        lat = step.gathered(layer, c.window, cache, plan)
        kv = F.linear(lat[:, :spec.cpad], self.expand)
        keys, values = amd.latent_expand(kv, lat, spec.cpad, c.heads, c.dim, c.rot_dim, c.vdim, p.kpad, p.vpad)
        qr = amd.latent_rotate_query(q, c.heads, c.dim, p.kpad, l.positions, self.rotation.turns,
                                     self.rotation.grow)
        amd.head_attention(out, qr, keys, values, plan.tables, plan.seq_lens, l.query_start_loc, gate, c.vdim, c.scale, 1.0,
                           l.max_query_len, plan.max_seq_len, c.window, ABSORBED_MAX + 1, sink=self.sink)
