"""Sublayers of local decoders on the gfx950 operators: rotary attention over windows, chunks and kept first tokens (one
softmax per head or the difference of two), retention, both side by side, the clamped feed-forward, and the norms around a
sublayer.

A sublayer takes the normed rows h (compute dtype) and returns what it adds to the stream, which one launch norms, adds and norms
again for the next sublayer.  Constants come from the configuration; nothing here knows a model's sizes."""
from typing import List, NamedTuple, Optional

import numpy as np
import torch

from .local_config import ClampedMlpConfig, ParallelHeadsConfig, RetentionConfig, RotaryConfig, RotaryHeadsConfig
from .mixers import DECODE_ROWS, LayerCache, StepLayout, make_weight, pad_columns, project_to_residual, stack_rows
from .model import Weight, linear
from .moe import MixtureOfExperts

amd = torch.ops._C_amd


class Branch(NamedTuple):
    """A sublayer's output: rows, split-K slabs, or (with slots) the rows of a mixture's slots, which are added."""
    y: torch.Tensor
    bias: Optional[torch.Tensor] = None
    slots: Optional[torch.Tensor] = None


class SandwichNorm:
    """x += norm of the sublayer's output, then the norm in front of the next sublayer (`next_weight`)."""

    def __init__(self, get, name: str, eps: float):
        self.weight, self.eps, self.next_weight = get(name).float().contiguous(), eps, None

    def __call__(self, x: torch.Tensor, out, dtype) -> torch.Tensor:
        """x is changed in place; `out`: a Branch, or two of them with their norms' weights."""
        if isinstance(out, Branch):
            return amd.sandwich_norm(x, out.y, out.slots, out.bias, None, None, None, None, self.weight, self.next_weight,
                                     self.eps, dtype)
        (a, wa), (b, wb) = out
        return amd.sandwich_norm(x, a.y, a.slots, a.bias, wa, b.y, b.bias, wb, self.weight, self.next_weight, self.eps, dtype)


class Projections:
    """Several projections of one input as one product, with their biases; columns by name."""

    def __init__(self, get, parts: List[tuple], pack: bool):
        """parts: (name, bias or not)"""
        ws = [get(name) for name, _ in parts]
        stack, at = stack_rows(ws)
        self.columns = [slice(o, o + w.shape[0]) for o, w in zip(at, ws)]
        self.weight = make_weight(stack, pack)
        self.bias = None
        if any(b for _, b in parts):
            self.bias = stack.new_zeros(stack.shape[0])
            for (name, b), c in zip(parts, self.columns):
                if b:
                    self.bias[c] = get(name + ".b")

    def __call__(self, h: torch.Tensor) -> List[torch.Tensor]:
        y = linear(h, self.weight, self.bias)
        return [y[:, c] for c in self.columns]


class OutputProjection:
    """W_o, its bias left to the launch that reads the result."""

    def __init__(self, get, name: str, bias: bool, pack: bool):
        w = get(name)
        self.cols = w.shape[1]
        self.weight = make_weight(pad_columns(w), pack)
        self.bias = get(name + ".b").float().contiguous() if bias else None

    def rows(self, h: torch.Tensor) -> torch.Tensor:
        """Where the heads' results go: [rows, columns up to the padded size], the padding zero."""
        make = torch.empty if self.weight.K == self.cols else torch.zeros
        return make(h.shape[0], self.weight.K, dtype=h.dtype, device=h.device)

    def __call__(self, rows: torch.Tensor) -> Branch:
        return Branch(project_to_residual(rows, self.weight), self.bias)


def turns_of(cfg: RotaryConfig, device) -> torch.Tensor:
    """Full turns per position of every pair, in double: angles are reduced in double before the fp32 sine and cosine."""
    return torch.tensor(np.asarray(cfg.frequencies(), np.float64) / (2 * np.pi), dtype=torch.float64, device=device)


class RotaryHeads:
    """Softmax attention with rotary positions over the paged cache."""

    def __init__(self, get, name: str, cfg: RotaryHeadsConfig, eps: float, pack: bool):
        self.cfg, self.eps, self.spec = cfg, eps, cfg.spec
        self.parts = [(f"{name}.{s}", cfg.bias) for s in ("qk" if cfg.keys_are_values else "qkv")]
        self.q_norm, self.k_norm = (get(f"{name}.{s}.norm").float().contiguous() if cfg.norm else None for s in "qk")
        self.sink = get(name + ".sink").float().contiguous() if cfg.sink else None
        self.map_weight, self.out_scale = 0.0, 1.0
        if cfg.diff is not None:
            lq1, lk1, lq2, lk2 = (get(f"{name}.{s}").double() for s in ("lq1", "lk1", "lq2", "lk2"))
            self.map_weight = float((lq1 * lk1).sum().exp() - (lq2 * lk2).sum().exp()) + cfg.diff
            self.out_scale = 1.0 - cfg.diff
        self.out = OutputProjection(get, name + ".o", cfg.bias, pack)
        self.turns = turns_of(cfg.rot, self.out.weight.w.device)

    def attend(self, cols: List[torch.Tensor], cache: LayerCache, step: StepLayout, attn) -> Branch:
        """cols: what `parts` project to."""
        c, (q, k) = self.cfg, cols[:2]
        v = k if c.keys_are_values else cols[2]
        kc, vc = attn.split_kv_cache(cache.kv, self.spec, step.block_size)
        rot = amd.rotary_cache(q, k, v, self.q_norm, self.k_norm, self.eps, c.heads, c.kv_heads, c.maps, step.positions,
                               self.turns, kc, vc, step.slot_mapping)
        rows = self.out.rows(q)
        shortest = min(step.query_lens) if step.query_lens else 0  # (no short portions: no launch for them)
        amd.head_attention(rows[:, :self.out.cols], rot, kc, vc, step.block_tables, step.seq_lens, step.query_start_loc, None,
                           c.vdim, c.scale, self.out_scale, step.max_query_len, step.max_seq_len, c.sees.window, shortest,
                           c.sees.chunk, c.sees.keep_first, c.softcap, self.sink, c.maps, self.map_weight, self.eps)
        return self.out(rows)


class RetentionHeads:

    def __init__(self, get, name: str, cfg: RetentionConfig, eps: float, pack: bool):
        self.cfg, self.eps = cfg, eps
        self.parts = [(f"{name}.{s}", False) for s in "qkvg"]
        self.out = OutputProjection(get, name + ".o", False, pack)
        dev = self.out.weight.w.device
        self.turns = turns_of(cfg.rot, dev)
        decay = torch.tensor(cfg.decay, dtype=torch.float64)
        # (a finite logarithm of no memory at all keeps sums of logarithms finite)
        self.decay = torch.stack([decay, decay.log().clamp_min(-1e4)]).float().to(dev)

    def attend(self, cols: List[torch.Tensor], cache: LayerCache, step: StepLayout) -> Branch:
        c, (q, k, v, g) = self.cfg, cols
        rows = self.out.rows(q)
        amd.retention(rows[:, :self.out.cols], q, k, v, step.positions, self.turns, self.decay, c.dim ** -0.5, g, None, self.eps,
                      1.0, cache.state["matrix"], step.state_slots, step.query_start_loc, step.seq_lens, step.max_query_len)
        return self.out(rows)


class AttentionMixer:

    def __init__(self, get, name: str, cfg: RotaryHeadsConfig, eps: float, pack: bool):
        self.heads = RotaryHeads(get, name, cfg, eps, pack)
        self.proj = Projections(get, self.heads.parts, pack)

    def weights(self) -> List[Weight]:
        return [self.proj.weight, self.heads.out.weight]

    def __call__(self, h: torch.Tensor, cache: LayerCache, step: StepLayout, attn) -> Branch:
        return self.heads.attend(self.proj(h), cache, step, attn)


class ParallelHeads:
    """Attention and retention over one input projection; each result has a norm of its own."""

    def __init__(self, get, name: str, cfg: ParallelHeadsConfig, eps: float, pack: bool):
        self.left = RotaryHeads(get, name + ".left", cfg.left, eps, pack)
        self.right = RetentionHeads(get, name + ".right", cfg.right, eps, pack)
        self.proj = Projections(get, self.left.parts + self.right.parts, pack)
        self.norms = [get(f"{name}.{s}.out").float().contiguous() for s in ("left", "right")]

    def weights(self) -> List[Weight]:
        return [self.proj.weight, self.left.out.weight, self.right.out.weight]

    def __call__(self, h: torch.Tensor, cache: LayerCache, step: StepLayout, attn):
        cols, n = self.proj(h), len(self.left.parts)
        left = self.left.attend(cols[:n], cache, step, attn)
        return (left, self.norms[0]), (self.right.attend(cols[n:], cache, step), self.norms[1])


class ClampedMlp:

    def __init__(self, get, name: str, cfg: ClampedMlpConfig, pack: bool):
        self.limit = cfg.limit
        # zero rows of gate and up give zero activations: all sizes may be padded for the weight-streaming kernel
        self.up = make_weight(stack_rows([get(name + ".gate"), get(name + ".up")], 32)[0], pack)
        self.down = make_weight(pad_columns(get(name + ".down")), pack)

    def numel(self) -> int:
        return self.up.numel() + self.down.numel()

    def __call__(self, h: torch.Tensor) -> Branch:
        if 0 < h.shape[0] <= DECODE_ROWS and self.up.packed is not None:
            a = amd.skinny_linear_packed_clamped_unit(h, self.up.packed, self.up.N, self.up.K, self.limit)
        else:
            a = amd.clamped_unit(linear(h, self.up), self.limit)
        return Branch(project_to_residual(a, self.down))


class MixtureMlp(MixtureOfExperts):

    def __call__(self, h: torch.Tensor) -> Branch:
        out = super().__call__(h)
        return Branch(out.y, slots=out.slots)
