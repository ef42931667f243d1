"""Sublayers of stream decoders on the gfx950 operators: the gated delta rule behind short convolutions, and the launch between two
sublayers that reads and writes all residual streams (latent attention: engine/latent_layers.py, feed-forwards: engine/moe.py and
engine/mixers.py).

A sublayer takes the normed rows h (compute dtype) and returns what it adds to the streams.  Constants come from the
configuration; nothing here knows a model's sizes."""
from typing import Optional

import torch
import torch.nn.functional as F

from .mixers import LayerCache, StepLayout, ceil_to, make_weight, pad_columns, project_to_residual, stack_rows
from .model import linear
from .moe import SublayerOutput
from .stream_config import DeltaRuleConfig

amd = torch.ops._C_amd


class StreamReader:
    """What a sublayer reads: the norm of a weighted sum of the streams."""

    def __init__(self, weights: torch.Tensor, norm: torch.Tensor):
        self.weights, self.norm = weights.float().contiguous(), norm.float().contiguous()


class StreamWriter:
    """What a sublayer leaves: every stream from all old ones (mix [from, to]) and the sublayer's output."""

    def __init__(self, mix: torch.Tensor, out: torch.Tensor):
        self.mix, self.out = mix.float().contiguous(), out.float().contiguous()

    def __call__(self, x: torch.Tensor, y: SublayerOutput, x_out: Optional[torch.Tensor], reader: StreamReader, eps: float,
                 dtype) -> torch.Tensor:
        """x, x_out [streams, rows, width] (may be the same); returns what `reader`'s sublayer takes."""
        return amd.stream_mix(x_out, x, y.y, y.slots, y.weights, self.mix, self.out, reader.weights, reader.norm, eps, dtype)


def in_pieces(w: torch.Tensor) -> torch.Tensor:
    """[rows, rank] -> [pieces, rows, 16 bytes], zeros behind the rank."""
    n = 16 // w.element_size()
    w = F.pad(w, (0, -w.shape[1] % n))
    return w.view(w.shape[0], -1, n).transpose(0, 1).contiguous()


class DeltaRule:

    def __init__(self, get, name: str, cfg: DeltaRuleConfig, eps: float, pack: bool):
        self.cfg, self.eps, self.fused = cfg, eps, True
        a2, g2 = get(name + ".a2"), get(name + ".g2")
        stack, at = stack_rows([get(f"{name}.{s}") for s in ("q", "k", "v", "a1", "g1", "b")], 32)
        self.proj = make_weight(stack, pack)
        self.k_at, self.v_at, self.channels = at[1:4]
        assert self.channels == sum(cfg.columns)
        self.conv = stack.new_zeros(cfg.taps, self.channels, dtype=torch.float32)
        for s, o in zip("qkv", at):
            w = get(f"{name}.{s}.conv").float()
            self.conv[:, o:o + w.shape[0]] = w.t()
        self.u, self.z, self.beta = (slice(o, o + n) for o, n in zip(at[3:], (a2.shape[1], g2.shape[1], cfg.heads)))
        self.z_padded = slice(self.z.start, self.z.start + ceil_to(g2.shape[1], 32))
        self.a_t = a2.float().t().contiguous()
        self.decay_w, self.gate_w = in_pieces(a2), in_pieces(g2)
        self.gate = make_weight(stack_rows([pad_columns(g2)])[0], pack)  # of portions
        self.decay_scale = get(name + ".A_log").float().exp().repeat_interleave(cfg.dim)
        self.decay_bias = get(name + ".dt_bias").float().contiguous()
        self.norm = get(name + ".norm").float().contiguous()
        self.out_cols = cfg.heads * cfg.vdim
        self.out = make_weight(pad_columns(get(name + ".o")), pack)

    def numel(self) -> int:
        """What a decode step reads of the weights."""
        return sum(w.numel() for w in (self.proj, self.out, self.decay_w, self.gate_w))

    def __call__(self, h: torch.Tensor, cache: LayerCache, step: StepLayout) -> SublayerOutput:
        c, state = self.cfg, cache.state
        proj = linear(h, self.proj)
        rows = (torch.empty if self.out.K == self.out_cols else torch.zeros)(h.shape[0], self.out.K, dtype=h.dtype, device=h.device)
        out, u, beta = rows[:, :self.out_cols], proj[:, self.u], proj[:, self.beta]
        decay = self.decay_scale, self.decay_bias
        if self.fused and step.max_query_len <= 1:
            amd.delta_step(out, proj, c.kv_heads, self.k_at, self.v_at, u, proj[:, self.z], beta, self.conv, state["conv"],
                           self.decay_w, self.gate_w, *decay, self.norm, self.eps, state["matrix"], step.state_slots, step.seq_lens)
        else:
            y = amd.short_conv(proj[:, :self.channels], self.conv, state["conv"], step.state_slots, step.query_start_loc,
                               step.seq_lens, step.max_query_len)
            gate = linear(proj[:, self.z_padded], self.gate)[:, :self.out_cols]
            amd.delta_chunks(out, y, c.kv_heads, self.k_at, self.v_at, u, beta, self.a_t, *decay, gate, self.norm, self.eps,
                             state["matrix"], step.state_slots, step.query_start_loc, step.seq_lens, step.max_query_len)
        return SublayerOutput(project_to_residual(rows, self.out))
