"""Mixture of experts on the gfx950 grouped products (csrc/moe.h): configuration and sublayer.  How tokens choose and weigh
their experts, the activation and the shared expert are parameters."""
from dataclasses import dataclass
from typing import NamedTuple, Optional

import numpy as np
import torch
import torch.nn.functional as F

from .mixers import ceil_to, pad_columns, stack_rows

amd = torch.ops._C_amd
SCORES = {"softmax": 0, "sigmoid": 1}     # include/lvllm_hip.h LVLLM_MOE_*
ACTIVATIONS = {"clamped": 0, "silu": 1, "relu_squared": 2}


class SublayerOutput(NamedTuple):
    """What a sublayer adds to the stream: rows (or split-K slabs), or the rows of a mixture's slots."""
    y: torch.Tensor
    slots: Optional[torch.Tensor] = None      # int32 [rows, assignments]
    weights: Optional[torch.Tensor] = None    # float32 [rows, assignments]; None: the rows are added as they are


@dataclass(frozen=True)
class ExpertConfig:
    ff: int
    limit: Optional[float] = None             # of the clamped activation


@dataclass(frozen=True)
class MixtureConfig:
    """`top` of `experts` small feed-forwards per token, and one that every token takes."""
    experts: int
    top: int
    expert: ExpertConfig
    shared: Optional[ExpertConfig]
    scores: str = "softmax"                   # weights: softmax over the chosen logits, or each logit's sigmoid
    activation: str = "clamped"               # g sigmoid(1.702 g) (u + 1) of clamped g, u; "silu": g sigmoid(g) u;
                                              # "relu_squared": max(u, 0)^2, without gate rows
    router_bias: bool = True
    shared_gate: bool = True                  # the shared expert is weighted by a logit of its own; else by 1
    weigh_input: bool = False                 # a weight scales what its expert reads, not what it returns
    groups: int = 1                           # equal runs of neighbouring experts, of which a token may choose from the
    keep: int = 1                             # `keep` with the largest best scores
    weight_scale: float = 1.0                 # of the chosen experts' weights

    def check(self, where: str) -> None:
        if not 1 <= self.top <= self.experts:
            raise ValueError(f"{where}: {self.top} of {self.experts} experts")
        if self.groups < 1 or self.groups > 64 or self.experts % self.groups or not 1 <= self.keep <= self.groups:
            raise ValueError(f"{where}: {self.keep} of {self.groups} groups of {self.experts} experts")
        if self.top > self.keep * (self.experts // self.groups):
            raise ValueError(f"{where}: {self.top} experts out of {self.keep} groups of {self.experts // self.groups}")


def interleave_16(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """[ff, k] twice -> [2 ffp, k]: 16 rows of one, 16 of the other, ...; ffp: ff up to a multiple of 32 with zero rows."""
    pad = ceil_to(gate.shape[0], 32) - gate.shape[0]
    g, u = (F.pad(t, (0, 0, 0, pad)).view(-1, 1, 16, t.shape[1]) for t in (gate, up))
    return torch.cat([g, u], 1).reshape(-1, gate.shape[1])


class MixtureOfExperts:
    """The shared expert is one more expert of the grouped products, with sizes and a limit of its own."""

    def __init__(self, get, name: str, cfg: MixtureConfig, pack: bool):
        self.cfg = cfg
        router = get(name + ".router")
        self.bias = get(name + ".router.b").float().contiguous() if cfg.router_bias else None
        names, ff = [f"{name}.e{i}" for i in range(cfg.experts)], [cfg.expert.ff] * cfg.experts
        limits = [cfg.expert.limit] * cfg.experts
        if cfg.shared is not None:
            names.append(name + ".shared")
            ff.append(cfg.shared.ff)
            limits.append(cfg.shared.limit)
            if cfg.shared_gate:
                router = torch.cat([router, get(name + ".shared.sg")])
        self.width, dev = router.shape[1], router.device
        self.packed = pack and router.dtype == torch.bfloat16 and self.width % 32 == 0
        self.router = amd.pack_weight(stack_rows([router])[0]) if self.packed else router.contiguous()
        ffp = [ceil_to(n, 32) for n in ff]
        self.ff_max, self.ff_first, self.ff_last, self.experts = max(ffp), max(ffp[:-1] or ffp), ffp[-1], len(names)
        gated = cfg.activation != "relu_squared"
        up_at, down_at = ([0] + np.cumsum([k * n * self.width for n in ffp]).tolist() for k in (1 + gated, 1))
        self.up = torch.empty(up_at[-1], dtype=router.dtype, device=dev)
        self.down = torch.empty(down_at[-1], dtype=router.dtype, device=dev)
        for i, s in enumerate(names):
            up = interleave_16(get(s + ".gate"), get(s + ".up")) if gated else stack_rows([get(s + ".up")], 32)[0]
            down = pad_columns(get(s + ".down")).contiguous()
            if self.packed:
                up, down = amd.pack_weight(up), amd.pack_weight(down)
            self.up[up_at[i]:up_at[i + 1]] = up.reshape(-1)
            self.down[down_at[i]:down_at[i + 1]] = down.reshape(-1)
        self.up_at, self.down_at = (torch.tensor(a[:-1], dtype=torch.int64, device=dev) for a in (up_at, down_at))
        self.ff = torch.tensor(ffp, dtype=torch.int32, device=dev)
        clamped = cfg.activation == "clamped"
        self.limits = torch.tensor(limits, dtype=torch.float32, device=dev) if clamped else None

    def numel(self) -> int:
        return self.up.numel() + self.down.numel()

    def __call__(self, h: torch.Tensor) -> SublayerOutput:
        c = self.cfg
        _, weights, offsets, token, slots, tiles, by_slot = amd.moe_route(
            h, self.router, self.bias, c.top, c.shared is not None, self.packed, c.experts, c.shared_gate, SCORES[c.scores],
            c.weigh_input, c.groups, c.keep, c.weight_scale)
        rows = h.shape[0]
        sizes = rows, self.width, self.ff_max, self.ff_first, self.ff_last
        a = amd.moe_experts(h, self.up, self.up_at, self.ff, self.limits, offsets, token, tiles, *sizes, True, self.packed,
                            by_slot if c.weigh_input else None, ACTIVATIONS[c.activation])
        y = amd.moe_experts(a, self.down, self.down_at, self.ff, None, offsets, token, tiles, *sizes, False, self.packed)
        return SublayerOutput(y, slots, None if c.weigh_input else weights)
