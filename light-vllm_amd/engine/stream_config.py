"""Configuration of stream decoders: a list of layers, each naming its mixer (latent attention whose queries come out of a latent
of their own, or the gated delta rule behind short convolutions) and its feed-forward (dense or a mixture of experts), over several
residual streams that every sublayer reads and writes with weights of its own; a run of neighbouring layers may be passed through
several times, each time with a cache or state of its own.

The engine asks for what it has to provide (`kv_cache_specs`, `state_specs`, `step_activation_bytes`), as for every model: one
entry per layer that runs."""
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch

from .latent_config import LatentAttentionConfig, LatentKVSpec, RampScaling, RotationConfig
from .moe import ExpertConfig, MixtureConfig


@dataclass(frozen=True)
class DeltaRuleConfig:
    """Heads over a matrix state; queries and keys are shared by heads / kv_heads of them."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int                      # of the convolutions

    @property
    def columns(self) -> Tuple[int, int, int]:
        """Columns of queries, keys and values, each up to a multiple of 32."""
        up = (-(-n // 32) * 32 for n in (self.kv_heads * self.dim, self.kv_heads * self.dim, self.heads * self.vdim))
        return tuple(up)


@dataclass(frozen=True)
class SiluMlpConfig:
    ff: int


@dataclass(frozen=True)
class StreamLayerConfig:
    mixer: object
    mlp: Optional[object] = None


@dataclass(frozen=True)
class LoopConfig:
    """Layers start .. stop - 1 run `times` times in a row."""
    start: int
    stop: int
    times: int


@dataclass
class StreamModelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[StreamLayerConfig]
    streams: int
    loop: Optional[LoopConfig] = None
    norm_eps: float = 1e-5
    dtype: torch.dtype = torch.bfloat16
    architecture: str = "Susalorn"
    weights_dir: Optional[str] = None     # a folder with model.safetensors; None: random weights
    random_rank: int = 16                 # inner size of the low-rank projections of random weights
    pack_weights: bool = True             # keep an MFMA-ordered copy of each projection for decode
    stream_gemm_max_rows: int = 256       # as ModelConfig's
    quantization: Optional[str] = None
    fuse_decode_ops: bool = True          # fused launches for steps of single tokens (off: they are portions of one token)
    max_position_embeddings: int = 1 << 30  # angles are computed: unlimited

    def __post_init__(self) -> None:
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("stream decoders run in bfloat16 or float32")
        if self.quantization is not None:
            raise ValueError("stream decoders have no quantised path")
        if not 1 <= self.streams <= 16:
            raise ValueError(f"{self.streams} streams: 1 to 16")
        if self.loop is not None and not (0 <= self.loop.start < self.loop.stop <= len(self.layers) and self.loop.times >= 1):
            raise ValueError(f"a loop over layers {self.loop.start} .. {self.loop.stop} of {len(self.layers)}, {self.loop.times} times")
        for i, l in enumerate(self.layers):
            m = l.mixer
            if isinstance(m, LatentAttentionConfig):
                if m.rot.dims % 2 or not 0 <= m.rot.dims <= m.rot_dim:
                    raise ValueError(f"layer {i}: {m.rot.dims} rotated entries of {m.rot_dim}")
            else:
                if m.kv_heads < 1 or m.heads % m.kv_heads:
                    raise ValueError(f"layer {i}: {m.heads} heads over {m.kv_heads}")
                if m.dim > 256 or m.vdim > 1024 or not 1 <= m.taps <= 16:
                    raise ValueError(f"layer {i}: the delta rule has keys of at most 256, values of at most 1024, 1 to 16 taps")
            if isinstance(l.mlp, MixtureConfig):
                l.mlp.check(f"layer {i}")

    @property
    def runs(self) -> List[int]:
        """The layers in the order they run."""
        n = list(range(len(self.layers)))
        if self.loop is None:
            return n
        a, b, times = self.loop.start, self.loop.stop, self.loop.times
        return n[:a] + n[a:b] * times + n[b:]

    @property
    def num_hidden_layers(self) -> int:
        return len(self.runs)

    # ---- what the engine provides ----
    def kv_cache_specs(self) -> List[Optional[LatentKVSpec]]:
        mixers = [self.layers[i].mixer for i in self.runs]
        return [m.spec if isinstance(m, LatentAttentionConfig) else None for m in mixers]

    def state_specs(self) -> List[Dict[str, Tuple[int, ...]]]:
        mixers = [self.layers[i].mixer for i in self.runs]
        return [{"matrix": (m.heads, m.dim, m.vdim), "conv": (m.taps, sum(m.columns))} if isinstance(m, DeltaRuleConfig) else {}
                for m in mixers]

    def step_activation_bytes(self, rows: int) -> int:
        """Upper bound of the activations one step of `rows` tokens keeps alive, all layers (captured steps)."""
        w = self.hidden_size
        total = (self.streams + 1) * rows * w * 4
        for i in self.runs:
            m, mlp = self.layers[i].mixer, self.layers[i].mlp
            if isinstance(m, LatentAttentionConfig):
                cols = m.heads * (m.dim + m.rot_dim + m.vdim + m.spec.row) + 2 * m.spec.row + 2 * (m.q_rank or 0)
                total += (rows * m.heads + 512 * 32) * (m.spec.cpad + 2) * 4  # shares of the attention
            else:
                cols = 4 * sum(m.columns) + 4096
            total += rows * (cols + 4 * w) * 4 + 2 * 8 * rows * w * 4
            if isinstance(mlp, MixtureConfig):
                total += rows * (mlp.top + 1) * (mlp.expert.ff + w) * 4
            elif mlp is not None:
                total += rows * 3 * mlp.ff * 4
        return total

    # ---- config.json ----
    @staticmethod
    def from_dict(c: dict, dtype: torch.dtype = torch.bfloat16, weights_dir: Optional[str] = None) -> "StreamModelConfig":
        def mixer(kind: str, m: dict):
            if kind == "latent_attention":
                r, s = m["rot"], m["rot"].get("scaling")
                scaling = None if s is None else RampScaling(float(s["factor"]), float(s["original"]), float(s["fast"]), float(s["slow"]))
                return LatentAttentionConfig(
                    int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                    RotationConfig(int(r["dims"]), float(r["base"]), True, scaling), float(m["scale"]), 0,
                    q_rank=int(m["q_rank"]), gate=False, sink=True)
            if kind == "channel_delta":
                return DeltaRuleConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), int(m["conv"]))
            raise ValueError(f"unknown mixer {kind!r}")

        def feed_forward(f: Optional[dict]):
            if f is None:
                return None
            if f["kind"] == "dense":
                return SiluMlpConfig(int(f["ff"]))
            if f["kind"] == "moe":
                r = f["router"]
                g = r.get("groups") or {"count": 1, "keep": 1}
                return MixtureConfig(int(r["experts"]), int(r["top"]), ExpertConfig(int(f["expert"]["ff"])), None,
                                     activation="relu_squared", router_bias=False, groups=int(g["count"]), keep=int(g["keep"]),
                                     weight_scale=float(r["scale"]))
            raise ValueError(f"unknown feed-forward {f['kind']!r}")

        layers = [StreamLayerConfig(mixer(e["type"], e["mixer"]), feed_forward(e.get("mlp"))) for e in c["layers"]]
        loop = c.get("loop")
        return StreamModelConfig(
            vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers, streams=int(c["streams"]),
            loop=None if loop is None else LoopConfig(int(loop["start"]), int(loop["stop"]), int(loop["times"])),
            norm_eps=float(c["norm"]["eps"]), dtype=dtype, architecture=c["architecture"], weights_dir=weights_dir)
