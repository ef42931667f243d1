"""Configuration of latent decoders: a list of layers, each with latent attention (one cached latent and one rotated key
part per token for all heads) and an optional mixture of experts, norms on what the sublayers return, and an average over
the depth after every layer.  A layer may read an earlier layer's cache instead of having one.

The engine asks for what it has to provide (`kv_cache_specs`, `state_specs`, `step_activation_bytes`), as for every model."""
import math
from dataclasses import dataclass
from typing import List, Optional

import torch

from .moe import ExpertConfig, MixtureConfig


@dataclass(frozen=True)
class RampScaling:
    """Pairs that turn `fast` times or more within `original` positions keep their frequency, those that turn `slow` times or
    less are slowed down by `factor`, a linear ramp over the pairs lies between.  Vectors grow with the logarithm of the factor."""
    factor: float
    original: float
    fast: float
    slow: float

    def __call__(self, frequencies: List[float], dims: int, base: float) -> List[float]:
        def pair(turns):  # the (fractional) pair that turns so often
            return dims * math.log(self.original / (2 * math.pi * turns)) / (2 * math.log(base))
        first, last = max(math.floor(pair(self.fast)), 0), min(math.ceil(pair(self.slow)), dims - 1)
        slowed = [min(max((i - first) / max(last - first, 1e-3), 0.0), 1.0) for i in range(len(frequencies))]
        return [f / self.factor * s + f * (1.0 - s) for f, s in zip(frequencies, slowed)]

    @property
    def grow(self) -> float:
        return 0.1 * math.log(self.factor) + 1.0


@dataclass(frozen=True)
class RotationConfig:
    """Pairs of the first `dims` entries -- (2i, 2i + 1), or (i, i + dims / 2) with `halves` -- turn by
    position * base^(-2i / dims), scaled."""
    dims: int
    base: float
    halves: bool = False
    scaling: Optional[RampScaling] = None

    def frequencies(self) -> List[float]:
        """Radians per position of every pair."""
        out = [self.base ** (-2.0 * i / self.dims) for i in range(self.dims // 2)]
        return out if self.scaling is None else self.scaling(out, self.dims, self.base)

    @property
    def grow(self) -> float:
        """What a rotated vector's length is multiplied by."""
        return 1.0 if self.scaling is None else self.scaling.grow


@dataclass(frozen=True)
class LatentKVSpec:
    """One layer's paged cache: a row per token, [latent | zeros to cpad | rotated key part | zeros to the row's end]."""
    kv_rank: int
    rot_dim: int

    @property
    def cpad(self) -> int:
        return self._padded(self.kv_rank, (64, 128, 256, 512))

    @property
    def rpad(self) -> int:
        return self._padded(self.rot_dim, (32, 64))

    @staticmethod
    def _padded(n: int, sizes) -> int:
        """The next size the MFMA body has (csrc/latent_attention_mfma.hip); beyond them multiples of 32."""
        return next((s for s in sizes if n <= s), (n + 31) // 32 * 32)

    @property
    def row(self) -> int:
        return self.cpad + self.rpad

    def block_elements(self, block_size: int) -> int:
        return self.row * block_size


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int                       # query / key size per head beside the rotated part
    rot_dim: int
    vdim: int
    kv_rank: int
    rot: RotationConfig
    scale: float
    window: int                    # keys a query sees, its own included (0: all up to its own)
    kv_from: Optional[int] = None  # the layer whose cache this one reads
    q_rank: Optional[int] = None   # queries come out of a normed latent of this size
    gate: bool = True              # a logit per head whose sigmoid scales the head's result
    sink: bool = False             # one more score per head, without a key

    @property
    def spec(self) -> LatentKVSpec:
        return LatentKVSpec(self.kv_rank, self.rot_dim)


@dataclass(frozen=True)
class LatentLayerConfig:
    mixer: LatentAttentionConfig
    mlp: Optional[MixtureConfig] = None


@dataclass
class LatentModelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[LatentLayerConfig]
    embedding_scale: float = 1.0
    norm_eps: float = 1e-5
    dtype: torch.dtype = torch.bfloat16
    architecture: str = "Lepalorn"
    weights_dir: Optional[str] = None     # a folder with model.safetensors; None: random weights
    pack_weights: bool = True             # keep an MFMA-ordered copy of each projection for decode
    stream_gemm_max_rows: int = 256       # as ModelConfig's
    quantization: Optional[str] = None
    fuse_decode_ops: bool = True          # small mixed steps (portions beside single tokens) may be captured
    max_position_embeddings: int = 1 << 30  # angles are computed: unlimited

    def __post_init__(self) -> None:
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("latent decoders run in bfloat16 or float32")
        if self.quantization is not None:
            raise ValueError("latent decoders have no quantised path")
        for i, l in enumerate(self.layers):
            m = l.mixer
            if m.rot.dims % 2 or m.rot.dims > m.rot_dim:
                raise ValueError(f"layer {i}: {m.rot.dims} rotated entries of {m.rot_dim}")
            if m.window < 1:
                raise ValueError(f"layer {i}: a window of {m.window}")
            if l.mlp is not None and not 1 <= l.mlp.top <= l.mlp.experts:
                raise ValueError(f"layer {i}: {l.mlp.top} of {l.mlp.experts} experts")
            if m.kv_from is not None:
                if not 0 <= m.kv_from < i or self.layers[m.kv_from].mixer.kv_from is not None:
                    raise ValueError(f"layer {i}: kv_from names layer {m.kv_from}, which is no earlier layer with a cache")
                s = self.layers[m.kv_from].mixer
                if (m.spec, m.rot) != (s.spec, s.rot):
                    raise ValueError(f"layer {i}: its latent or rotation differs from layer {m.kv_from}'s, whose cache it reads")

    def kv_layer(self, i: int) -> int:
        """The layer whose cache layer i reads."""
        j = self.layers[i].mixer.kv_from
        return i if j is None else j

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    # ---- what the engine provides ----
    def kv_cache_specs(self) -> List[Optional[LatentKVSpec]]:
        return [l.mixer.spec if l.mixer.kv_from is None else None for l in self.layers]

    def state_specs(self):
        """No recurrent state."""
        return None

    def step_activation_bytes(self, rows: int) -> int:
        """Upper bound of the activations one step of `rows` tokens keeps alive, all layers (captured steps)."""
        w = self.hidden_size
        total = (len(self.layers) + 1) * rows * w * 4
        for l in self.layers:
            m = l.mixer
            total += rows * (m.heads * (m.dim + m.rot_dim + m.vdim + m.spec.row) + m.spec.row + 4 * w) * 4
            total += (rows * m.heads + 512 * 32) * (m.spec.cpad + 2) * 4  # shares of the attention
            if l.mlp is not None:
                n = l.mlp.top + 1
                ff = max(l.mlp.expert.ff, l.mlp.shared.ff if l.mlp.shared is not None else 0)
                total += rows * n * (ff + w) * 4
            total += 2 * 8 * rows * w * 4
        return total

    # ---- config.json ----
    @staticmethod
    def from_dict(c: dict, dtype: torch.dtype = torch.bfloat16, weights_dir: Optional[str] = None) -> "LatentModelConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            m, mlp = e["mixer"], e.get("mlp")
            if e["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            src = m.get("kv_from")
            mixer = LatentAttentionConfig(
                int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                RotationConfig(int(m["rot"]["dims"]), float(m["rot"]["base"])), float(m["scale"]), int(m["mask"]["size"]),
                None if src is None else int(src))
            if mlp is not None and mlp["kind"] != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")

            def expert(d):
                return ExpertConfig(int(d["ff"]), float(d["limit"]))
            layers.append(LatentLayerConfig(mixer, None if mlp is None else MixtureConfig(
                int(mlp["router"]["experts"]), int(mlp["router"]["top"]), expert(mlp["expert"]),
                expert(mlp["shared"]) if mlp.get("shared") is not None else None)))
        return LatentModelConfig(vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                                 embedding_scale=float(c["embedding"]["scale"]), norm_eps=float(c["norm"]["eps"]), dtype=dtype,
                                 architecture=c["architecture"], weights_dir=weights_dir)
