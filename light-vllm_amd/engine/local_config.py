"""Configuration of local decoders: a list of layers, each naming its mixer (rotary attention over a window, over a window
beside kept first tokens as the difference of two softmaxes, or over chunks in parallel with retention) and its feed-forward
(dense or a mixture of experts), every sublayer between two norms.

The engine asks for what it has to provide (`kv_cache_specs`, `state_specs`, `sequence_state_specs`,
`step_activation_bytes`), as for every model."""
import math
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch

from .hybrid_config import KVSpec
from .moe import ExpertConfig, MixtureConfig


@dataclass(frozen=True)
class FrequencyScaling:
    """Pairs that turn often within `original` positions (over `high` times) keep their frequency, those that do so less than
    `low` times are slowed down by `factor`, those between are blended."""
    factor: float
    low: float
    high: float
    original: float

    def __call__(self, f: float) -> float:
        n = self.original * f / (2 * math.pi)   # turns within the original length
        if n > self.high:
            return f
        if n < self.low:
            return f / self.factor
        s = (n - self.low) / (self.high - self.low)
        return (1 - s) * f / self.factor + s * f


@dataclass(frozen=True)
class RotaryConfig:
    """Entries i and i + dims / 2 turn by position * base^(-2i / dims), scaled."""
    dims: int
    base: float
    scaling: Optional[FrequencyScaling] = None

    def frequencies(self) -> List[float]:
        """Radians per position of every pair."""
        out = [self.base ** (-2.0 * i / self.dims) for i in range(self.dims // 2)]
        return out if self.scaling is None else [self.scaling(f) for f in out]


@dataclass(frozen=True)
class VisibleKeys:
    """Of the keys up to its own a query sees the last `window`, those of its own aligned run of `chunk` positions, and the
    first `keep_first` (0: not limited, none kept)."""
    window: int = 0
    chunk: int = 0
    keep_first: int = 0


@dataclass(frozen=True)
class RotaryHeadsConfig:
    """Softmax attention with rotary positions."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotaryConfig
    sees: VisibleKeys
    bias: bool = False             # of all projections
    keys_are_values: bool = False  # as projected, before norm and rotation
    norm: bool = False             # queries and keys are RMS normed over all heads at once
    softcap: float = 0.0
    sink: bool = False
    diff: Optional[float] = None   # two softmaxes per head over the same values; their difference, normed per head

    @property
    def maps(self) -> int:
        return 1 if self.diff is None else 2

    @property
    def spec(self) -> KVSpec:
        return KVSpec(self.kv_heads, self.dim, self.vdim, self.maps)


@dataclass(frozen=True)
class RetentionConfig:
    """Linear attention with a fixed decay per head."""
    heads: int
    dim: int
    vdim: int
    rot: RotaryConfig
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class ParallelHeadsConfig:
    """Half the sum of both mixers' normed outputs."""
    left: RotaryHeadsConfig
    right: RetentionConfig


@dataclass(frozen=True)
class ClampedMlpConfig:
    ff: int
    limit: float


@dataclass(frozen=True)
class PairTableConfig:
    """A second embedding: row (previous token * mul_previous + token * mul_current) mod buckets, the last one at the start."""
    buckets: int
    mul_previous: int
    mul_current: int


@dataclass(frozen=True)
class LocalLayerConfig:
    mixer: object
    mlp: Optional[object] = None


@dataclass
class LocalModelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[LocalLayerConfig]
    pairs: Optional[PairTableConfig] = None
    norm_eps: float = 1e-6
    dtype: torch.dtype = torch.bfloat16
    architecture: str = "Lizazen"
    weights_dir: Optional[str] = None     # a folder with model.safetensors; None: random weights
    pack_weights: bool = True             # keep an MFMA-ordered copy of each projection for decode
    stream_gemm_max_rows: int = 256       # as ModelConfig's
    quantization: Optional[str] = None
    fuse_decode_ops: bool = True
    max_position_embeddings: int = 1 << 30  # angles are computed: unlimited

    def __post_init__(self) -> None:
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("local decoders run in bfloat16 or float32")
        if self.quantization is not None:
            raise ValueError("local decoders have no quantised path")
        p = self.pairs
        if p is not None and (p.buckets < 1 or p.mul_previous < 0 or p.mul_current < 0):
            raise ValueError("a table of token pairs has buckets, and multipliers that are not negative")
        for i, l in enumerate(self.layers):
            for a in self.attention_of(l), self.retention_of(l):
                if a is not None and (a.rot.dims % 2 or not 0 <= a.rot.dims <= a.dim):
                    raise ValueError(f"layer {i}: {a.rot.dims} rotated entries of {a.dim}")
            a, r = self.attention_of(l), self.retention_of(l)
            if a.heads % a.kv_heads:
                raise ValueError(f"layer {i}: {a.heads} heads over {a.kv_heads}")
            if min(a.sees.window, a.sees.chunk, a.sees.keep_first) < 0:
                raise ValueError(f"layer {i}: a negative window, chunk or number of kept tokens")
            if a.keys_are_values and a.dim != a.vdim:
                raise ValueError(f"layer {i}: keys of {a.dim} as values of {a.vdim}")
            if r is not None and (len(r.decay) != r.heads or not all(0.0 <= d <= 1.0 for d in r.decay)):
                raise ValueError(f"layer {i}: a decay in 0 .. 1 per head")
            if r is not None and (r.dim > 256 or r.vdim > 1024):
                raise ValueError(f"layer {i}: retention has keys of at most 256, values of at most 1024")
            if isinstance(l.mlp, MixtureConfig) and not 1 <= l.mlp.top <= l.mlp.experts:
                raise ValueError(f"layer {i}: {l.mlp.top} of {l.mlp.experts} experts")

    @staticmethod
    def attention_of(l: LocalLayerConfig) -> RotaryHeadsConfig:
        return l.mixer.left if isinstance(l.mixer, ParallelHeadsConfig) else l.mixer

    @staticmethod
    def retention_of(l: LocalLayerConfig) -> Optional[RetentionConfig]:
        return l.mixer.right if isinstance(l.mixer, ParallelHeadsConfig) else None

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    # ---- what the engine provides ----
    def kv_cache_specs(self) -> List[Optional[KVSpec]]:
        return [self.attention_of(l).spec for l in self.layers]

    def state_specs(self) -> List[Dict[str, Tuple[int, ...]]]:
        rs = [self.retention_of(l) for l in self.layers]
        return [{} if r is None else {"matrix": (r.heads, r.dim, r.vdim)} for r in rs]

    def sequence_state_specs(self) -> Dict[str, Tuple[Tuple[int, ...], torch.dtype]]:
        """What a sequence carries besides its layers' states."""
        return {"previous_token": ((), torch.int32)}

    def step_activation_bytes(self, rows: int) -> int:
        """Upper bound of the activations one step of `rows` tokens keeps alive, all layers (captured steps)."""
        w = self.hidden_size
        total = rows * w * 8
        for l in self.layers:
            a, r = self.attention_of(l), self.retention_of(l)
            cols = (2 * a.heads + a.kv_heads) * a.spec.kpad + (a.heads + a.kv_heads) * a.spec.vpad
            if r is not None:
                cols += 6 * r.heads * (r.dim + r.vdim)
            # shares of the attention, slabs of the projections
            total += rows * (cols + 6 * w) * 4 + rows * a.heads * a.maps * 64 * (a.spec.vpad + 2) * 4 + 3 * 8 * rows * w * 4
            if isinstance(l.mlp, MixtureConfig):
                ff = max(l.mlp.expert.ff, l.mlp.shared.ff if l.mlp.shared is not None else 0)
                total += rows * (l.mlp.top + 1) * (ff + w) * 4
            elif l.mlp is not None:
                total += rows * 3 * l.mlp.ff * 4
        return total

    # ---- config.json ----
    @staticmethod
    def from_dict(c: dict, dtype: torch.dtype = torch.bfloat16, weights_dir: Optional[str] = None) -> "LocalModelConfig":
        def rotary(m: dict) -> RotaryConfig:
            r, s = m["rot"], m["rot"].get("scaling")
            return RotaryConfig(int(r["dims"]), float(r["base"]), None if s is None else FrequencyScaling(
                float(s["factor"]), float(s["low"]), float(s["high"]), float(s["original"])))

        def heads(m: dict, sees: VisibleKeys, **kw) -> RotaryHeadsConfig:
            if min(sees.window or 1, sees.chunk or 1) < 1 or not (sees.window or sees.chunk):
                raise ValueError(f"a window or chunk of {m['mask']['size']}")
            return RotaryHeadsConfig(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]),
                                     rotary(m), sees, **kw)

        def mixer(kind: str, m: dict):
            if kind == "attention":
                return heads(m, VisibleKeys(window=int(m["mask"]["size"])), bias=True, keys_are_values=True, norm=True,
                             softcap=float(m["softcap"]), sink=True)
            if kind == "attention_2":
                k = m["mask"]
                return heads(m, VisibleKeys(window=int(k["size"]), keep_first=int(k["keep_first"])), diff=float(m["diff"]))
            if kind == "parallel":
                l, r = m["left"], m["right"]
                return ParallelHeadsConfig(
                    heads(l, VisibleKeys(chunk=int(l["mask"]["size"])), bias=True),
                    RetentionConfig(int(r["heads"]), int(r["dim"]), int(r["vdim"]), rotary(r), tuple(map(float, r["decay"]))))
            raise ValueError(f"unknown mixer {kind!r}")

        def feed_forward(f: Optional[dict]):
            if f is None:
                return None
            if f["kind"] == "dense":
                return ClampedMlpConfig(int(f["ff"]), float(f["limit"]))
            if f["kind"] == "moe":
                shared = f.get("shared")
                return MixtureConfig(int(f["router"]["experts"]), int(f["router"]["top"]), ExpertConfig(int(f["expert"]["ff"])),
                                     None if shared is None else ExpertConfig(int(shared["ff"])), scores="sigmoid",
                                     activation="silu", router_bias=False, shared_gate=False, weigh_input=True)
            raise ValueError(f"unknown feed-forward {f['kind']!r}")

        layers = [LocalLayerConfig(mixer(e["type"], e["mixer"]), feed_forward(e.get("mlp"))) for e in c["layers"]]
        b = c["embedding"].get("bigram")
        return LocalModelConfig(
            vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
            pairs=None if b is None else PairTableConfig(int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])),
            norm_eps=float(c["norm"]["eps"]), dtype=dtype, architecture=c["architecture"], weights_dir=weights_dir)
