"""Configuration of hybrid decoders: a list of layers, each naming its mixer (softmax attention beside gated linear
attention, RWKV-style time mixing) and its feed-forward, with every size of its own.

The engine asks a model configuration for what it has to provide, not for a family: `kv_cache_specs()` (per layer: key /
value heads of the paged cache or None) and `state_specs()` (per layer: the fp32 tensors a sequence carries)."""
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch


@dataclass(frozen=True)
class KVSpec:
    """One layer's paged cache: key and value rows of unequal size per kv head, padded for the kernels' vector loads."""
    kv_heads: int
    dim: int
    vdim: int
    maps: int = 1    # key vectors per kv head (csrc/head_attention.h), each padded by itself

    @property
    def kpad(self) -> int:
        if self.maps == 2:
            return 2 * self._padded(self.dim, (32, 64, 96, 128))
        return self._padded(self.dim, (64, 96, 128, 192, 256))

    @property
    def vpad(self) -> int:
        return self._padded(self.vdim, (32, 64, 96, 128, 192, 256))

    @staticmethod
    def _padded(n: int, sizes) -> int:
        """The next size the MFMA bodies of the attention have (csrc/head_attention.hip); beyond them multiples of 32."""
        return next((s for s in sizes if n <= s), (n + 31) // 32 * 32)

    def block_elements(self, block_size: int) -> int:
        return self.kv_heads * (self.kpad + self.vpad) * block_size


@dataclass(frozen=True)
class SoftmaxHeadsConfig:
    """Causal softmax attention without positions: normed queries and keys, one output gate per head."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float


@dataclass(frozen=True)
class LinearHeadsConfig:
    """Gated linear attention: a decay sigmoid(z)^(1/tau) per key channel."""
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class ParallelMixerConfig:
    left: SoftmaxHeadsConfig
    right: LinearHeadsConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class TimeMixerConfig:
    """RWKV-style time mixing: token shift, a decay per head and key channel, a bonus for the current token."""
    heads: int
    dim: int


@dataclass(frozen=True)
class HybridLayerConfig:
    mixer: object
    ff: Optional[int] = None           # None: the layer has no feed-forward
    weights_of: Optional[int] = None   # the layer whose tensors this one uses


@dataclass
class HybridModelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[HybridLayerConfig]
    norm_eps: float = 1e-5
    dtype: torch.dtype = torch.bfloat16
    architecture: str = "Sasilorn"
    weights_dir: Optional[str] = None     # a folder with model.safetensors; None: random weights
    random_rank: int = 16                 # inner size of the low-rank decays of random weights
    pack_weights: bool = True             # keep an MFMA-ordered copy of each projection for decode
    stream_gemm_max_rows: int = 256       # as ModelConfig's
    quantization: Optional[str] = None
    fuse_decode_ops: bool = True          # fused launches for steps of single tokens (off: the unfused sequence)
    max_position_embeddings: int = 1 << 30  # no positions anywhere: unlimited

    def __post_init__(self) -> None:
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid decoders run in bfloat16 or float32")
        if self.quantization is not None:
            raise ValueError("hybrid decoders have no quantised path")
        for i, l in enumerate(self.layers):
            j = self.weights_layer(i)
            a, b = l, self.layers[j]
            if (a.mixer, a.ff) != (b.mixer, b.ff):
                raise ValueError(f"layer {i} uses layer {j}'s weights but differs from it")

    def weights_layer(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen:
                raise ValueError(f"weights_of: layer {i} refers to itself")
            seen.add(i)
            j = self.layers[i].weights_of
            if not 0 <= j < len(self.layers):
                raise ValueError(f"weights_of: layer {i} names layer {j}")
            i = j
        return i

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    # ---- what the engine provides ----
    def kv_cache_specs(self) -> List[Optional[KVSpec]]:
        return [KVSpec(l.mixer.left.kv_heads, l.mixer.left.dim, l.mixer.left.vdim)
                if isinstance(l.mixer, ParallelMixerConfig) else None for l in self.layers]

    def state_specs(self) -> List[Dict[str, Tuple[int, ...]]]:
        out = []
        for l in self.layers:
            if isinstance(l.mixer, ParallelMixerConfig):
                r = l.mixer.right
                out.append({"matrix": (r.heads, r.dim, r.vdim)})
            else:
                out.append({"matrix": (l.mixer.heads, l.mixer.dim, l.mixer.dim), "shift": (self.hidden_size,)})
        return out

    def step_activation_bytes(self, rows: int) -> int:
        """Upper bound of the activations one step of `rows` tokens keeps alive, all layers (captured steps)."""
        total = 0
        for l in self.layers:
            if isinstance(l.mixer, ParallelMixerConfig):
                a, r = l.mixer.left, l.mixer.right
                cols = (a.heads + a.kv_heads) * (2 * a.dim + a.vdim) + 6 * r.heads * (r.dim + r.vdim)
            else:
                cols = 12 * l.mixer.heads * l.mixer.dim + 6 * self.hidden_size
            total += rows * (cols * 4 + 4 * self.hidden_size * 4 + (l.ff or 0) * 4) + 2 * 8 * rows * self.hidden_size * 4
        return total

    # ---- config.json ----
    @staticmethod
    def from_dict(c: dict, dtype: torch.dtype = torch.bfloat16, weights_dir: Optional[str] = None) -> "HybridModelConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            kind, m, mlp = e["type"], e["mixer"], e.get("mlp")
            if kind == "parallel":
                a, r = m["left"], m["right"]
                mixer = ParallelMixerConfig(
                    SoftmaxHeadsConfig(int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"])),
                    LinearHeadsConfig(int(r["heads"]), int(r["dim"]), int(r["vdim"]), float(r["tau"])),
                    float(m["left_scale"]), float(m["right_scale"]))
            elif kind == "wkv":
                mixer = TimeMixerConfig(int(m["heads"]), int(m["dim"]))
            else:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(HybridLayerConfig(mixer, None if mlp is None else int(mlp["ff"]), e.get("weights_of")))
        return HybridModelConfig(vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                                 norm_eps=float(c["norm"]["eps"]), dtype=dtype, architecture=c["architecture"],
                                 weights_dir=weights_dir)
