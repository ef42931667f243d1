"""Decoder of mixed layers (engine/hybrid_config.py): embedding -> layers -> norm -> head, over the engine's paged caches
and state slots.  Serves prompts, portions of prompts and decoded tokens in one batch; every tensor that steers a step is
on the device, so decode steps are captured as they are."""
from typing import Dict, List, Optional

import torch
import torch.nn.functional as F

from .hybrid_config import HybridModelConfig, ParallelMixerConfig
from .layered_model import LayeredModel
from .mixers import DynTanhNorm, LayerCache, ParallelMixer, SquaredReluMlp, TimeMixer


def tensor_shapes(cfg: HybridModelConfig) -> Dict[str, tuple]:
    """Names and shapes of the tensors a model of `cfg` has (low ranks: cfg.random_rank)."""
    w, rank = cfg.hidden_size, cfg.random_rank
    out: Dict[str, tuple] = {"embed": (cfg.vocab_size, w), "head": (cfg.vocab_size, w)}

    def norm(name):
        out[name], out[name + ".b"], out[name + ".alpha"] = (w,), (w,), ()
    norm("final.norm")
    for i, l in enumerate(cfg.layers):
        if cfg.weights_layer(i) != i:
            continue
        p = f"l{i}"
        norm(p + ".norm1")
        if isinstance(l.mixer, ParallelMixerConfig):
            a, r = l.mixer.left, l.mixer.right
            m = p + ".mix.left"
            out.update({m + ".q": (a.heads * a.dim, w), m + ".k": (a.kv_heads * a.dim, w), m + ".v": (a.kv_heads * a.vdim, w),
                        m + ".q.norm": (a.dim,), m + ".k.norm": (a.dim,), m + ".g": (a.heads, w), m + ".o": (w, a.heads * a.vdim)})
            m = p + ".mix.right"
            out.update({m + ".q": (r.heads * r.dim, w), m + ".k": (r.heads * r.dim, w), m + ".v": (r.heads * r.vdim, w),
                        m + ".g": (r.heads * r.vdim, w), m + ".o": (w, r.heads * r.vdim), m + ".norm": (r.vdim,),
                        m + ".a1": (rank, w), m + ".a2": (r.heads * r.dim, rank), m + ".a2.b": (r.heads * r.dim,)})
        else:
            m, n = p + ".mix", l.mixer.heads * l.mixer.dim
            out.update({f"{m}.mu.{s}": (w,) for s in TimeMixer.MIXES})
            out.update({f"{m}.{s}": (n, w) for s in "rkvg"})
            out.update({m + ".w1": (rank, w), m + ".w2": (n, rank), m + ".w0": (n,), m + ".u": (l.mixer.heads, l.mixer.dim),
                        m + ".norm": (n,), m + ".o": (w, n)})
        if l.ff is not None:
            norm(p + ".norm2")
            out.update({p + ".mlp.up": (l.ff, w), p + ".mlp.down": (w, l.ff)})
    return out


def random_tensor(name: str, shape: tuple, gen: torch.Generator, device) -> torch.Tensor:
    """Random weights of sane magnitude: projections of variance 1 / fan-in, norms near 1, decays spread over short and
    long memories."""
    t = torch.randn(shape, generator=gen, device=device)
    if name.endswith(".alpha"):
        return torch.full(shape, 0.5, device=device)
    if name.endswith("norm"):
        return 1.0 + 0.1 * t
    if name.endswith("norm1") or name.endswith("norm2"):
        return 1.0 + 0.1 * t
    if name.endswith("norm.b") or name.endswith("norm1.b") or name.endswith("norm2.b"):
        return 0.1 * t
    if ".mu." in name:
        return torch.rand(shape, generator=gen, device=device)
    if name.endswith(".w0"):
        return -6.0 + 5.5 * torch.rand(shape, generator=gen, device=device)
    if name.endswith(".a2.b"):
        return 2.0 + t
    if name.endswith(".u"):
        return 0.5 * t
    if name == "embed":
        return t
    return t * shape[-1] ** -0.5


class HybridModel(LayeredModel):

    tensor_shapes, random_tensor = staticmethod(tensor_shapes), staticmethod(random_tensor)

    def load(self, get, pack: bool) -> None:
        cfg = self.cfg
        self.embed = get("embed").float()
        self.layers: List[tuple] = []
        for i, l in enumerate(cfg.layers):
            j = cfg.weights_layer(i)
            if j != i and j < i:
                self.layers.append(self.layers[j])
            else:
                self.layers.append(self._layer(get, f"l{j}", l, pack))
        self.final_norm = DynTanhNorm(get, "final.norm")

    def _layer(self, get, name: str, l, pack: bool):
        mixer = (ParallelMixer if isinstance(l.mixer, ParallelMixerConfig) else TimeMixer)(
            get, name + ".mix", l.mixer, self.cfg.norm_eps, pack)
        mixer.recurrence.fused = self.cfg.fuse_decode_ops
        ff = (DynTanhNorm(get, name + ".norm2"), SquaredReluMlp(get, name + ".mlp", pack)) if l.ff is not None else None
        return DynTanhNorm(get, name + ".norm1"), mixer, ff

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches: List[LayerCache], attn_metadata,
                on_layer=None) -> torch.Tensor:
        """`on_layer(i, x)`: called with the residual stream after every layer (tests)."""
        dtype = self.cfg.dtype
        step = self.step_layout(attn_metadata, positions, caches.block_size)
        x, y = F.embedding(input_ids, self.embed), None
        for i, ((norm1, mixer, ff), cache) in enumerate(zip(self.layers, caches.layers)):
            x, y = mixer(x, y, norm1, cache, step, self.attn, dtype)
            if ff is not None:
                norm2, mlp = ff
                y = mlp(norm2(x, y, dtype))
            if on_layer is not None:
                on_layer(i, x + (y.sum(0) if y.dim() == 3 else y).float())
        return self.final_norm(x, y, dtype)

    def weight_bytes(self) -> int:
        n, seen = self.head.numel(), set()
        for norm1, mixer, ff in self.layers:
            if id(mixer) in seen:
                continue
            seen.add(id(mixer))
            ws = [mixer.proj, mixer.out] if isinstance(mixer, ParallelMixer) else [*mixer.rkvg, mixer.w1, mixer.out]
            if ff is not None:
                ws += [ff[1].up, ff[1].down]
            n += sum(w.numel() for w in ws)
        return n * torch.empty((), dtype=self.cfg.dtype).element_size()
