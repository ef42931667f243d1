"""Decoder of local-attention layers (engine/local_config.py): embedding -> layers -> norm -> head, over the engine's paged
caches and state slots.  Serves prompts, portions of prompts and decoded tokens in one batch; every tensor that steers a step is
on the device, so decode steps are captured as they are."""
from typing import Dict, List

import torch

from .layered_model import LayeredModel
from .local_config import LocalModelConfig, ParallelHeadsConfig, RetentionConfig, RotaryHeadsConfig
from .local_layers import AttentionMixer, ClampedMlp, MixtureMlp, ParallelHeads, SandwichNorm
from .moe import MixtureConfig

amd = torch.ops._C_amd


def heads_shapes(name: str, a: RotaryHeadsConfig, width: int) -> Dict[str, tuple]:
    out = {f"{name}.q": (a.heads * a.maps * a.dim, width), f"{name}.k": (a.kv_heads * a.maps * a.dim, width),
           f"{name}.o": (width, a.heads * a.vdim)}
    if not a.keys_are_values:
        out[f"{name}.v"] = (a.kv_heads * a.vdim, width)
    if a.bias:
        out.update({s + ".b": shape[:1] for s, shape in list(out.items())})
    if a.norm:
        out.update({f"{name}.q.norm": (a.heads * a.dim,), f"{name}.k.norm": (a.kv_heads * a.dim,)})
    if a.sink:
        out[f"{name}.sink"] = (a.heads,)
    if a.diff is not None:
        out.update({f"{name}.{s}": (a.dim,) for s in ("lq1", "lk1", "lq2", "lk2")})
    return out


def retention_shapes(name: str, r: RetentionConfig, width: int) -> Dict[str, tuple]:
    k, v = (r.heads * r.dim, width), (r.heads * r.vdim, width)
    return {f"{name}.q": k, f"{name}.k": k, f"{name}.v": v, f"{name}.g": v, f"{name}.o": v[::-1]}


class LocalModel(LayeredModel):

    @staticmethod
    def tensor_shapes(cfg: LocalModelConfig) -> Dict[str, tuple]:
        w = cfg.hidden_size
        out: Dict[str, tuple] = {"embed": (cfg.vocab_size, w), "head": (cfg.vocab_size, w), "final.norm": (w,)}
        if cfg.pairs is not None:
            out["bigram"] = (cfg.pairs.buckets + 1, w)
        for i, l in enumerate(cfg.layers):
            p = f"l{i}"
            out.update({p + ".norm1": (w,), p + ".norm1b": (w,)})
            if isinstance(l.mixer, ParallelHeadsConfig):
                out.update(heads_shapes(p + ".mix.left", l.mixer.left, w))
                out.update(retention_shapes(p + ".mix.right", l.mixer.right, w))
                out.update({p + ".mix.left.out": (w,), p + ".mix.right.out": (w,)})
            else:
                out.update(heads_shapes(p + ".mix", l.mixer, w))
            if l.mlp is None:
                continue
            out.update({p + ".norm2": (w,), p + ".norm2b": (w,)})
            experts = [(p + ".mlp", l.mlp)]
            if isinstance(l.mlp, MixtureConfig):
                experts = [(f"{p}.mlp.e{e}", l.mlp.expert) for e in range(l.mlp.experts)]
                out[p + ".mlp.router"] = (l.mlp.experts, w)
                if l.mlp.shared is not None:
                    experts.append((p + ".mlp.shared", l.mlp.shared))
            for e, c in experts:
                out.update({e + ".gate": (c.ff, w), e + ".up": (c.ff, w), e + ".down": (w, c.ff)})
        return out

    @staticmethod
    def random_tensor(name: str, shape: tuple, gen: torch.Generator, device) -> torch.Tensor:
        """Random weights of sane magnitude: projections of variance 1 / fan-in, norms near 1."""
        t = torch.randn(shape, generator=gen, device=device)
        if name.endswith(("norm", "norm1", "norm1b", "norm2", "norm2b", ".out")):
            return 1.0 + 0.1 * t
        if name.endswith((".b", ".lq1", ".lk1", ".lq2", ".lk2")):
            return 0.1 * t
        if len(shape) == 1 or name in ("embed", "bigram"):
            return t
        return t * shape[-1] ** -0.5

    def load(self, get, pack: bool) -> None:
        cfg, eps = self.cfg, self.cfg.norm_eps
        self.embed = get("embed").contiguous()
        self.pairs = get("bigram").contiguous() if cfg.pairs is not None else None
        self.layers: List[tuple] = []
        before, norms = [], []  # the norms in front of the sublayers, those behind them
        for i, l in enumerate(cfg.layers):
            p = f"l{i}"
            before.append(get(p + ".norm1").float().contiguous())
            norms.append(SandwichNorm(get, p + ".norm1b", eps))
            kind = ParallelHeads if isinstance(l.mixer, ParallelHeadsConfig) else AttentionMixer
            sub = [(kind(get, p + ".mix", l.mixer, eps, pack), norms[-1])]
            if l.mlp is not None:
                before.append(get(p + ".norm2").float().contiguous())
                norms.append(SandwichNorm(get, p + ".norm2b", eps))
                kind = MixtureMlp if isinstance(l.mlp, MixtureConfig) else ClampedMlp
                sub.append((kind(get, p + ".mlp", l.mlp, pack), norms[-1]))
            self.layers.append(tuple(sub))
        before.append(get("final.norm").float().contiguous())
        self.first_norm = before[0]
        for norm, weight in zip(norms, before[1:]):
            norm.next_weight = weight

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches, attn_metadata, on_layer=None) -> torch.Tensor:
        """`on_layer(i, x)`: called with the residual stream after every layer (tests)."""
        cfg, dtype = self.cfg, self.cfg.dtype
        step = self.step_layout(attn_metadata, positions, caches.block_size)
        x = torch.empty(input_ids.shape[0], cfg.hidden_size, dtype=torch.float32, device=self.device)
        mul = (cfg.pairs.mul_previous, cfg.pairs.mul_current) if cfg.pairs is not None else (0, 0)
        h = amd.pair_embed(x, self.embed, self.pairs, input_ids, caches.sequence["previous_token"], step.state_slots,
                           step.query_start_loc, step.seq_lens, *mul, self.first_norm, cfg.norm_eps)
        for i, (((mixer, norm), *ff), cache) in enumerate(zip(self.layers, caches.layers)):
            h = norm(x, mixer(h, cache, step, self.attn), dtype)
            for mlp, norm in ff:
                h = norm(x, mlp(h), dtype)
            if on_layer is not None:
                on_layer(i, x.clone())
        return h

    def weight_bytes(self) -> int:
        """Bytes of the projections and of all experts (a decode step reads the experts its tokens take)."""
        n = self.head.numel()
        for (mixer, _), *ff in self.layers:
            n += sum(w.numel() for w in mixer.weights()) + sum(mlp.numel() for mlp, _ in ff)
        return n * torch.empty((), dtype=self.cfg.dtype).element_size()
