"""Decoder of latent-attention and delta-rule layers over several residual streams (engine/stream_config.py): embedding -> layers,
some of them several times -> norm -> the embedding table as the head, over the engine's paged caches and state slots.  Serves
prompts, portions of prompts and decoded tokens in one batch; every tensor that steers a step of single tokens is on the device, so
decode steps are captured as they are."""
from typing import Dict, List

import torch

from .latent_config import LatentAttentionConfig
from .latent_layers import LatentAttention, LatentStep
from .layered_model import LayeredModel
from .mixers import SiluMlp
from .moe import MixtureConfig, MixtureOfExperts, SublayerOutput
from .stream_config import StreamModelConfig
from .stream_layers import DeltaRule, StreamReader, StreamWriter

amd = torch.ops._C_amd


class StreamModel(LayeredModel):

    @staticmethod
    def tensor_shapes(cfg: StreamModelConfig) -> Dict[str, tuple]:
        """Names and shapes of the tensors (low ranks of the delta rule: cfg.random_rank)."""
        w, n, rank = cfg.hidden_size, cfg.streams, cfg.random_rank
        out: Dict[str, tuple] = {"embed": (cfg.vocab_size, w), "final.norm": (w,)}
        for i, l in enumerate(cfg.layers):
            p, m, q = f"l{i}", l.mixer, f"l{i}.mix"
            for sub in (1, 2) if l.mlp is not None else (1,):
                out.update({f"{p}.norm{sub}": (w,), f"{p}.hc{sub}.in": (n,), f"{p}.hc{sub}.out": (n,), f"{p}.hc{sub}.mix": (n, n)})
            if isinstance(m, LatentAttentionConfig):
                out.update({q + ".dq": (m.q_rank, w), q + ".dq.norm": (m.q_rank,),
                            q + ".uq": (m.heads * (m.dim + m.rot_dim), m.q_rank), q + ".dkv": (m.kv_rank + m.rot_dim, w),
                            q + ".dkv.norm": (m.kv_rank,), q + ".uk": (m.heads * m.dim, m.kv_rank),
                            q + ".uv": (m.heads * m.vdim, m.kv_rank), q + ".sink": (m.heads,), q + ".o": (w, m.heads * m.vdim)})
            else:
                keys, values = m.kv_heads * m.dim, m.heads * m.vdim
                for s, cols in (("q", keys), ("k", keys), ("v", values)):
                    out.update({f"{q}.{s}": (cols, w), f"{q}.{s}.conv": (cols, m.taps)})
                out.update({q + ".b": (m.heads, w), q + ".A_log": (m.heads,), q + ".norm": (m.vdim,), q + ".a1": (rank, w),
                            q + ".a2": (m.heads * m.dim, rank), q + ".dt_bias": (m.heads * m.dim,), q + ".g1": (rank, w),
                            q + ".g2": (values, rank), q + ".o": (w, values)})
            f = p + ".mlp"
            if isinstance(l.mlp, MixtureConfig):
                out[f + ".router"] = (l.mlp.experts, w)
                for e in range(l.mlp.experts):
                    out.update({f"{f}.e{e}.up": (l.mlp.expert.ff, w), f"{f}.e{e}.down": (w, l.mlp.expert.ff)})
            elif l.mlp is not None:
                out.update({f + ".gate": (l.mlp.ff, w), f + ".up": (l.mlp.ff, w), f + ".down": (w, l.mlp.ff)})
        return out

    @staticmethod
    def random_tensor(name: str, shape: tuple, gen: torch.Generator, device) -> torch.Tensor:
        """Random weights of sane magnitude: projections of variance 1 / fan-in, norms near 1, streams that mostly keep what they
        hold, decays spread over short and long memories."""
        t = torch.randn(shape, generator=gen, device=device)
        if name.endswith(("norm", "norm1", "norm2")) or ".hc" in name and name.endswith(".out"):
            return 1.0 + 0.1 * t
        if ".hc" in name and name.endswith(".mix"):
            return torch.eye(shape[0], device=device) + 0.1 * t / shape[0]
        if ".hc" in name:
            return (1.0 + 0.3 * t) / shape[0]
        if name.endswith(".A_log"):
            return (1.0 + 15.0 * torch.rand(shape, generator=gen, device=device)).log()
        if name.endswith(".dt_bias"):
            return -4.0 + t
        if len(shape) == 1 or name == "embed":
            return t
        return t * shape[-1] ** -0.5

    def load(self, get, pack: bool) -> None:
        cfg, eps = self.cfg, self.cfg.norm_eps
        self.embed = get("embed").contiguous()
        layers: List[list] = []
        for i, l in enumerate(cfg.layers):
            p = f"l{i}"
            kind = LatentAttention if isinstance(l.mixer, LatentAttentionConfig) else DeltaRule
            subs = [kind(get, p + ".mix", l.mixer, eps, pack)]
            if kind is DeltaRule:
                subs[0].fused = cfg.fuse_decode_ops
            if isinstance(l.mlp, MixtureConfig):
                subs.append(MixtureOfExperts(get, p + ".mlp", l.mlp, pack))
            elif l.mlp is not None:
                subs.append(SiluMlp(get, p + ".mlp", pack))
            layers.append([(sub, StreamReader(get(f"{p}.hc{q}.in"), get(f"{p}.norm{q}")),
                            StreamWriter(get(f"{p}.hc{q}.mix"), get(f"{p}.hc{q}.out"))) for q, sub in enumerate(subs, 1)])
        self.layers = [layers[i] for i in cfg.runs]
        # behind the last sublayer the streams' sum is read
        self.last = StreamReader(torch.ones(cfg.streams, device=self.device), get("final.norm"))

    def head_rows(self, get) -> torch.Tensor:
        return self.embed

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches, attn_metadata, on_layer=None) -> torch.Tensor:
        """`on_layer(i, x)`: called with the streams' sum after the i-th layer that runs (tests)."""
        cfg, eps, dtype = self.cfg, self.cfg.norm_eps, self.cfg.dtype
        step = LatentStep(self.step_layout(attn_metadata, positions, caches.block_size))
        rows, width = input_ids.shape[0], cfg.hidden_size
        streams = torch.empty(cfg.streams, rows, width, dtype=torch.float32, device=self.device)
        start = torch.empty(rows, width, dtype=torch.float32, device=self.device)
        x = start.expand(cfg.streams, rows, width)  # (all streams begin as the same rows)
        subs = [(i, sub) for i, layer in enumerate(self.layers) for sub in layer]
        readers = [reader for _, (_, reader, _) in subs] + [self.last]
        h = amd.stream_embed(start, self.embed, input_ids, readers[0].weights, readers[0].norm, eps)
        for at, (i, (sub, _, writer)) in enumerate(subs):
            cache = caches.layers[i]
            if isinstance(sub, LatentAttention):
                y = sub(h, cache.kv, i, step, self.attn)
            elif isinstance(sub, DeltaRule):
                y = sub(h, cache, step.layout)
            else:
                y = sub(h)
            last = at + 1 == len(subs)
            h = writer(x, y if isinstance(y, SublayerOutput) else SublayerOutput(y),
                       None if last and on_layer is None else streams, readers[at + 1], eps, dtype)
            x = streams
            if on_layer is not None and (last or subs[at + 1][0] != i):
                on_layer(i, x.sum(0))
        return h

    def weight_bytes(self) -> int:
        """Bytes of the projections and of all experts (a decode step reads the experts its tokens take), once per pass."""
        n = self.head.numel() + sum(sub.numel() for layer in self.layers for sub, _, _ in layer)
        return n * torch.empty((), dtype=self.cfg.dtype).element_size()
