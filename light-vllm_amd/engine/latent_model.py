"""Decoder of latent-attention layers (engine/latent_config.py): scaled embedding -> layers -> norm -> head, over the engine's
paged caches.  Serves prompts, portions of prompts and decoded tokens in one batch; every tensor that steers a step of
single tokens is on the device, so decode steps (and small mixed ones) are captured as they are."""
from typing import Dict, List

import torch

from .latent_config import LatentModelConfig
from .latent_layers import LatentAttention, LatentStep, MixtureOfExperts, OutputNorm
from .layered_model import LayeredModel

amd = torch.ops._C_amd


class LatentModel(LayeredModel):

    @staticmethod
    def tensor_shapes(cfg: LatentModelConfig) -> Dict[str, tuple]:
        w = cfg.hidden_size
        out: Dict[str, tuple] = {"embed": (cfg.vocab_size, w), "head": (cfg.vocab_size, w), "final.norm": ()}
        for i, l in enumerate(cfg.layers):
            p, m = f"l{i}", l.mixer
            out.update({p + ".norm1": (), p + ".dwa": (i + 2,),
                        p + ".mix.q": (m.heads * (m.dim + m.rot_dim), w), p + ".mix.uk": (m.heads * m.dim, m.kv_rank),
                        p + ".mix.uv": (m.heads * m.vdim, m.kv_rank), p + ".mix.g": (m.heads, w),
                        p + ".mix.o": (w, m.heads * m.vdim)})
            if m.kv_from is None:
                out.update({p + ".mix.dkv": (m.kv_rank + m.rot_dim, w), p + ".mix.dkv.norm": (m.kv_rank,)})
            if l.mlp is None:
                continue
            q = p + ".mlp"
            out.update({p + ".norm2": (), q + ".router": (l.mlp.experts, w), q + ".router.b": (l.mlp.experts,)})
            experts = [(f"{q}.e{e}", l.mlp.expert.ff) for e in range(l.mlp.experts)]
            if l.mlp.shared is not None:
                experts.append((q + ".shared", l.mlp.shared.ff))
                out[q + ".shared.sg"] = (1, w)
            for e, ff in experts:
                out.update({e + ".gate": (ff, w), e + ".up": (ff, w), e + ".down": (w, ff)})
        return out

    @staticmethod
    def random_tensor(name: str, shape: tuple, gen: torch.Generator, device) -> torch.Tensor:
        """Random weights of sane magnitude: projections of variance 1 / fan-in, gains near 1, depth averages that keep most
        of the last stream."""
        t = torch.randn(shape, generator=gen, device=device)
        if name.endswith(".dwa"):
            t = 0.1 * t / shape[0]
            t[-1] += 1.0
            return t
        if name.endswith(("norm", "norm1", "norm2")):
            return 1.0 + 0.1 * t
        if name.endswith(".router.b"):
            return 0.1 * t
        if name == "embed":
            return t
        return t * shape[-1] ** -0.5

    def load(self, get, pack: bool) -> None:
        cfg = self.cfg
        self.embed = get("embed").contiguous()
        self.layers: List[tuple] = []
        for i, l in enumerate(cfg.layers):
            p = f"l{i}"
            mixer = LatentAttention(get, p + ".mix", l.mixer, cfg.norm_eps, pack)
            ff = None
            if l.mlp is not None:
                ff = OutputNorm(get, p + ".norm2", cfg.norm_eps), MixtureOfExperts(get, p + ".mlp", l.mlp, pack)
            self.layers.append((OutputNorm(get, p + ".norm1", cfg.norm_eps), mixer, ff, get(p + ".dwa").float().contiguous()))
        self.final_norm = OutputNorm(get, "final.norm", cfg.norm_eps)

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, caches, attn_metadata, unified=None,
                on_layer=None) -> torch.Tensor:
        """`on_layer(i, x)`: called with what leaves every layer (tests)."""
        cfg, dtype, rows = self.cfg, self.cfg.dtype, input_ids.shape[0]
        step = LatentStep(self.step_layout(attn_metadata, positions, caches.block_size, unified))
        # the embedding and every layer's result, which all later layers' averages read
        streams = torch.empty(len(self.layers) + 1, rows, cfg.hidden_size, dtype=torch.float32, device=self.device)
        x, running = streams[0], torch.empty(rows, cfg.hidden_size, dtype=torch.float32, device=self.device)
        h = amd.embed_scale(x, self.embed, input_ids, cfg.embedding_scale)
        for i, (norm1, mixer, ff, depth) in enumerate(self.layers):
            source = cfg.kv_layer(i)
            last = i + 1 == len(self.layers)
            after = dict(x_out=None if last and on_layer is None else running, v_out=None if last else streams[i + 1],
                         streams=streams[:i + 1], depth=depth, final=self.final_norm if last else None)
            y = mixer(h, caches.layers[source].kv, source, step, self.attn)
            if ff is not None:
                norm2, mixture = ff
                h = norm1(y, x, dtype, x_out=running)
                x, norm1, y = running, norm2, mixture(h)
            h = norm1(y, x, dtype, **after)
            x = running
            if on_layer is not None:
                on_layer(i, x.clone())
        return h

    def weight_bytes(self) -> int:
        """Bytes of the projections and of all experts (a decode step reads the experts its tokens take)."""
        n = self.head.numel()
        for _, mixer, ff, _ in self.layers:
            n += mixer.numel()
            if ff is not None:
                n += ff[1].numel()
        return n * torch.empty((), dtype=self.cfg.dtype).element_size()

