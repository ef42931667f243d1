"""What decoders of listed layers share: where their weights come from, the layout of a step, the head."""
from typing import Callable, Dict, Optional

import torch

from .mixers import StepLayout
from .model import Weight, linear
from .weights import load_checkpoint


class LayeredModel:
    """forward(input_ids, positions, caches, attn_metadata) -> normed hidden states [rows, width].

    A subclass names its tensors (`tensor_shapes(cfg)`) and their random stand-ins (`random_tensor`)."""

    def __init__(self, cfg, attn_impl, device="cuda:0", seed: int = 0, tensors=None):
        """Weights come from `tensors` (name -> tensor), else from cfg.weights_dir, else from the seed."""
        self.cfg, self.device, self.attn = cfg, torch.device(device), attn_impl
        if tensors is None and cfg.weights_dir is not None:
            tensors = load_checkpoint(cfg.weights_dir)
        if tensors is None:
            gen, shapes = torch.Generator(device=self.device).manual_seed(seed), self.tensor_shapes(cfg)

            def get(name):
                return self.random_tensor(name, shapes[name], gen, self.device).to(cfg.dtype)
        else:
            def get(name):
                return tensors[name].to(self.device).to(cfg.dtype)
        pack = cfg.pack_weights and self.device.type == "cuda"
        self.load(get, pack)
        self.head = Weight(self.head_rows(get).contiguous(), pack and cfg.dtype != torch.float32)

    @staticmethod
    def tensor_shapes(cfg) -> Dict[str, tuple]:
        raise NotImplementedError

    @staticmethod
    def random_tensor(name: str, shape: tuple, gen: torch.Generator, device) -> torch.Tensor:
        raise NotImplementedError

    def load(self, get: Callable[[str], torch.Tensor], pack: bool) -> None:
        """Everything but the head."""
        raise NotImplementedError

    def head_rows(self, get: Callable[[str], torch.Tensor]) -> torch.Tensor:
        """[vocab, width]"""
        return get("head")

    def step_layout(self, md, positions: torch.Tensor, block_size: int, unified: Optional[tuple] = None) -> StepLayout:
        """`unified`: the device tensors of a captured mixed step (graph_runner.MixedGraph) in place of metadata."""
        if unified is not None:
            tables, seq_lens, query_start_loc, max_query_len, slot_mapping = unified
            return StepLayout(query_start_loc, seq_lens, tables, slot_mapping, None, max_query_len,
                              tables.shape[1] * block_size, block_size, positions)
        return StepLayout(md.query_start_loc, md.seq_lens_tensor, md.block_tables, md.slot_mapping, md.state_slots,
                          md.max_query_len or 1, max(md.max_prefill_seq_len or 0, md.max_decode_seq_len or 0), block_size,
                          positions, md.query_lens, md.context_lens)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return linear(hidden, self.head)

    def greedy_tokens(self, hidden: torch.Tensor) -> torch.Tensor:
        w = self.head
        if 0 < hidden.shape[0] <= 64 and w.packed is not None:
            return torch.ops._C_amd.skinny_linear_packed_argmax(hidden, w.packed, w.N, w.K)
        return torch.argmax(self.compute_logits(hidden), dim=-1)
