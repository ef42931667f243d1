"""Attention backend of hybrid decoders: the paged metadata of `PagedAttnBackend`, caches whose key and value rows differ
in size, and one entry that serves prompts, portions of prompts and single decoded tokens alike (every sequence of a step
is a chunk that ends its context).

A layer's cache is one buffer [num_blocks, keys | values (| padding)], so that block copies and swaps move a block of a
layer as one run; `split_kv_cache` gives the two views the kernels take."""
from typing import List, Tuple, Type

import torch

from .. import _custom_ops as ops
from .backend import PagedAttnBackend


class HeadAttnImpl:
    """Stateless: sizes come with the cache views, constants with the call."""

    @staticmethod
    def split_kv_cache(kv_cache: torch.Tensor, spec, block_size: int) -> Tuple[torch.Tensor, torch.Tensor]:
        n = kv_cache.shape[0]
        x = 16 // kv_cache.element_size()
        stride, off = kv_cache.stride(0), spec.kv_heads * spec.kpad * block_size
        k = kv_cache.as_strided((n, spec.kv_heads, spec.kpad // x, block_size, x),
                                (stride, spec.kpad * block_size, block_size * x, x, 1), kv_cache.storage_offset())
        v = kv_cache.as_strided((n, spec.kv_heads, spec.vpad, block_size),
                                (stride, spec.vpad * block_size, block_size, 1), kv_cache.storage_offset() + off)
        return k, v


class HeadAttnBackend(PagedAttnBackend):

    @staticmethod
    def get_name() -> str:
        return "head-attn-hip"

    @staticmethod
    def get_impl_cls() -> Type[HeadAttnImpl]:
        return HeadAttnImpl

    @staticmethod
    def swap_blocks(src_kv_cache: torch.Tensor, dst_kv_cache: torch.Tensor, src_to_dst: torch.Tensor) -> None:
        ops.swap_blocks(src_kv_cache, dst_kv_cache, src_to_dst)

    @staticmethod
    def copy_blocks(kv_caches: List[torch.Tensor], src_to_dists: torch.Tensor) -> None:
        """Layers of one block size go to the kernel in pairs, as its two planes (an odd one out is both: the same bytes
        are written twice)."""
        by_stride = {}
        for c in kv_caches:
            by_stride.setdefault(c.stride(0), []).append(c)
        for group in by_stride.values():
            first, second = group[0::2], group[1::2]
            if len(second) < len(first):
                second = second + [first[-1]]
            if src_to_dists.device != group[0].device:
                src_to_dists = src_to_dists.to(group[0].device, non_blocking=True)
            ops.copy_blocks(first, second, src_to_dists)
