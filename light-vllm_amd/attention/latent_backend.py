"""Attention backend of latent decoders: the paged metadata and block movement of `HeadAttnBackend`, over caches of one row
per token (engine/latent_config.LatentKVSpec)."""
from typing import Type

import torch

from .head_backend import HeadAttnBackend, HeadAttnImpl


class LatentAttnImpl(HeadAttnImpl):

    @staticmethod
    def rows_view(kv_cache: torch.Tensor, spec, block_size: int) -> torch.Tensor:
        """[blocks, block_size, row], blocks as far apart as the allocation has them."""
        return kv_cache.as_strided((kv_cache.shape[0], block_size, spec.row), (kv_cache.stride(0), spec.row, 1),
                                   kv_cache.storage_offset())


class LatentAttnBackend(HeadAttnBackend):

    @staticmethod
    def get_name() -> str:
        return "latent-attn-hip"

    @staticmethod
    def get_impl_cls() -> Type[LatentAttnImpl]:
        return LatentAttnImpl
