"""Tiny Mapedra configurations for the tests, each different from the others in every size, and their model folders."""
from __future__ import annotations

import os

import torch

from microllm_rocm_amd.config.mapedra import (AttentionConfig, BandScalingConfig, DenseMlpConfig, LightningConfig, MapedraConfig,
                                              MapedraLayerConfig)
from microllm_rocm_amd.weights import write_model_folder


def _attention(heads, kv_heads, dim, vdim, scale, rot_dims, softcap, base=10000.0, bands=None):
    return AttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot_base=base, rot_dims=rot_dims,
                           softcap=softcap, rot_scaling=BandScalingConfig(*bands) if bands is not None else None)


def _lightning(dim, vdim, decay):
    return LightningConfig(heads=len(decay), dim=dim, vdim=vdim, decay=tuple(decay))


def _layer(mixer, ff):
    kind = "attention" if isinstance(mixer, AttentionConfig) else "lightning"
    return MapedraLayerConfig(kind, mixer, DenseMlpConfig(ff) if ff else None)


# Attention first (heads of 16: the MFMA kernels in bfloat16, half a head turned, rates in all three bands, a tight cap),
# lightning of three heads with a feed-forward, attention of equal head counts and of unequal key and value sizes (plain
# pages) without a feed-forward, whole heads turned; norms in four parts.
TINY_A = MapedraConfig(
    vocab=211, width=64, norm_eps=1e-5, norm_groups=4, side_dim=8, embedding_scale=3.0,
    layers=(
        _layer(_attention(4, 2, 16, 16, 0.3, 8, 4.0, bands=(3.0, 1.0, 8.0, 64.0)), 96),
        _layer(_lightning(12, 10, [0.9, 0.5, 0.99]), 40),
        _layer(_attention(6, 6, 10, 6, 0.4, 10, 9.0, base=77.0), None),
        _layer(_attention(4, 1, 32, 32, 0.2, 16, 20.0, base=500.0, bands=(8.0, 2.0, 3.0, 100.0)), 72),
    ))
# A width that is no multiple of 8, norms in one part, an odd side size; two lightning layers without a feed-forward (a
# head that forgets nothing, one that keeps the token alone; a single head whose keys are wider than its values); three query
# heads on one key/value head, no cap and no stretched rates.
TINY_B = MapedraConfig(
    vocab=97, width=50, norm_eps=1e-6, norm_groups=1, side_dim=7, embedding_scale=1.0,
    layers=(
        _layer(_lightning(8, 12, [1.0, 0.0, 0.7, 0.97, 0.85]), None),
        _layer(_attention(3, 1, 48, 48, 0.15, 48, None), 60),
        _layer(_lightning(40, 7, [0.998]), None),
        _layer(_attention(2, 2, 14, 20, 0.3, 4, 2.5, base=100.0, bands=(2.0, 0.5, 0.5, 40.0)), 33),
    ))
# Norms in parts of six channels (no multiple of four), a side vector as wide as the model, a large factor on the
# embedding, eps that matters; heads of 112 (an odd number of tiles of 16) with 64 turned; a lightning layer last.
TINY_C = MapedraConfig(
    vocab=150, width=96, norm_eps=1e-3, norm_groups=16, side_dim=96, embedding_scale=12.0,
    layers=(
        _layer(_lightning(16, 24, [0.75, 0.95]), 128),
        _layer(_attention(8, 2, 112, 112, 0.1, 64, 15.0, base=3e5, bands=(5.0, 1.0, 6.0, 512.0)), 160),
        _layer(_attention(2, 1, 24, 40, 0.3, 24, 6.0), 16),
        _layer(_lightning(5, 32, [0.9375, 0.875, 0.6, 0.999, 0.3, 0.98, 0.2]), None),
    ))

CONFIGS = {"A": TINY_A, "B": TINY_B, "C": TINY_C}
SEEDS = {"A": 61, "B": 62, "C": 63}
STDS = {"std": 0.1, "norm_std": 0.15}


def make_mapedra_folder(tmp_path, which: str) -> str:
    folder = os.path.join(str(tmp_path), f"mapedra_{which}")
    write_model_folder(folder, CONFIGS[which], SEEDS[which], dtype=torch.bfloat16, stds=STDS)
    return folder
