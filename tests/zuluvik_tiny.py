"""Tiny Zuluvik configurations for the tests, each different from the others in every size, and their model folders."""
from __future__ import annotations

import dataclasses
import os

import torch

from microllm_rocm_amd.config.zuluvik import (DifferentialAttentionConfig, ExpertConfig, LatentAttentionConfig, MoeMlpConfig,
                                              RampScalingConfig, RotaryAttentionConfig, RotationConfig, ZuluvikConfig, ZuluvikLayerConfig)
from microllm_rocm_amd.weights import write_model_folder

_TYPES = {DifferentialAttentionConfig: "attention", RotaryAttentionConfig: "attention_2", LatentAttentionConfig: "latent_attention"}


def _layer(mixer, mlp, weights_of=None):
    return ZuluvikLayerConfig(_TYPES[type(mixer)], mixer, mlp, weights_of)


def _differential(heads, kv_heads, dim, vdim, conv, diff, scale):
    return DifferentialAttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, diff=diff, scale=scale)


def _rotary(heads, kv_heads, dim, vdim, scale, base, dims, scaling=None):
    return RotaryAttentionConfig(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=RotationConfig(base, dims, scaling))


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, scaling=None):
    return LatentAttentionConfig(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale,
                                 rot=RotationConfig(base, rot_dim, scaling))


def _build(vocab, width, eps, embedding_scale, layers):
    """Layers as (mixer, mlp), or the number of the layer whose tensors this one runs with."""
    built = []
    for layer in layers:
        if isinstance(layer, int):
            built.append(dataclasses.replace(built[layer], weights_of=layer))
        else:
            built.append(_layer(*layer))
    return ZuluvikConfig(vocab=vocab, width=width, norm_eps=eps, embedding_scale=embedding_scale, layers=tuple(built))


# Every size a multiple of 16 where the MFMA kernels ask for one: maps of 8 channels over values of 16, half a head turned
# with a ramp inside it, cached rows of 48; a layer that runs again with another's tensors, one with a feed-forward and
# one without; two identity places among eight in four groups.
TINY_A = _build(211, 64, 1e-5, 3.0, (
    (_differential(4, 2, 8, 16, 4, 0.35, 0.35), MoeMlpConfig(6, 3, ExpertConfig(24, 0.6), identity=2, groups=4, keep_groups=2, scale=1.5,
                                                             shared=ExpertConfig(40, 0.4))),
    (_rotary(4, 1, 16, 16, 0.3, 1e3, 8, RampScalingConfig(4.0, 64.0, 8.0, 0.5)),
     MoeMlpConfig(5, 2, ExpertConfig(16, 1.1), identity=1, groups=2, keep_groups=1, scale=0.7, shared=ExpertConfig(24, 0.9))),
    (_latent(4, 16, 8, 12, 40, 0.2, 1e4, RampScalingConfig(2.0, 32.0, 4.0, 1.0)), None),
    0, 2))
# A width that is no multiple of 8; heads of odd sizes (padded in the MFMA kernels' pages, plain pages in float32), as many
# key/value heads as heads; one tap (nothing kept); a whole head turned at plain rates; latent rows of 42 (plain pages in
# either format); no identity place, no groups, one expert a token, no shared expert; a chain of borrowed tensors.
TINY_B = _build(97, 50, 1e-6, 1.0, (
    (_differential(3, 3, 6, 10, 1, 0.8, 0.4), MoeMlpConfig(5, 1, ExpertConfig(20, 0.5), scale=1.0)),
    (_rotary(6, 3, 10, 14, 0.4, 50.0, 10), None),
    (_latent(3, 10, 6, 14, 36, 0.25, 300.0, RampScalingConfig(16.0, 40.0, 2.0, 0.1)), MoeMlpConfig(4, 4, ExpertConfig(12, 2.0), identity=2, groups=3, keep_groups=2,
                                                                                             scale=2.0, shared=ExpertConfig(28, 0.3))),
    1, 3, 0))
# Values wider than both maps' keys and the reverse; two taps; latent rows of 256 (the widest the MFMA kernels take);
# sixteen experts of 64 channels and four identity places in five groups, six a token (in bfloat16 prompts the experts' tiled products).
TINY_C = _build(150, 96, 1e-6, 0.5, (
    (_rotary(6, 2, 32, 64, 0.18, 500.0, 20, RampScalingConfig(8.0, 100.0, 16.0, 1.0)),
     MoeMlpConfig(16, 6, ExpertConfig(64, 0.8), identity=4, groups=5, keep_groups=3, scale=1.2, shared=ExpertConfig(32, 0.7))),
    (_differential(6, 2, 16, 40, 2, 0.2, 0.25), None),
    (_latent(5, 24, 32, 40, 224, 0.15, 1e4, RampScalingConfig(3.0, 256.0, 24.0, 1.5)),
     MoeMlpConfig(7, 3, ExpertConfig(48, 1.0), identity=5, groups=4, keep_groups=4, scale=0.5, shared=ExpertConfig(16, 1.0))),
    (_differential(2, 1, 40, 24, 7, 0.5, 0.2), MoeMlpConfig(3, 2, ExpertConfig(16, 0.2), identity=1, groups=2, keep_groups=2, scale=1.0,
                                                           shared=ExpertConfig(8, 5.0))),
    1))

CONFIGS = {"A": TINY_A, "B": TINY_B, "C": TINY_C}
SEEDS = {"A": 61, "B": 62, "C": 63}
STDS = {"std": 0.1, "norm_std": 0.15, "conv_std": 0.5}


def without_choice(config: ZuluvikConfig) -> ZuluvikConfig:
    """The same model with every token sent to all of its places, weighted by their scores. Which places a token takes is a
    step function of the router's scores: an engine that rounds to bfloat16 takes another one than the plain run wherever two
    lie within the rounding of each other, and what such a token then caches moves every later position. The bfloat16
    engine is therefore held against the plain run on these models, where the sum is continuous; the choice itself is
    held in float32."""
    layers = tuple(dataclasses.replace(layer, mlp=dataclasses.replace(layer.mlp, top=layer.mlp.places, groups=1, keep_groups=1))
                   if layer.mlp is not None else layer for layer in config.layers)
    return dataclasses.replace(config, layers=layers)


def make_zuluvik_folder(tmp_path, which: str, choice: bool = True) -> str:
    folder = os.path.join(str(tmp_path), f"zuluvik_{which}" + ("" if choice else "_all"))
    write_model_folder(folder, CONFIGS[which] if choice else without_choice(CONFIGS[which]), SEEDS[which], dtype=torch.bfloat16, stds=STDS)
    return folder
