"""The Zuluvik decoder as a ``ModelSpec``.

Token embedding times a factor; layers whose mixer and feed-forward read one norm of the stream and join it together (the
``parallel_sublayers`` arrangement); per layer one of three mixers: a differential attention (two maps a head over the same
values, a short convolution over time on queries, keys and values, no rotation), a causal attention with biases whose
queries and keys are turned (neighbouring channels together, rates stretched along a ramp) and then normed without a
weight, or an attention through cached latents (queries straight from the input, a rotated key part shared by all heads,
the same rotation, no gate); a mixture of experts with clamped gates (softmax scores, a correction of the choice, groups of
places of which only the best can be chosen, places that return their input, a shared expert) or none; a final norm and an
untied head. A layer may run with another's tensors on a cache of its own: it is one more entry of the run order.

Tensor names: ``embed``, ``head``, ``final.norm``; per layer with tensors of its own ``l<i>.norm1``, ``l<i>.mix.*`` (a bias is
its weight's name with ``.b``, a convolution's taps its projection's name with ``.conv``) and
``l<i>.mlp.{router,correction,e<n>.gate,e<n>.up,e<n>.down,shared.gate,shared.up,shared.down}``.
"""
from __future__ import annotations

from ..config.registry import Architecture, register_architecture
from ..config.zuluvik import (DifferentialAttentionConfig, LatentAttentionConfig, MoeMlpConfig, RotaryAttentionConfig, RotationConfig,
                              ZuluvikConfig)
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from ..weights.random_init import InitRule

MAX_POSITIONS = 1 << 20     # no part has a longest position; block tables and requests need a bound
GATE_SLOPE = 1.702          # of the experts' sigmoid
WEIGHT_EPS = 1e-20          # added to the sum that the chosen experts' scores are divided by
MAGNITUDE_SLOPE = 0.1       # stretched rotations multiply what they turn by this times ln(factor), plus one


def _position_spec(head_dim: int, rot: RotationConfig) -> PartSpec:
    ramp = {**rot.scaling.to_dict(), "magnitude_slope": MAGNITUDE_SLOPE} if rot.scaling is not None else None
    return PartSpec("rope_neighbours", {"theta": rot.base, "head_dim": head_dim, "rotary_dim": rot.dims, "scaling_ramp": ramp})


def _differential_spec(width: int, prefix: str, mixer: DifferentialAttentionConfig, eps: float) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("q", "k", "v", "o", "lq1", "lk1", "lq2", "lk2")}
    names.update({f"{role}_conv": f"{prefix}.{role}.conv" for role in ("q", "k", "v")})
    return PartSpec("differential_attention", {
        "hidden_size": width, "heads": mixer.heads, "kv_heads": mixer.kv_heads, "dim": mixer.dim, "value_dim": mixer.vdim,
        "scale": mixer.scale, "conv": mixer.conv, "difference": mixer.diff, "eps": eps}, names)


def _rotary_spec(width: int, prefix: str, mixer: RotaryAttentionConfig, eps: float) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("q", "k", "v", "o")}
    names.update({f"{role}_bias": f"{prefix}.{role}.b" for role in ("q", "k", "v")})
    return PartSpec("bucket_bias_attention", {
        "hidden_size": width, "heads": mixer.heads, "kv_heads": mixer.kv_heads, "key_dim": mixer.dim, "value_dim": mixer.vdim,
        "scale": mixer.scale, "qk_norm": True, "qk_norm_weight": False, "norm_turned": True, "eps": eps, "sink": False,
        "projection_bias": True, "output_bias": False, "pad_heads": True, "position": _position_spec(mixer.dim, mixer.rot)}, names)


def _latent_spec(width: int, prefix: str, mixer: LatentAttentionConfig, eps: float) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("q", "dkv", "uk", "uv", "o")}
    names["dkv_norm"] = f"{prefix}.dkv.norm"
    return PartSpec("latent_attention", {
        "hidden_size": width, "heads": mixer.heads, "dim": mixer.dim, "rot_dim": mixer.rot_dim, "vdim": mixer.vdim,
        "q_rank": None, "kv_rank": mixer.kv_rank, "scale": mixer.scale, "window": None, "eps": eps,
        "owns_kv": True, "output_gate": False, "position": _position_spec(mixer.rot_dim, mixer.rot)}, names)


def _mixer_spec(width: int, prefix: str, mixer, eps: float) -> PartSpec:
    if isinstance(mixer, DifferentialAttentionConfig):
        return _differential_spec(width, prefix, mixer, eps)
    if isinstance(mixer, RotaryAttentionConfig):
        return _rotary_spec(width, prefix, mixer, eps)
    assert isinstance(mixer, LatentAttentionConfig)
    return _latent_spec(width, prefix, mixer, eps)


def _moe_spec(width: int, prefix: str, mlp: MoeMlpConfig) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("router", "correction")}
    for expert in range(mlp.experts):
        names.update({f"expert{expert}.{role}": f"{prefix}.e{expert}.{role}" for role in ("gate", "up", "down")})
    if mlp.shared is not None:
        names.update({f"shared.{role}": f"{prefix}.shared.{role}" for role in ("gate", "up", "down")})
    return PartSpec("routed_experts", {
        "hidden_size": width, "experts": mlp.experts, "identity": mlp.identity, "top": mlp.top, "expert_size": mlp.expert.ff,
        "shared_size": mlp.shared.ff if mlp.shared is not None else None, "score": "softmax", "correction": True,
        "renormalize": True, "weight_eps": WEIGHT_EPS, "weight_scale": mlp.scale, "weight_on": "output",
        "activation": "clamped_glu", "limit": mlp.expert.limit, "shared_limit": mlp.shared.limit if mlp.shared is not None else None,
        "slope": GATE_SLOPE, "groups": mlp.groups if mlp.groups > 1 else 0, "keep_groups": mlp.keep_groups if mlp.groups > 1 else 0}, names)


def build_spec(config: ZuluvikConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps
    norm = {"size": width, "eps": eps}
    layers, place_of = [], {}       # place_of: a layer with tensors of its own -> where its spec stands
    for index, layer in enumerate(config.layers):
        if layer.weights_of is not None:
            continue
        prefix = f"l{index}"
        place_of[index] = len(layers)
        layers.append(LayerSpec(
            arrangement="parallel_sublayers", mixer_norm=PartSpec("rms_norm", norm, {"weight": f"{prefix}.norm1"}),
            mixer=_mixer_spec(width, f"{prefix}.mix", layer.mixer, eps),
            ffn=_moe_spec(width, f"{prefix}.mlp", layer.mlp) if layer.mlp is not None else None))
    order = tuple(RunEntry(layer=place_of[config.owner_of(index)]) for index in range(len(config.layers)))
    sizes = {"vocab_size": config.vocab, "hidden_size": width}
    return ModelSpec(
        architecture=config.architecture, vocab_size=config.vocab, hidden_size=width, max_positions=MAX_POSITIONS,
        embedding=PartSpec("token_embedding", {**sizes, "scale": config.embedding_scale}, {"weight": "embed"}),
        layers=tuple(layers), order=order,
        final_norm=PartSpec("rms_norm", norm, {"weight": "final.norm"}),
        head=PartSpec("lm_head", sizes, {"weight": "head"}))


def init_rules(config: ZuluvikConfig):
    """Random weights: norm weights around one; convolutions' taps ~ N(0, conv_std); everything else ~ N(0, std)."""
    return [
        InitRule(suffix="norm", mean=1.0, std_key="norm_std"),
        InitRule(suffix="norm1", mean=1.0, std_key="norm_std"),
        InitRule(suffix=".conv", mean=0.0, std_key="conv_std"),
        InitRule(suffix="", mean=0.0, std_key="std"),
    ]


register_architecture(Architecture(
    name="Zuluvik",
    config_from_dict=ZuluvikConfig.from_dict,
    build_spec=build_spec,
    init_rules=init_rules,
))
