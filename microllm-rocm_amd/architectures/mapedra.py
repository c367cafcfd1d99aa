"""The Mapedra decoder as a ``ModelSpec``.

Token embedding times a factor; layers whose sublayers read the stream as it is and pass a norm in groups before they
join it (the ``sandwich_norm`` arrangement with nothing before and a factor of one); per layer one of two mixers: lightning
attention (linear attention with one fixed decay a head, SiLU on queries, keys and values, one norm over all heads, a
sigmoid gate), or a causal softmax attention (grouped key/value heads, norms of queries, keys and values, neighbouring
channels of part of the head turned together at rates stretched by bands, capped scores, a gate a channel); a dense
feed-forward gated by the tanh form of gelu, or none; after it a vector of the token's own from a side table, gated by the
stream, through a plain RMS norm; a final norm in groups and an untied head.

Tensor names: ``embed``, ``side.embed`` (``[vocab, layers * dim]``), ``head``, ``final.norm``; per layer ``l<i>.norm1``,
``l<i>.norm2`` (after the mixer and the feed-forward), ``l<i>.mix.*``, ``l<i>.mlp.{gate,up,down}``,
``l<i>.side.{gate,proj,norm}``.
"""
from __future__ import annotations

from ..config.mapedra import AttentionConfig, LightningConfig, MapedraConfig
from ..config.registry import Architecture, register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, in_order
from ..weights.random_init import InitRule

MAX_POSITIONS = 1 << 20     # no part has a longest position; block tables and requests need a bound
GATE_ACTIVATION = "gelu_tanh"   # of the feed-forward


def _attention_spec(width: int, prefix: str, mixer: AttentionConfig, eps: float) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("q", "k", "v", "g", "o")}
    names.update({"q_norm": f"{prefix}.q.norm", "k_norm": f"{prefix}.k.norm"})
    bands = mixer.rot_scaling
    position = PartSpec("rope_neighbours", {"theta": mixer.rot_base, "head_dim": mixer.dim, "rotary_dim": mixer.rot_dims,
                                            "scaling_bands": bands.to_dict() if bands is not None else None})
    return PartSpec("bucket_bias_attention", {
        "hidden_size": width, "heads": mixer.heads, "kv_heads": mixer.kv_heads, "key_dim": mixer.dim, "value_dim": mixer.vdim,
        "scale": mixer.scale, "qk_norm": True, "qk_norm_weight": True, "value_norm": True, "eps": eps, "sink": False,
        "softcap": mixer.softcap, "channel_gate": True, "position": position}, names)


def _lightning_spec(width: int, prefix: str, mixer: LightningConfig, eps: float) -> PartSpec:
    names = {role: f"{prefix}.{role}" for role in ("q", "k", "v", "g", "o", "norm")}
    return PartSpec("gated_linear_attention", {
        "hidden_size": width, "heads": mixer.heads, "key_dim": mixer.dim, "value_dim": mixer.vdim, "fixed_decay": list(mixer.decay),
        "silu_inputs": True, "heads_together": True, "chunked": True, "eps": eps, "query_scale": 1.0}, names)


def build_spec(config: MapedraConfig) -> ModelSpec:
    width, eps = config.width, config.norm_eps
    grouped = {"size": width, "eps": eps, "groups": config.norm_groups}
    nothing = PartSpec("unnormed")
    sizes = {"vocab_size": config.vocab, "hidden_size": width}
    layers = []
    for index, layer in enumerate(config.layers):
        prefix = f"l{index}"
        build = _attention_spec if isinstance(layer.mixer, AttentionConfig) else _lightning_spec
        extra = {
            "mixer_after": ("norm", PartSpec("rms_norm", grouped, {"weight": f"{prefix}.norm1"})),
            "side": ("ffn", PartSpec("token_side_input", {**sizes, "dim": config.side_dim, "column_at": index * config.side_dim,
                                                          "table_columns": len(config.layers) * config.side_dim},
                                     {"table": "side.embed", "gate": f"{prefix}.side.gate", "proj": f"{prefix}.side.proj"})),
            "side_norm": ("norm", nothing),
            "side_after": ("norm", PartSpec("rms_norm", {"size": width, "eps": eps}, {"weight": f"{prefix}.side.norm"})),
        }
        ffn = None
        if layer.mlp is not None:
            ffn = PartSpec("swiglu", {"hidden_size": width, "intermediate_size": layer.mlp.ff, "activation": GATE_ACTIVATION},
                           {f"{role}_proj.weight": f"{prefix}.mlp.{role}" for role in ("gate", "up", "down")})
            extra["ffn_after"] = ("norm", PartSpec("rms_norm", grouped, {"weight": f"{prefix}.norm2"}))
        layers.append(LayerSpec(arrangement="sandwich_norm", mixer_norm=nothing, mixer=build(width, f"{prefix}.mix", layer.mixer, eps),
                                ffn_norm=nothing if ffn is not None else None, ffn=ffn, extra=extra, params={"residual_mult": 1.0}))
    return ModelSpec(
        architecture=config.architecture, vocab_size=config.vocab, hidden_size=width, max_positions=MAX_POSITIONS,
        embedding=PartSpec("token_embedding", {**sizes, "scale": config.embedding_scale}, {"weight": "embed"}),
        layers=tuple(layers), order=in_order(len(layers)),
        final_norm=PartSpec("rms_norm", grouped, {"weight": "final.norm"}),
        head=PartSpec("lm_head", sizes, {"weight": "head"}))


def init_rules(config: MapedraConfig):
    """Random weights: norm weights around one; every matrix and table ~ N(0, std)."""
    return [
        InitRule(suffix="norm", mean=1.0, std_key="norm_std"),
        InitRule(suffix="norm1", mean=1.0, std_key="norm_std"),
        InitRule(suffix="norm2", mean=1.0, std_key="norm_std"),
        InitRule(suffix="", mean=0.0, std_key="std"),
    ]


register_architecture(Architecture(
    name="Mapedra",
    config_from_dict=MapedraConfig.from_dict,
    build_spec=build_spec,
    init_rules=init_rules,
))
