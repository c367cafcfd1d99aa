"""A plain, slow implementation of the Zuluvik decoder on the CPU, one function per mechanism.

It shares no code with the engine: it takes the configuration as the dictionary that config.json holds and the
tensors by their file names, and computes every sequence whole, in float64.

Notation. ``x`` is the residual stream ``[T, width]``, at the start ``E[ids] * embedding.scale``; ``rms(a) = a /
sqrt(mean(a^2) + eps)`` over the last axis. A layer reads the stream once: with ``a = rms(x) * w1``,

    x += M(a) + F(a)        (F absent where the layer has no feed-forward)

and a layer that names ``weights_of`` runs with that layer's tensors on keys, values and inputs of its own. The mixers ``M``:

* ``attention``: ``u = W a`` for q, k and v, each channel convolved over time, ``y_t = sum_j c[j] u_(t - taps + 1 + j)``
  with ``u = 0`` before the start. Query head ``h`` and key head ``g = h // (H / G)`` are pairs of vectors ``(q1, q2)``,
  ``(k1, k2)``; ``a_m = softmax(scale * q_m . k_m) v_g`` over ``j <= i``; with ``l = exp(lq1 . lk1) - exp(lq2 . lk2) +
  diff`` the head gives ``(1 - diff) * rms(a_1 - l a_2)``; ``Wo``.
* ``attention_2``: q, k, v with biases; of q's and k's heads the first ``rot.dims`` dimensions turn (``2i`` with ``2i + 1``)
  by ``p f_i``, the turned values times ``m`` (``f`` and ``m`` from ``yarn``); then ``rms`` over the head; softmax of ``scale *
  q . k`` over ``j <= i``; ``Wo``.
* ``latent_attention``: ``q = Wq a`` head by head as ``[dim | rot_dim]``; ``Wdkv a`` gives the latent ``c`` (``kv_rank``
  numbers, ``rms`` times a weight) and one key part ``r`` for all heads, turned and scaled as above like q's second part;
  head ``h`` has keys ``[Wuk_h c | r]`` and values ``Wuv_h c``; softmax of ``scale * q . k``; ``Wo``.

``F`` sends every token through ``top`` experts. ``s = softmax(z)`` over the experts and, after them, ``identity`` places
that return their input; ``s + correction`` decides: the ``groups.keep`` groups with the largest members, in them the
``top`` largest. The weights are the chosen ``s`` over their sum (+ 1e-20), times ``router.scale``. An expert is
``Wd (g sigmoid(1.702 g) (u + 1))`` with ``g = min(Wg a, limit)`` and ``u = clamp(Wu a, -limit, limit)``; a shared one of
the same form, with a limit of its own, is added.
"""
from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional, Tuple

import torch

F = torch.float64


def t64(tensors: Mapping[str, torch.Tensor], name: str) -> torch.Tensor:
    return tensors[name].to(F)


def rms(a: torch.Tensor, eps: float) -> torch.Tensor:
    return a / torch.sqrt((a * a).mean(-1, keepdim=True) + eps)


def yarn(base: float, n: int, scaling: Optional[Mapping] = None) -> Tuple[List[float], float]:
    """The angle a position of each of the ``n / 2`` pairs, and the factor on what is turned. A pair that turns often over
    the original length keeps its rate, one that turns seldom has it divided by the factor, and along the ramp between
    them (in the pair's number) the two are blended."""
    plain = [base ** (-2.0 * i / n) for i in range(n // 2)]
    if scaling is None:
        return plain, 1.0
    factor, original = scaling["factor"], scaling["original"]

    def pair_turning(times: float) -> float:
        return n * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(base))

    low = max(math.floor(pair_turning(scaling["fast"])), 0)
    high = min(math.ceil(pair_turning(scaling["slow"])), n - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def turn_neighbours(a: torch.Tensor, positions: torch.Tensor, rot: Mapping) -> torch.Tensor:
    """``a`` is ``[T, ..., D]``; of its first ``rot.dims`` dims ``2i`` and ``2i + 1`` are turned together and multiplied by
    yarn's factor; the rest pass."""
    n = rot["dims"]
    rates, factor = yarn(rot["base"], n, rot.get("scaling"))
    angle = positions.to(torch.float64)[:, None] * torch.tensor(rates, dtype=torch.float64)[None, :]
    shape = [a.shape[0]] + [1] * (a.dim() - 2) + [n // 2]
    cos, sin = (torch.cos(angle) * factor).to(F).view(shape), (torch.sin(angle) * factor).to(F).view(shape)
    u, v = a[..., 0:n:2], a[..., 1:n:2]
    out = a.clone()
    out[..., 0:n:2] = u * cos - v * sin
    out[..., 1:n:2] = v * cos + u * sin
    return out


def convolve(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``u`` ``[T, C]``, ``taps`` ``[C, n]``: channel by channel, the last tap on the token itself, zeros before the first."""
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, u.shape[1], dtype=u.dtype), u])
    out = torch.zeros_like(u)
    for j in range(n):
        out += taps[:, j] * padded[j:j + u.shape[0]]
    return out


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """``q`` ``[T, H, d]``, ``k`` ``[T, G, d]``, ``v`` ``[T, G, dv]`` as they enter the scores; position ``i`` sees ``j <= i``."""
    T, H = q.shape[0], q.shape[1]
    G = k.shape[1]
    hidden = torch.triu(torch.ones(T, T, dtype=torch.bool), 1)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1) @ v[:, g]
    return out


def difference_factor(tensors, prefix: str, diff: float) -> float:
    dot = [float((t64(tensors, f"{prefix}.lq{m}") * t64(tensors, f"{prefix}.lk{m}")).sum()) for m in (1, 2)]
    return math.exp(dot[0]) - math.exp(dot[1]) + diff


def differential_attention(a: torch.Tensor, tensors, prefix: str, mixer: Mapping, eps: float) -> torch.Tensor:
    T = a.shape[0]
    H, G, dim, vdim, diff = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"], mixer["diff"]
    q, k, v = (convolve(a @ t64(tensors, f"{prefix}.{role}").T, t64(tensors, f"{prefix}.{role}.conv")) for role in ("q", "k", "v"))
    q, k, v = q.view(T, H, 2, dim), k.view(T, G, 2, dim), v.view(T, G, vdim)
    first, second = (attend(q[:, :, m], k[:, :, m], v, mixer["scale"]) for m in (0, 1))
    out = rms(first - difference_factor(tensors, prefix, diff) * second, eps) * (1.0 - diff)
    return out.reshape(T, H * vdim) @ t64(tensors, f"{prefix}.o").T


def rotary_attention(a: torch.Tensor, tensors, prefix: str, mixer: Mapping, eps: float) -> torch.Tensor:
    T = a.shape[0]
    H, G, dim, vdim = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"]
    positions = torch.arange(T)
    q, k, v = (a @ t64(tensors, f"{prefix}.{role}").T + t64(tensors, f"{prefix}.{role}.b") for role in ("q", "k", "v"))
    q = rms(turn_neighbours(q.view(T, H, dim), positions, mixer["rot"]), eps)
    k = rms(turn_neighbours(k.view(T, G, dim), positions, mixer["rot"]), eps)
    out = attend(q, k, v.view(T, G, vdim), mixer["scale"])
    return out.reshape(T, H * vdim) @ t64(tensors, f"{prefix}.o").T


def latent_attention(a: torch.Tensor, tensors, prefix: str, mixer: Mapping, eps: float) -> torch.Tensor:
    T = a.shape[0]
    H, dim, rot, vdim, rank = mixer["heads"], mixer["dim"], mixer["rot_dim"], mixer["vdim"], mixer["kv_rank"]
    positions = torch.arange(T)
    q = (a @ t64(tensors, f"{prefix}.q").T).view(T, H, dim + rot)
    down = a @ t64(tensors, f"{prefix}.dkv").T
    c = rms(down[:, :rank], eps) * t64(tensors, f"{prefix}.dkv.norm")
    r = turn_neighbours(down[:, rank:], positions, mixer["rot"])
    q_rot = turn_neighbours(q[:, :, dim:], positions, mixer["rot"])
    keys = (c @ t64(tensors, f"{prefix}.uk").T).view(T, H, dim)
    values = (c @ t64(tensors, f"{prefix}.uv").T).view(T, H, vdim)
    whole = torch.cat([keys, r[:, None, :].expand(T, H, rot)], dim=-1)
    out = attend(torch.cat([q[:, :, :dim], q_rot], dim=-1), whole, values, mixer["scale"])
    return out.reshape(T, H * vdim) @ t64(tensors, f"{prefix}.o").T


def clamped_expert(a: torch.Tensor, tensors, prefix: str, limit: float) -> torch.Tensor:
    g = torch.clamp(a @ t64(tensors, f"{prefix}.gate").T, max=limit)
    u = torch.clamp(a @ t64(tensors, f"{prefix}.up").T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ t64(tensors, f"{prefix}.down").T


def route(scores: torch.Tensor, correction: torch.Tensor, router: Mapping) -> Tuple[List[int], float]:
    """The places one token takes, and how far it is from another choice: the smallest gap between a number that decided
    and the best one that lost (over places in the kept groups, and over groups)."""
    choice = (scores + correction).tolist()
    count, keep, top = router["groups"]["count"], router["groups"]["keep"], router["top"]
    size = len(choice) // count
    best = [max(choice[g * size:(g + 1) * size]) for g in range(count)]
    ranked = sorted(range(count), key=lambda g: (-best[g], g))
    kept = ranked[:keep]
    allowed = sorted((e for e in range(len(choice)) if e // size in kept), key=lambda e: (-choice[e], e))
    gap = best[ranked[keep - 1]] - best[ranked[keep]] if keep < count else float("inf")
    if len(allowed) > top:
        gap = min(gap, choice[allowed[top - 1]] - choice[allowed[top]])
    return allowed[:top], gap


def moe(a: torch.Tensor, tensors, prefix: str, mlp: Mapping, margins: Optional[list] = None) -> torch.Tensor:
    router = mlp["router"]
    experts = router["experts"]
    scores = torch.softmax(a @ t64(tensors, f"{prefix}.router").T, dim=-1)
    weight = torch.zeros_like(scores)
    for t in range(a.shape[0]):
        chosen, gap = route(scores[t], t64(tensors, f"{prefix}.correction"), router)
        if margins is not None:
            margins.append(gap)
        weight[t, chosen] = scores[t, chosen] / (scores[t, chosen].sum() + 1e-20) * router["scale"]
    out = a * weight[:, experts:].sum(-1, keepdim=True)
    for e in range(experts):
        took = weight[:, e].nonzero()[:, 0]
        if len(took):
            out[took] += weight[took, e:e + 1] * clamped_expert(a[took], tensors, f"{prefix}.e{e}", mlp["expert"]["limit"])
    if mlp.get("shared"):
        out = out + clamped_expert(a, tensors, f"{prefix}.shared", mlp["shared"]["limit"])
    return out


MIXERS = {"attention": differential_attention, "attention_2": rotary_attention, "latent_attention": latent_attention}


def owner(config: Mapping, index: int) -> int:
    """The layer whose tensors layer ``index`` runs with."""
    while config["layers"][index].get("weights_of") is not None:
        index = config["layers"][index]["weights_of"]
    return index


def forward(config: Mapping, tensors: Mapping[str, torch.Tensor], ids, layers_out: Optional[list] = None,
            margins: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence run whole."""
    eps = config["norm"]["eps"]
    ids = torch.as_tensor(ids, dtype=torch.int64)
    x = t64(tensors, "embed")[ids] * (config.get("embedding") or {}).get("scale", 1.0)
    for index, layer in enumerate(config["layers"]):
        prefix = f"l{owner(config, index)}"
        a = rms(x, eps) * t64(tensors, f"{prefix}.norm1")
        added = MIXERS[layer["type"]](a, tensors, f"{prefix}.mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            added = added + moe(a, tensors, f"{prefix}.mlp", layer["mlp"], margins)
        x = x + added
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * t64(tensors, "final.norm")) @ t64(tensors, "head").T


def read_config(folder: str) -> dict:
    import json
    import os
    with open(os.path.join(folder, "config.json"), "r", encoding="utf-8") as handle:
        return json.load(handle)


def read_tensors(folder: str) -> Dict[str, torch.Tensor]:
    import os
    from safetensors.torch import load_file
    return load_file(os.path.join(folder, "model.safetensors"))


def generate_greedy(config: Mapping, tensors: Mapping[str, torch.Tensor], prompt: List[int], count: int) -> List[int]:
    """``count`` tokens after ``prompt``, each the first maximum of the last position's logits; every step runs the
    whole sequence again."""
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(torch.argmax(forward(config, tensors, tokens)[-1])))
    return tokens[len(prompt):]
