"""A plain, slow implementation of the Mapedra decoder on the CPU, one function per mechanism.

It shares no code with the engine: it takes the configuration as the dictionary that config.json holds and the
tensors by their file names, and computes every sequence whole, position by position where the mechanism is a
recurrence, in float64.

Notation. ``x`` is the residual stream ``[T, width]``, at the start ``E[ids] * embedding.scale``; ``rms(a) = a /
sqrt(mean(a^2) + eps)`` over the last axis; ``N(a, w)`` cuts ``a`` into ``norm.groups`` equal runs of neighbours, takes
``rms`` of each and multiplies the whole by ``w``. Layer ``i``:

    x += N(M(x), w1);    x += N(F(x), w2) if it has a feed-forward;
    x += rms(P (gelu(G x) * e_i)) * ws,    e_i = columns i n .. (i + 1) n - 1 of the token's row of the side table

with the tanh form of gelu. The mixers ``M``:

* ``attention``: grouped heads; ``q`` and ``k`` are ``rms`` over the head times a weight all heads share; of each head's
  first ``rot.dims`` dimensions ``2i`` turns with ``2i + 1`` by ``p * f_i`` (``f_i`` from ``rates`` below); ``v`` is ``rms``
  over the head; ``s = c * tanh(scale * q . k / c)`` over ``j <= i``; softmax; the heads side by side times
  ``sigmoid(Wg x)``; ``Wo``.
* ``lightning``: ``q = silu(Wq x)``, ``k = silu(Wk x)``, ``v = silu(Wv x)``; per head
  ``S <- decay_h S + k v^T``, ``o = S^T q``; the heads side by side are ``rms`` together, times a weight, times
  ``sigmoid(Wg x)``; ``Wo``.

``F`` is ``Wd (gelu(Wg x) * (Wu x))``. At the end ``N(x, wf)`` and the head.
"""
from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional

import torch

F = torch.float64


def t64(tensors: Mapping[str, torch.Tensor], name: str) -> torch.Tensor:
    return tensors[name].to(F)


def rms(a: torch.Tensor, eps: float) -> torch.Tensor:
    return a / torch.sqrt((a * a).mean(-1, keepdim=True) + eps)


def grouped_rms(a: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    size = a.shape[-1] // groups
    return torch.cat([rms(a[..., g * size:(g + 1) * size], eps) for g in range(groups)], dim=-1)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rates(base: float, n: int, scaling: Optional[Mapping] = None) -> List[float]:
    """Angle a position for each of the ``n / 2`` pairs. With ``scaling`` (factor, low, high, original) a slow rate (a
    wavelength above ``original / low``) is divided by the factor, a fast one (below ``original / high``) is left, and
    one between is a blend of the two."""
    out = []
    for i in range(n // 2):
        f = base ** (-2.0 * i / n)
        if scaling is not None:
            wave = 2.0 * math.pi / f
            if wave > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif wave >= scaling["original"] / scaling["high"]:
                s = (scaling["original"] / wave - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def turn_neighbours(a: torch.Tensor, positions: torch.Tensor, base: float, n: int, scaling: Optional[Mapping] = None) -> torch.Tensor:
    """``a`` is ``[T, ..., D]``; of its first ``n`` dims, ``2i`` and ``2i + 1`` are turned together; the rest pass."""
    # a float32 evaluation rounds its angles' sines and cosines, not its angles
    angle = positions.to(torch.float64)[:, None] * torch.tensor(rates(base, n, scaling), dtype=torch.float64)[None, :]
    shape = [a.shape[0]] + [1] * (a.dim() - 2) + [n // 2]
    cos, sin = torch.cos(angle).to(F).view(shape), torch.sin(angle).to(F).view(shape)
    u, v = a[..., 0:n:2], a[..., 1:n:2]
    out = a.clone()
    out[..., 0:n:2] = u * cos - v * sin
    out[..., 1:n:2] = v * cos + u * sin
    return out


def attend_capped(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: Optional[float]) -> torch.Tensor:
    """``q`` ``[T, H, d]``, ``k`` ``[T, G, d]``, ``v`` ``[T, G, dv]`` as they enter the scores; position ``i`` sees ``j <= i``."""
    T, H = q.shape[0], q.shape[1]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if cap is not None:
            s = cap * torch.tanh(s / cap)
        out[:, h] = torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1) @ v[:, g]
    return out


def attention(a: torch.Tensor, tensors, prefix: str, mixer: Mapping, eps: float) -> torch.Tensor:
    T = a.shape[0]
    H, G, dim, vdim, rot = mixer["heads"], mixer["kv_heads"], mixer["dim"], mixer["vdim"], mixer["rot"]
    positions = torch.arange(T)
    q = rms((a @ t64(tensors, f"{prefix}.q").T).view(T, H, dim), eps) * t64(tensors, f"{prefix}.q.norm")
    k = rms((a @ t64(tensors, f"{prefix}.k").T).view(T, G, dim), eps) * t64(tensors, f"{prefix}.k.norm")
    v = rms((a @ t64(tensors, f"{prefix}.v").T).view(T, G, vdim), eps)
    q = turn_neighbours(q, positions, rot["base"], rot["dims"], rot.get("scaling"))
    k = turn_neighbours(k, positions, rot["base"], rot["dims"], rot.get("scaling"))
    out = attend_capped(q, k, v, mixer["scale"], mixer.get("softcap")).reshape(T, H * vdim)
    return (out * torch.sigmoid(a @ t64(tensors, f"{prefix}.g").T)) @ t64(tensors, f"{prefix}.o").T


def retain(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay, state: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``S <- decay_h S + k v^T``, ``o = S^T q`` token by token; ``q``, ``k`` ``[T, H, d]``, ``v`` ``[T, H, dv]``."""
    T, H, dim = q.shape
    decay = torch.as_tensor(decay, dtype=F)
    state = torch.zeros(H, dim, v.shape[2], dtype=F) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        state = decay[:, None, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (state * q[t][:, :, None]).sum(1)
    return out


def lightning(a: torch.Tensor, tensors, prefix: str, mixer: Mapping, eps: float) -> torch.Tensor:
    T = a.shape[0]
    H, dim, vdim = mixer["heads"], mixer["dim"], mixer["vdim"]
    q = silu(a @ t64(tensors, f"{prefix}.q").T).view(T, H, dim)
    k = silu(a @ t64(tensors, f"{prefix}.k").T).view(T, H, dim)
    v = silu(a @ t64(tensors, f"{prefix}.v").T).view(T, H, vdim)
    out = rms(retain(q, k, v, mixer["decay"]).reshape(T, H * vdim), eps) * t64(tensors, f"{prefix}.norm")
    return (out * torch.sigmoid(a @ t64(tensors, f"{prefix}.g").T)) @ t64(tensors, f"{prefix}.o").T


def gated_gelu(a: torch.Tensor, tensors, prefix: str) -> torch.Tensor:
    return (gelu_tanh(a @ t64(tensors, f"{prefix}.gate").T) * (a @ t64(tensors, f"{prefix}.up").T)) @ t64(tensors, f"{prefix}.down").T


def token_side_input(a: torch.Tensor, tensors, index: int, n: int, ids: torch.Tensor) -> torch.Tensor:
    """``P (gelu(G a) * e)`` before its norm."""
    e = t64(tensors, "side.embed")[ids][:, index * n:(index + 1) * n]
    return (gelu_tanh(a @ t64(tensors, f"l{index}.side.gate").T) * e) @ t64(tensors, f"l{index}.side.proj").T


MIXERS = {"attention": attention, "lightning": lightning}


def forward(config: Mapping, tensors: Mapping[str, torch.Tensor], ids, layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence run whole."""
    eps, groups = config["norm"]["eps"], config["norm"].get("groups", 1)
    n = config["token_side"]["dim"]
    ids = torch.as_tensor(ids, dtype=torch.int64)
    x = t64(tensors, "embed")[ids] * (config.get("embedding") or {}).get("scale", 1.0)
    for index, layer in enumerate(config["layers"]):
        prefix = f"l{index}"
        mixed = MIXERS[layer["type"]](x, tensors, f"{prefix}.mix", layer["mixer"], eps)
        x = x + grouped_rms(mixed, groups, eps) * t64(tensors, f"{prefix}.norm1")
        if layer.get("mlp") is not None:
            assert layer["mlp"]["kind"] == "dense"
            x = x + grouped_rms(gated_gelu(x, tensors, f"{prefix}.mlp"), groups, eps) * t64(tensors, f"{prefix}.norm2")
        x = x + rms(token_side_input(x, tensors, index, n, ids), eps) * t64(tensors, f"{prefix}.side.norm")
        if layers_out is not None:
            layers_out.append(x.clone())
    return (grouped_rms(x, groups, eps) * t64(tensors, "final.norm")) @ t64(tensors, "head").T


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
