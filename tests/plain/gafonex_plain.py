"""Plain, slow Gafonex decoder: whole sequences, no cache, one function per mechanism.

Written from the design's equations in this file's own notation; it shares no code with `tokenizer_amd`.
Everything runs on the CPU in the dtype given (float64 by default).  A model is a config dict (the keys of
its config.json) and a dict of tensors by name.
"""
from __future__ import annotations

import json
import math
import os

import torch


def load_folder(folder: str, dtype=torch.float64):
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    tensors = {k: (v if v.dtype in (torch.int32, torch.int64) else v.to(dtype))
               for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return cfg, tensors


# ------------------------------------------------------------------ norms
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over the root of (its mean square + eps), along the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def group_norm(x: torch.Tensor, w: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Each of `groups` equal runs of neighbours brought to unit RMS on its own, the whole times w."""
    n, width = x.shape
    return torch.cat([unit_rms(run, eps) for run in x.reshape(n, groups, width // groups).unbind(1)], dim=-1) * w


# ------------------------------------------------------------------ rotation
def rotation(rot: dict | None) -> tuple[list[float], float]:
    """The rates of a rotation and the factor on its cosines and sines.  With `scaling`, rate i is a mix of f_i and
    f_i / factor whose share climbs from 0 to 1 between the pair that turns `fast` times in `original` positions and
    the pair that turns `slow` times."""
    if not rot or not int(rot["dims"]):
        return [], 1.0
    n, base = int(rot["dims"]), float(rot["base"])
    rates = [base ** (-2.0 * i / n) for i in range(n // 2)]
    scaling = rot.get("scaling")
    if not scaling:
        return rates, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_turning(times: float) -> float:
        return n * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(base))
    first = max(math.floor(pair_turning(float(scaling["fast"]))), 0)
    last = min(math.ceil(pair_turning(float(scaling["slow"]))), n - 1)
    out = []
    for i, f in enumerate(rates):
        share = min(max((i - first) / max(last - first, 0.001), 0.0), 1.0)
        out.append(f / factor * share + f * (1.0 - share))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x: torch.Tensor, positions: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x [n, heads, d]: coordinates i and i + m of every head turn together, m = the number of rates; the
    coordinates from 2 m on pass through as they are."""
    rates, size = rotation(rot)
    m = len(rates)
    if m == 0:
        return x
    angles = positions.to(torch.float64)[:, None] * torch.tensor(rates, dtype=torch.float64)[None, :]
    cos, sin = (size * angles.cos()).to(x.dtype)[:, None, :], (size * angles.sin()).to(x.dtype)[:, None, :]
    u, v, rest = x[..., :m], x[..., m:2 * m], x[..., 2 * m:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


# ------------------------------------------------------------------ mixers
def softmax_maps(q: torch.Tensor, k: torch.Tensor, scale: float) -> torch.Tensor:
    """q [n, H, d], k [n, G, d] -> [H, n, n]: every head's softmax over the keys at or before the query."""
    n, H = q.shape[:2]
    reach = torch.arange(n)[None, :] <= torch.arange(n)[:, None]
    maps = []
    for head in range(H):
        scores = q[:, head] @ k[:, head // (H // k.shape[1])].T * scale
        maps.append(torch.softmax(scores.masked_fill(~reach, float("-inf")), dim=-1))
    return torch.stack(maps)


def talk(maps: torch.Tensor, table: torch.Tensor) -> torch.Tensor:
    """The heads' maps as sums over all heads' maps, row h of the table giving head h's coefficients."""
    return torch.einsum("hg,gij->hij", table, maps)


def talking_attention(h: torch.Tensor, w: dict, m: dict, eps: float, first_values: torch.Tensor | None):
    """(the mixer's output, this layer's values [n, G, dv] after their norm and mix).  `first_values`: the values that
    are mixed in, or None where the layer mixes none in."""
    n = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    positions = torch.arange(n)
    q = rotate(unit_rms((h @ w["q"].T).reshape(n, H, d), eps) * w["q.norm"], positions, m.get("rot"))
    k = rotate(unit_rms((h @ w["k"].T).reshape(n, G, d), eps) * w["k.norm"], positions, m.get("rot"))
    v = unit_rms((h @ w["v"].T).reshape(n, G, dv), eps)
    if first_values is not None:
        share = w["vmix"].reshape(())
        v = (1.0 - share) * v + share * first_values
    maps = talk(softmax_maps(q, k, float(m["scale"])), w["talk"])
    out = torch.stack([maps[head] @ v[:, head // (H // G)] for head in range(H)], dim=1)
    return out.reshape(n, H * dv) @ w["o"].T, v


def retention(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    positions = torch.arange(n)
    q = rotate((h @ w["q"].T).reshape(n, H, d), positions, m.get("rot"))
    k = rotate((h @ w["k"].T).reshape(n, H, d), positions, m.get("rot")) * d ** -0.5
    v = (h @ w["v"].T).reshape(n, H, dv)
    decay = torch.tensor([float(x) for x in m["decay"]], dtype=h.dtype)[:, None, None]
    state = torch.zeros((H, d, dv), dtype=h.dtype)
    reads = []
    for t in range(n):
        state = decay * state + k[t][:, :, None] * v[t][:, None, :]
        reads.append((state * q[t][:, :, None]).sum(dim=1))
    o = unit_rms(torch.stack(reads), eps).reshape(n, H * dv)
    g = h @ w["g"].T
    return (o * (g * torch.sigmoid(g))) @ w["o"].T


# ------------------------------------------------------------------ feed-forward
def relu_gated(h: torch.Tensor, w: dict) -> torch.Tensor:
    return (torch.clamp(h @ w["gate"].T, min=0.0) * (h @ w["up"].T)) @ w["down"].T


# ------------------------------------------------------------------ the model
def sub(tensors: dict, prefix: str) -> dict:
    lead = prefix + "."
    return {name[len(lead):]: value for name, value in tensors.items() if name.startswith(lead)}


def forward(cfg: dict, tensors: dict, tokens, return_layers: bool = False):
    """Logits [n, vocab] of one whole sequence (and, if asked, the stream after every layer)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps, groups = float(cfg["norm"]["eps"]), int(cfg["norm"]["groups"])
    x = tensors["embed"][tokens]
    first_values, after = None, []
    for index, layer in enumerate(cfg["layers"]):
        w = sub(tensors, f"l{index}")
        mix = sub(w, "mix")
        if layer["type"] == "attention":
            mixes = bool(layer["mixer"].get("v_mix"))
            y, values = talking_attention(x, mix, layer["mixer"], eps, first_values if mixes else None)
            if mixes and first_values is None:
                first_values = values
        elif layer["type"] == "retention":
            y = retention(x, mix, layer["mixer"], eps)
        else:
            raise ValueError(layer["type"])
        x = x + group_norm(y, w["norm1"], groups, eps) * w["ls1"]
        if layer.get("mlp") is not None:
            x = x + group_norm(relu_gated(x, sub(w, "mlp")), w["norm2"], groups, eps) * w["ls2"]
        after.append(x)
    logits = group_norm(x, tensors["final.norm"], groups, eps) @ tensors["head"].T
    limit = cfg.get("logit_softcap")
    if limit:
        logits = float(limit) * torch.tanh(logits / float(limit))
    return (logits, after) if return_layers else logits


def greedy_generate(cfg: dict, tensors: dict, prompt, n_new: int) -> list[int]:
    """The first maximum of the last position's logits, appended and run again from the start, `n_new` times."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        logits = forward(cfg, tensors, ids)[-1]
        out.append(int(torch.argmax(logits)))
        ids.append(out[-1])
    return out
