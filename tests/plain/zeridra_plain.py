"""Plain, slow Zeridra decoder: whole sequences, no cache, one function per mechanism.

Written from the design's equations in this file's own notation; it shares no code with `tokenizer_amd`.
Everything runs on the CPU in the dtype given (float64 by default).  A model is a config dict (the keys of
its config.json) and a dict of tensors by name.
"""
from __future__ import annotations

import json
import os

import torch


def load_folder(folder: str, dtype=torch.float64):
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    tensors = {k: (v if v.dtype in (torch.int32, torch.int64) else v.to(dtype))
               for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return cfg, tensors


# ------------------------------------------------------------------ small pieces
def norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """x over the root of (its mean square + eps), times w, along the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ positions
def turn_neighbours(x: torch.Tensor, positions: torch.Tensor, base: float) -> torch.Tensor:
    """x [T, ..., n]: coordinates 2i and 2i + 1 turn together by the angle p * base^(-2i/n)."""
    n = x.shape[-1]
    rates = torch.tensor([float(base) ** (-2.0 * i / n) for i in range(n // 2)], dtype=x.dtype)
    angles = positions.to(x.dtype)[:, None] * rates[None, :]
    while angles.dim() < x.dim():
        angles = angles.unsqueeze(1)
    cos, sin = torch.cos(angles), torch.sin(angles)
    u, v = x[..., 0::2], x[..., 1::2]
    out = torch.empty_like(x)
    out[..., 0::2] = u * cos - v * sin
    out[..., 1::2] = v * cos + u * sin
    return out


def temperature(positions: torch.Tensor, coef: float, every: int, dtype=torch.float64) -> torch.Tensor:
    """The factor on the query at each position: 1 + coef ln(floor((p + 1) / every) + 1)."""
    steps = torch.div(positions + 1, every, rounding_mode="floor")
    return 1.0 + coef * torch.log(steps.to(dtype) + 1.0)


# ------------------------------------------------------------------ softmax over what a query sees
def visible(T: int, window: int | None = None) -> torch.Tensor:
    """[query, key]: the key is the query itself or before it and, with a window of so many positions, among the last
    `window` ones up to the query."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen if window is None else seen & (i - j < window)


def softmax_with_sink(scores: torch.Tensor, sink: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    """scores [H, T, T], sink [H]: exp(score) over (exp(sink) + the sum of exp(score) over the keys a query sees)."""
    scores = scores.masked_fill(~seen, float("-inf"))
    top = torch.maximum(scores.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(scores - top)
    return e / (torch.exp(sink[:, None, None] - top) + e.sum(dim=-1, keepdim=True))


# ------------------------------------------------------------------ mixers
def latent_pair(h: torch.Tensor, m: dict, w: dict, eps: float):
    """What a token keeps: the normalised latent [T, kv_rank] and the rotated key part [T, rot_dim]."""
    rank = m["kv_rank"]
    down = h @ w["dkv"].T
    return norm(down[:, :rank], w["dkv.norm"], eps), turn_neighbours(down[:, rank:], torch.arange(h.shape[0]), m["rot"]["base"])


def latent_attention(h: torch.Tensor, m: dict, w: dict, eps: float, kept) -> torch.Tensor:
    """Keys and values expanded head by head from the kept latents (this layer's or another's)."""
    T, H, d, e, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = kept
    q = (norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).reshape(T, H, d + e)
    q_rot = turn_neighbours(q[..., d:], torch.arange(T), m["rot"]["base"])
    k, v = (c @ w["uk"].T).reshape(T, H, d), (c @ w["uv"].T).reshape(T, H, dv)
    scores = torch.einsum("qhd,khd->hqk", q[..., :d], k) + torch.einsum("qhe,ke->hqk", q_rot, k_rot)
    weights = softmax_with_sink(scores * float(m["scale"]), w["sink"], visible(T, int(m["mask"]["size"])))
    return torch.einsum("hqk,khv->qhv", weights, v).reshape(T, H * dv) @ w["o"].T


def attention(h: torch.Tensor, m: dict, w: dict) -> torch.Tensor:
    """Grouped heads whose values are the keys; queries scaled by their position; one joins the softmax's denominator."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w["q"].T).reshape(T, H, d)
    k = (h @ w["k"].T).reshape(T, G, d)
    q = q * temperature(torch.arange(T), float(m["q_temp"]["coef"]), int(m["q_temp"]["every"]), h.dtype)[:, None, None]
    k = k.repeat_interleave(H // G, dim=1)                         # head h reads key head h // (H / G)
    scores = torch.einsum("qhd,khd->hqk", q, k) * float(m["scale"])
    weights = softmax_with_sink(scores, torch.zeros(H, dtype=h.dtype), visible(T))
    return torch.einsum("hqk,khd->qhd", weights, k).reshape(T, H * d) @ w["o"].T


# ------------------------------------------------------------------ routed feed-forward
def route(h: torch.Tensor, r: dict, w: dict):
    """Which experts each row uses and with what weights: (chosen [T, top], weights [T, top])."""
    s = torch.sigmoid(h @ w["router"].T)
    best = torch.topk(s, int(r["top"]), dim=-1)
    return best.indices, best.values


def routed_feed_forward(h: torch.Tensor, mlp: dict, w: dict) -> torch.Tensor:
    """A chosen expert is handed the row times its weight."""
    chosen, weights = route(h, mlp["router"], w)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t].tolist(), weights[t]):
            x = a * h[t]
            out[t] = out[t] + w[f"e{e}.down"] @ (silu(w[f"e{e}.gate"] @ x) * (w[f"e{e}.up"] @ x))
    return out


# ------------------------------------------------------------------ the model
def sub(tensors: dict, prefix: str) -> dict:
    lead = prefix + "."
    return {k[len(lead):]: v for k, v in tensors.items() if k.startswith(lead)}


def shaped_logits(z: torch.Tensor, cfg: dict) -> torch.Tensor:
    z = z * float(cfg.get("logit_scale") or 1.0)
    cap = cfg.get("logit_softcap")
    return z if not cap else float(cap) * torch.tanh(z / float(cap))


def forward(cfg: dict, tensors: dict, ids: list[int], layers_out: list | None = None) -> torch.Tensor:
    """Logits [T, vocab] of the whole sequence `ids`; `layers_out` collects the stream behind every layer."""
    eps = float(cfg["norm"]["eps"])
    x = tensors["embed"][torch.tensor(ids)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    kept = {}
    for index, layer in enumerate(cfg["layers"]):
        h = norm(x, tensors[f"l{index}.norm1"], eps)
        m, w = layer["mixer"], sub(tensors, f"l{index}.mix")
        if layer["type"] == "latent_attention":
            source = m.get("kv_from")
            if source is None:
                kept[index] = latent_pair(h, m, w, eps)
            y = latent_attention(h, m, w, eps, kept[index if source is None else int(source)])
        elif layer["type"] == "attention":
            y = attention(h, m, w)
        else:
            raise ValueError(layer["type"])
        y = y * tensors[f"l{index}.ls1"]
        if layer.get("mlp") is not None:
            y = y + routed_feed_forward(h, layer["mlp"], sub(tensors, f"l{index}.mlp")) * tensors[f"l{index}.ls2"]
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return shaped_logits(norm(x, tensors["final.norm"], eps) @ tensors["head"].T, cfg)


def greedy_generate(cfg: dict, tensors: dict, prompt, n_new: int) -> list[int]:
    """The first maximum of the last position's logits, appended and run again from the start, `n_new` times."""
    ids, out = list(prompt), []
    for _ in range(n_new):
        logits = forward(cfg, tensors, ids)[-1]
        out.append(int(torch.argmax(logits)))
        ids.append(out[-1])
    return out
