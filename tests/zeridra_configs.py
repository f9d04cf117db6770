"""Tiny Zeridra configurations for the tests, and their model folders.  They differ in every size and constant and in the
order of their layers; head counts and groupings, head, value and latent sizes, windows, rotated coordinates, query
temperatures and expert counts take values that make nothing equal by accident (and some the values 1 and 0)."""
import os

import torch


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, window, scale, base, kv_from=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
             "scale": scale, "mask": {"size": window}, "rot": {"dims": rot_dim, "base": base}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return "latent_attention", mixer


def _attention(heads, kv_heads, dim, scale, coef, every):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                         "q_temp": {"coef": coef, "every": every}}


def _layer(kind_mixer, moe=None):
    mlp = None if moe is None else {"kind": "moe", "expert": {"ff": moe[2]}, "router": {"experts": moe[0], "top": moe[1]}}
    return {"type": kind_mixer[0], "mixer": kind_mixer[1], "mlp": mlp}


def _model(vocab, width, eps, scale, logit_scale, cap, layers):
    out = {"architecture": "Zeridra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_scale": logit_scale, "layers": layers}
    if cap is not None:
        out["logit_softcap"] = cap
    return out


ZERIDRA = {
    # name: (config.json keys, weight seed)
    # Both mixers; layer 3 reads layer 1's latents over a wider window than layer 1's own, layer 5 over a narrower one;
    # another latent layer keeps its own; a layer without feed-forward.
    "A": (_model(211, 64, 1e-5, 8.0, 0.7, 20.0, [
        _layer(_attention(4, 2, 16, 0.3, 0.4, 11), (6, 2, 24)), _layer(_latent(4, 16, 8, 24, 24, 40, 19, 0.3, 10000.0), (4, 1, 20)),
        _layer(_attention(6, 2, 24, 0.2, 0.25, 30)), _layer(_latent(3, 20, 8, 16, 32, 40, 37, 0.25, 10000.0, kv_from=1), (5, 3, 16)),
        _layer(_latent(2, 16, 4, 8, 16, 32, 33, 0.35, 500.0), (8, 2, 16)),
        _layer(_latent(5, 12, 8, 10, 28, 40, 5, 0.3, 10000.0, kv_from=1), (3, 1, 40))]), 10),
    # Sizes that are no multiples of eight anywhere; as many key heads as query heads; every expert chosen.
    "B": (_model(97, 52, 2e-6, 3.5, 1.3, 9.0, [
        _layer(_latent(3, 10, 6, 14, 20, 22, 21, 0.35, 300.0), (5, 1, 10)), _layer(_attention(3, 3, 10, 0.4, 0.5, 7), (3, 3, 14)),
        _layer(_latent(2, 6, 6, 10, 12, 22, 22, 0.4, 300.0, kv_from=0), (4, 2, 12))]), 8),
    # Heads and latents in sixteens (the sizes the matrix-core kernels take); windows of a page, of a page and one, of
    # blocks of keys and one less; one key head for five heads.  (Few experts a layer: the more there are,
    # the more rows have two of nearly equal scores, which bfloat16 rounding tips.)
    "C": (_model(180, 128, 1e-6, 11.3, 0.4, 14.0, [
        _layer(_latent(4, 32, 16, 32, 48, 48, 65, 0.2, 50000.0), (4, 1, 32)), _layer(_attention(5, 1, 32, 0.25, 0.3, 16), (4, 3, 32)),
        _layer(_latent(3, 16, 16, 64, 64, 48, 64, 0.25, 50000.0, kv_from=0), (3, 1, 24)),
        _layer(_latent(2, 32, 32, 32, 40, 96, 17, 0.18, 100000.0), (4, 4, 48)),
        _layer(_attention(8, 2, 64, 0.15, 0.6, 45), (5, 2, 40)),
        _layer(_latent(6, 16, 32, 16, 32, 96, 16, 0.2, 100000.0, kv_from=3), (2, 1, 32))]), 21),
    # One of everything: one head, a pair of coordinates that turns, windows of one and two tokens, one expert, a
    # temperature that steps at every position and one that is none, no cap.
    "D": (_model(120, 40, 1e-6, 1.0, 1.0, None, [
        _layer(_latent(1, 24, 2, 40, 16, 30, 1, 0.2, 100.0), (1, 1, 16)), _layer(_attention(1, 1, 20, 0.35, 0.2, 1), (3, 1, 16)),
        _layer(_latent(2, 8, 2, 6, 8, 30, 2, 0.3, 100.0, kv_from=0), (2, 1, 8)), _layer(_attention(4, 4, 8, 0.5, 0.0, 5))]), 34),
}


def write_model(raw: dict, seed: int, folder: str, sharpen: float = 5.0, router: float = 0.6) -> str:
    """A model folder from the random-weights mode, with its matrices made `sharpen` times larger, so that attention
    weights are peaked: a key too many or too few then moves the logits by much more than rounding does.  The routers'
    scores (`router` times the drawn weights) lie well between 0 and 1, so that they weigh; the embedding is of the size of
    what the layers add, and the logits of a size that their cap bends."""
    import tokenizer_amd as ta
    from safetensors.torch import load_file, save_file
    from tokenizer_amd.config import ZeridraConfig

    ta.write_random_model(ZeridraConfig.from_dict(raw), seed, folder, norm_spread=0.3)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for name, tensor in tensors.items():
        if name == "embed":
            tensors[name] = (tensor.float() * 50.0 / float(raw["embedding"]["scale"])).to(torch.bfloat16)
        elif name == "head":
            tensors[name] = (tensor.float() * 12.0).to(torch.bfloat16)
        elif name.endswith(".router"):
            tensors[name] = (tensor.float() * router).to(torch.bfloat16)
        elif tensor.dim() == 2:
            tensors[name] = (tensor.float() * sharpen).to(torch.bfloat16)
    save_file(tensors, path)
    return folder


def random_config(seed: int) -> dict:
    """A Zeridra configuration drawn from a seed: the number and order of layers, head counts and groupings, head, value
    and latent sizes (some in sixteens, some odd multiples of two), windows, latents that later layers read, query
    temperatures, experts, layers without a feed-forward."""
    import random
    rng = random.Random(seed)
    width = rng.choice([32, 40, 64, 72, 96, 128])
    layers, owners = [], []
    for index in range(rng.randint(2, 6)):
        moe = None
        if rng.random() < 0.8:
            experts = rng.choice([1, 2, 3, 5, 8, 12, 20])
            moe = (experts, rng.randint(1, min(4, experts)), rng.choice([8, 10, 16, 24, 32]))
        dim = rng.choice([8, 12, 16, 16, 32, 32, 48, 64])
        if rng.random() < 0.4:
            kv_heads = rng.choice([1, 1, 2, 3])
            layers.append(_layer(_attention(kv_heads * rng.choice([1, 2, 3, 4]), kv_heads, dim, rng.choice([dim ** -0.5, 0.2, 0.35]),
                                            rng.choice([0.1, 0.3, 0.8]), rng.choice([1, 4, 9, 16, 50])), moe))
            continue
        heads, vdim, q_rank = rng.choice([1, 2, 3, 4, 6]), rng.choice([8, 10, 16, 24, 40]), rng.choice([8, 12, 16, 24, 40])
        scale, window = rng.choice([dim ** -0.5, 0.2, 0.35]), rng.choice([1, 2, 7, 15, 16, 17, 24, 31, 33, 40])
        if owners and rng.random() < 0.5:
            source = rng.choice(owners)
            theirs = layers[source]["mixer"]
            layers.append(_layer(_latent(heads, dim, theirs["rot_dim"], vdim, q_rank, theirs["kv_rank"], window, scale,
                                         theirs["rot"]["base"], kv_from=source), moe))
            continue
        owners.append(index)
        layers.append(_layer(_latent(heads, dim, rng.choice([2, 4, 8, 16, 16, 32]), vdim, q_rank, rng.choice([8, 16, 22, 32, 48, 64, 96]),
                                     window, scale, rng.choice([100.0, 10000.0, 500000.0])), moe))
    return _model(rng.choice([61, 128, 200, 333]), width, rng.choice([1e-6, 1e-5]), rng.choice([1.0, 5.0, width ** 0.5]),
                  rng.choice([0.3, 1.0, 1.7]), rng.choice([None, 12.0, 30.0]), layers)
