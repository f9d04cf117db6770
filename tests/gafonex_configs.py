"""Tiny Gafonex configurations for the tests, and their model folders.  They differ in every size and constant and in
the order of their layers; head counts and groupings, key and value sizes, rotated coordinates, decays, norm groups and
inner widths take values that make nothing equal by accident (and some the values 1 and 0)."""
import os

import torch


def _rot(dims, base, yarn=None):
    out = {"dims": dims, "base": base}
    if yarn is not None:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return out


def _attention(heads, kv_heads, dim, vdim, scale, rot=None, v_mix=None, ff=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        mixer["rot"] = rot
    if v_mix is not None:
        mixer["v_mix"] = v_mix
    return {"type": "attention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _retention(decay, dim, vdim, rot=None, ff=None):
    mixer = {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        mixer["rot"] = rot
    return {"type": "retention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _model(vocab, width, eps, groups, layers, softcap=None):
    out = {"architecture": "Gafonex", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "layers": layers}
    if softcap is not None:
        out["logit_softcap"] = softcap
    return out


GAFONEX = {
    # name: (config.json keys, weight seed)
    # Attention first; values given by layer 0 and taken in by layers 2 and 4, layer 3 stands aside; a layer of a mixer
    # alone of either kind; a rotation of a part of the head with slowed long waves; values wider than keys.
    "A": (_model(149, 64, 1e-5, 4, [
        _attention(4, 2, 16, 24, 0.6, _rot(12, 400.0, (4.0, 40, 6.0, 1.0)), True, 40),
        _retention((0.9, 0.97, 0.996), 20, 12, _rot(16, 3000.0), 56),
        _attention(6, 2, 12, 24, 0.7, _rot(12, 5000.0), True),
        _attention(2, 1, 32, 16, 0.5, _rot(32, 10000.0, (8.0, 64, 16.0, 2.0)), None, 24),
        _attention(2, 2, 20, 24, 0.5, None, True, 72),
        _retention((0.5, 0.999), 8, 40, None)], 11.0), 5),
    # Sizes that are no multiples of eight anywhere; as many key heads as heads; one head; an odd number of retention
    # heads; nothing rotated in one layer; the values are given and nobody takes them; logits as they are.
    "B": (_model(83, 54, 2e-6, 3, [
        _retention((0.98, 0.93, 0.7, 0.999, 1.0), 6, 10, _rot(4, 60.0), 30),
        _attention(3, 3, 10, 14, 0.9, _rot(6, 90.0, (2.0, 24, 3.0, 0.5)), False, 50),
        _attention(5, 1, 14, 6, 0.8, None, True, 22)]), 17),
    # Head sizes in sixteens (the matrix-core kernels' sizes), four and sixteen heads, two and one kv heads, a retention
    # whose heads fill sixty-four; one group over the whole width.
    "C": (_model(200, 128, 1e-6, 1, [
        _retention((0.97, 0.99), 64, 64, _rot(64, 10000.0), 96),
        _attention(4, 2, 64, 64, 0.3, _rot(64, 500000.0, (16.0, 128, 32.0, 1.0)), True, 160),
        _attention(16, 2, 32, 64, 0.45, _rot(32, 1000.0), True, 64),
        _retention((0.95, 0.995, 0.9, 0.9995), 32, 48, _rot(32, 100.0), 128),
        _attention(20, 4, 16, 32, 0.5, _rot(16, 100.0), False, 32)], 25.0), 33),
    # One of everything: one head, a pair of coordinates that turns, a decay of one, small groups; an attention layer gives
    # its values to the next.
    "D": (_model(60, 36, 1e-6, 3, [
        _retention((0.6,), 6, 9, _rot(2, 10.0), 8), _attention(1, 1, 2, 10, 0.7, _rot(2, 10.0), True, 12),
        _retention((1.0,), 5, 14, None), _attention(1, 1, 4, 10, 0.7, _rot(2, 20.0, (3.0, 16, 2.0, 1.0)), True, 16)]), 40),
    # A width that is no multiple of four, more kv heads than two under many heads, wide values.
    "E": (_model(131, 50, 1e-5, 5, [
        _attention(12, 4, 8, 40, 0.8, _rot(8, 50.0), True, 34), _attention(8, 4, 24, 40, 0.4, _rot(20, 700.0), True, 18),
        _retention((0.99, 0.96, 0.998, 0.9), 18, 26, _rot(10, 40.0, None), 44)], 14.0), 58),
}


def write_model(raw: dict, seed: int, folder: str, sharpen: float = 5.0) -> str:
    """A model folder from the random-weights mode, with its matrices made `sharpen` times larger (the sub-layers read
    the stream as it is, of the size the embedding gives it), the heads' mixing tables and the shares of the values that
    are taken in far from the identity and from zero, and norms and layer scales spread: a head's weights mixed wrongly,
    a lost state or values of the wrong layer then move the logits by much more than rounding does."""
    import tokenizer_amd as ta
    from safetensors.torch import load_file, save_file
    from tokenizer_amd.config import GafonexConfig

    ta.write_random_model(GafonexConfig.from_dict(raw), seed, folder, norm_spread=0.3)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for name, tensor in tensors.items():
        if name == "embed":
            tensors[name] = (tensor.float() * 50.0).to(torch.bfloat16)
        elif name == "head":
            tensors[name] = (tensor.float() * 8.0).to(torch.bfloat16)           # logits of order 1, so that their cap bends them
        elif name.endswith(".vmix"):
            tensors[name] = (0.45 + tensor.float()).to(torch.bfloat16)
        elif tensor.dim() == 2 and not name.endswith(".talk"):
            tensors[name] = (tensor.float() * sharpen).to(torch.bfloat16)
    save_file(tensors, path)
    return folder


def random_config(seed: int) -> dict:
    """A Gafonex configuration drawn from a seed: the number and order of layers, head counts and groupings, key and value
    sizes (some in sixteens, some not), rotated coordinates with and without slowed waves, decays, groups, inner widths,
    layers without a feed-forward, values that are given and taken in."""
    import random
    rng = random.Random(seed)
    groups = rng.choice([1, 1, 2, 4, 8])
    width = groups * rng.choice([8, 12, 16]) * rng.choice([1, 2])
    kv_heads, vdim = rng.choice([1, 2, 2, 3, 4]), rng.choice([8, 16, 16, 32, 48, 64, 20])    # of the layers that share values

    def rot(dim):
        dims = rng.choice([0, 2, dim // 4 * 2, dim // 2 * 2])
        if dims == 0 and rng.random() < 0.5:
            return None
        yarn = (rng.choice([2.0, 4.0, 32.0]), rng.choice([16, 64, 500]), rng.choice([4.0, 32.0]), 1.0) if dims and rng.random() < 0.5 else None
        return _rot(dims, rng.choice([40.0, 1000.0, 500000.0]), yarn)
    layers = []
    for _ in range(rng.randint(2, 5)):
        ff = rng.choice([None, 16, 24, 50, 64])
        if rng.random() < 0.5:
            dim = rng.choice([8, 12, 16, 32, 48])
            decay = [rng.choice([0.5, 0.9, 0.97, 0.99, 0.999, 1.0]) for _ in range(rng.choice([1, 2, 3, 4, 6]))]
            layers.append(_retention(decay, dim, rng.choice([8, 10, 16, 32, 64]), rot(dim), ff))
            continue
        dim, share = rng.choice([8, 10, 16, 32, 48, 64]), rng.random() < 0.7
        kv, dv = (kv_heads, vdim) if share else (rng.choice([1, 2, 3]), rng.choice([8, 16, 24, 32]))
        layers.append(_attention(kv * rng.choice([1, 2, 3, 4]), kv, dim, dv, rng.choice([0.3, 0.5, dim ** -0.5]), rot(dim), share, ff))
    return _model(rng.choice([61, 128, 200, 333]), width, rng.choice([1e-6, 1e-5]), groups, layers, rng.choice([None, 10.0, 35.0]))
