"""Gafonex through the framework against the plain implementation of tests/plain/gafonex_plain.py.

Every test runs on three backends: the engine on the CPU with the plain torch ops standing in for the kernel
library (the host side: tables, slots, batching), and the engine on the GPU in float32 and in bfloat16
(the HIP kernels).  The models are the tiny ones of gafonex_configs.py with sharpened weights; the mechanisms alone
run as the framework's own parts (the registered mixers and feed-forwards) over a cache manager and pools of their own.
"""
import copy
import math

import pytest
import torch

import trace_tools as tt
from gafonex_configs import GAFONEX, random_config, write_model
from plain import gafonex_plain as plain
from test_bokulorn import BACKENDS, CUTS, PartRunner, make_engine, ops_for, rounded, tolerance
from tiny_configs import random_ids


# float32: sums in another order, against logits of order 1 (sub-layers' outputs are brought to unit size whatever theirs
# is, which makes more of a small one's rounding).  bfloat16: the bound is on each row's root mean square error against
# the row's own spread; a lost key, a state that starts from zeros or a head mixed wrongly moves a row by its spread.
TOL = {"cpu": 1e-4, "gpu-float32": 2e-4, "gpu-bfloat16": 0.15}


def close(got, want, backend, what=""):
    got = got.float().cpu()
    if backend == "gpu-bfloat16":
        spread = (want - want.mean(dim=-1, keepdim=True)).pow(2).mean(dim=-1).sqrt()
        off = (got - want).pow(2).mean(dim=-1).sqrt() / spread
        assert int((off > TOL[backend]).sum()) <= max(1, off.numel() // 20) and float(off.median()) <= TOL[backend] / 2, \
            f"{what}: rows are off by up to {float(off.max())} of their spread, {int((off > TOL[backend]).sum())} over the bound"
        return
    err = float((got - want).abs().max())
    bound = TOL[backend] * max(float(want.abs().max()), 1.0)
    assert err <= bound, f"{what}: max abs error {err} against a bound of {bound}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("gafonex")
    return {name: write_model(raw, seed, str(root / name)) for name, (raw, seed) in GAFONEX.items()}


@pytest.fixture(scope="module")
def oracle(folders):
    cache = {}

    def get(name, ids):
        key = (name, tuple(ids))
        if key not in cache:
            cfg, tensors = plain.load_folder(folders[name])
            cache[key] = plain.forward(cfg, tensors, list(ids)).to(torch.float32)
        return cache[key]
    return get


def requests_for(name, lengths=(1, 2, 3, 21, 50, 97, 64, 33)):
    vocab = GAFONEX[name][0]["vocab"]
    return {f"r{i}": random_ids(vocab, n, 40 + i) for i, n in enumerate(lengths)}


def check_trace(folders, oracle, name, backend, steps, reqs, **kw):
    eng = make_engine(folders[name], backend, max_tokens=tt.peak_tokens(steps), max_requests=4, **kw)
    eng.pools.poison()          # pages and state rows that no request wrote read as NaN
    got = tt.run_in_process(eng, steps)
    for rid, ids in reqs.items():
        close(got[rid], oracle(name, ids), backend, rid)
    eng.cache.check_invariants()
    assert not eng.cache.requests
    return eng


NAMES = list(GAFONEX)


# ------------------------------------------------------------------ whole models through the engine
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts_and_the_first_tokens(folders, oracle, name, backend):
    reqs = requests_for(name)
    check_trace(folders, oracle, name, backend, tt.whole(reqs), reqs)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(folders, oracle, name, backend):
    # The tail of 50 passes page borders of 16 and carries the states from a prompt into single tokens; a request of 51
    # starts decoding behind its very first token.
    reqs = requests_for(name, (60, 97, 64, 51))
    check_trace(folders, oracle, name, backend, tt.decode_tail(reqs, 50), reqs)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("seed", [3, 4])
def test_portions_down_to_two_tokens(folders, oracle, name, backend, seed):
    reqs = requests_for(name, (97, 50, 64, 7))
    steps = tt.portions(reqs, seed)
    assert any(len(s["entries"][0]["tokens"]) == 2 for s in steps)
    check_trace(folders, oracle, name, backend, steps, reqs)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("seed", [6, 7])
def test_mixed_batches_with_pages_and_slots_used_again(folders, oracle, name, backend, seed):
    reqs = requests_for(name, (33, 97, 21, 64, 50, 80, 12, 45, 3, 70))
    steps = tt.mixed(reqs, seed, max_live=4, tail=14)
    assert max(len(s["entries"]) for s in steps) >= 3
    eng = check_trace(folders, oracle, name, backend, steps, reqs)
    assert eng.cache.max_requests == 4          # ten requests went through four slots


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["A", "C"])
@pytest.mark.parametrize("page_size", [16, 48])
def test_other_page_sizes_and_batches_against_each_request_alone(folders, oracle, backend, name, page_size):
    from tokenizer_amd.engine import StepEntry
    reqs = requests_for(name, (70, 9, 31))
    eng = make_engine(folders[name], backend, num_pages=24, page_size=page_size, max_requests=3)
    eng.pools.poison()
    for rid in reqs:
        eng.add_request(rid)
    heads = {rid: len(ids) - 5 for rid, ids in reqs.items()}
    got = {rid: [] for rid in reqs}
    logits = eng.step([StepEntry(rid, ids[:heads[rid]], list(range(heads[rid]))) for rid, ids in reqs.items()]).float().cpu()
    row = 0
    for rid in reqs:
        got[rid].append(logits[row:row + heads[rid]])
        row += heads[rid]
    for k in range(5):
        logits = eng.step([StepEntry(rid, [ids[heads[rid] + k]], [0]) for rid, ids in reqs.items()]).float().cpu()
        for row, rid in enumerate(reqs):
            got[rid].append(logits[row:row + 1])
    for rid, ids in reqs.items():
        close(torch.cat(got[rid]), oracle(name, ids), backend, rid)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_long_decoding(folders, oracle, name, backend):
    ids = random_ids(GAFONEX[name][0]["vocab"], 230, 77)
    reqs = {"long": ids}
    check_trace(folders, oracle, name, backend, tt.decode_tail(reqs, tail=227), reqs)


@pytest.mark.parametrize("backend", BACKENDS)
def test_greedy_generation_through_the_entry_point_and_the_scheduler(folders, backend):
    from tokenizer_amd.engine import GenerateParams, Scheduler, SchedulerConfig, generate
    name = "A"
    cfg, tensors = plain.load_folder(folders[name])
    prompts = [random_ids(cfg["vocab"], n, 90 + n) for n in (11, 30, 4)]
    want = [plain.greedy_generate(cfg, tensors, p, 9) for p in prompts]
    eng = make_engine(folders[name], backend, num_pages=16, max_requests=4)
    eng.pools.poison()
    alone = [generate(eng, p, GenerateParams.greedy(9)).tokens for p in prompts]
    sched = Scheduler(eng, SchedulerConfig(num_blocks=16, max_batch_size=4))
    rids = [sched.add_request(p, GenerateParams.greedy(9)) for p in prompts]
    results = sched.run()
    together = [results[rid].tokens for rid in rids]
    if backend != "gpu-bfloat16":           # (bfloat16 may pick another of two near-equal logits)
        assert alone == together == want
        return
    for prompt, *both in zip(prompts, alone, together):
        for picked in both:
            logits = plain.forward(cfg, tensors, prompt + picked)[len(prompt) - 1:-1]
            for row, token in zip(logits, picked):
                assert float(row.max() - row[token]) <= 0.3 * float(row.std())


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut", ["whole", "tail", "portions", "mixed"])
@pytest.mark.parametrize("name", ["C", "A", "E"])
def test_hundreds_of_tokens(folders, oracle, dtype, cut, name):
    """Prompts long enough for the prompt kernels' tiles and for the recurrence in chunks."""
    reqs = requests_for(name, (300, 17, 411, 130))
    steps = {"whole": lambda: tt.whole(reqs), "tail": lambda: tt.decode_tail(reqs, 40),
             "portions": lambda: tt.portions(reqs, 11), "mixed": lambda: tt.mixed(reqs, 12, max_live=4, tail=10)}[cut]()
    check_trace(folders, oracle, name, f"gpu-{dtype}", steps, reqs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_replay_program_on_a_model_folder(folders, oracle, tmp_path, dtype):
    name = "B"
    reqs = requests_for(name, (40, 23, 5, 64, 31))
    steps = tt.mixed(reqs, 9, max_live=4, tail=6)
    got = tt.run_program(folders[name], dtype, steps, str(tmp_path / "out"), tt.peak_tokens(steps), GAFONEX[name][0]["vocab"])
    for rid, ids in reqs.items():
        close(got[rid], oracle(name, ids), f"gpu-{dtype}", rid)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("seed", list(range(1, 17)))
def test_models_drawn_from_a_seed(tmp_path, backend, seed):
    """Other numbers of layers, sizes and constants; whole, then cut and batched."""
    raw = random_config(seed)
    folder = write_model(raw, 100 + seed, str(tmp_path / "m"), sharpen=3.0)
    cfg, tensors = plain.load_folder(folder)
    reqs = {f"r{i}": random_ids(raw["vocab"], n, seed * 10 + i) for i, n in enumerate((37, 5, 52))}
    steps = tt.mixed(reqs, seed, max_live=3, tail=5) if seed % 2 else tt.portions(reqs, seed)
    eng = make_engine(folder, backend, max_tokens=tt.peak_tokens(steps), max_requests=3)
    eng.pools.poison()
    got = tt.run_in_process(eng, steps)
    for rid, ids in reqs.items():
        close(got[rid], plain.forward(cfg, tensors, ids).float(), backend, f"seed {seed} {rid}")


def test_the_checks_above_would_see_each_mechanism(folders):
    """Each mechanism left out of the oracle moves its logits far beyond the tests' bounds."""
    name = "A"
    cfg, tensors = plain.load_folder(folders[name])
    ids = random_ids(cfg["vocab"], 60, 8)
    right = plain.forward(cfg, tensors, ids)
    spread = float((right - right.mean(-1, keepdim=True)).pow(2).mean().sqrt())

    def moved(change_cfg=None, change=None):
        c, t = copy.deepcopy(cfg), dict(tensors)
        if change_cfg:
            change_cfg(c)
        if change:
            t.update(change(t))
        return float((plain.forward(c, t, ids)[20:] - right[20:]).pow(2).mean().sqrt()) / spread
    assert moved(change=lambda t: {n: torch.eye(v.shape[0], dtype=v.dtype) for n, v in t.items() if n.endswith(".talk")}) > 0.2
    assert moved(change=lambda t: {n: 0 * v for n, v in t.items() if n.endswith(".vmix")}) > 0.2
    assert moved(change=lambda t: {n: 0 * v + 1 for n, v in t.items() if n.endswith((".ls1", ".ls2"))}) > 0.2
    assert moved(lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling")) > 0.02
    assert moved(lambda c: c["norm"].update(groups=2)) > 0.1
    assert moved(lambda c: c["layers"][1]["mixer"].update(decay=[0.9, 0.97, 0.98])) > 0.02
    assert moved(lambda c: c.pop("logit_softcap")) > 1e-3


# ------------------------------------------------------------------ configuration, registry
def test_the_spec_says_who_gives_values_and_what_the_layers_keep():
    from tokenizer_amd.config import GafonexConfig
    from tokenizer_amd.models.gafonex import gafonex_spec
    from tokenizer_amd.parts import cache_needs, expected_tensors
    spec = gafonex_spec(GafonexConfig.from_dict(GAFONEX["A"][0]))
    assert [layer.mixer.value_mix for layer in spec.layers] == ["give", None, "take", None, "take", None]
    needs = cache_needs(spec)
    assert needs[0].kind == "full" and (needs[0].n_kv_heads, needs[0].head_dim, needs[0].v_dim) == (2, 16, 24)
    assert needs[1].kind == "none" and needs[1].state_shape == (3 * 20 * 12,)
    names = set(expected_tensors(spec))
    assert {"l0.mix.vmix", "l0.mix.talk", "l0.mix.q.norm", "l1.mix.g", "l1.ls2", "l2.ls1", "head", "final.norm"} <= names
    assert not {"l2.ls2", "l2.norm2", "l3.mix.vmix", "l1.mix.talk", "l5.mlp.up"} & names


def test_a_config_with_a_missing_or_misfitting_key_is_refused():
    from tokenizer_amd.config import ConfigError, GafonexConfig
    raw = GAFONEX["A"][0]
    GafonexConfig.from_dict(raw)

    def broken(change):
        bad = copy.deepcopy(raw)
        change(bad)
        with pytest.raises(ConfigError):
            GafonexConfig.from_dict(bad)
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18))
    broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"))
    broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5]))
    broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5]))
    broken(lambda c: c["layers"][1]["mixer"].pop("decay"))
    broken(lambda c: c["layers"][2]["mixer"].update(vdim=16))                 # takes in values of another size
    broken(lambda c: c["layers"][2].update(type="latent"))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="moe"))
    broken(lambda c: c["norm"].update(groups=3))
    broken(lambda c: c["norm"].pop("groups"))
    broken(lambda c: c.update(logit_softcap=-1.0))


def test_the_registry_picks_the_design_by_its_config(folders):
    from tokenizer_amd.config import get_architecture, load_config
    cfg = load_config(folders["D"])
    assert cfg.architecture == "Gafonex" and cfg.groups == 3 and len(cfg.layers) == 4
    assert get_architecture("Gafonex").config_class is type(cfg)


@pytest.mark.gpu
def test_the_command_line_generates_from_a_model_folder(folders):
    """Ids in, ids out through the scheduler, and with random weights from the folder's config.json alone."""
    import subprocess
    import sys
    name = "B"
    cfg, tensors = plain.load_folder(folders[name])
    prompt = random_ids(cfg["vocab"], 19, 5)
    want = plain.greedy_generate(cfg, tensors, prompt, 7)
    run = subprocess.run([sys.executable, f"{tt.ROOT}/bin/qwen-infer", "--model", folders[name], "--dtype", "fp32",
                          "--max-tokens", "7", "--token-ids", " ".join(map(str, prompt))],
                         capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr
    assert f"generated ids: {want}" in run.stderr and "stop: MaxTokens" in run.stderr
    run = subprocess.run([sys.executable, f"{tt.ROOT}/bin/qwen-infer", "--model", folders[name], "--random-weights", "3",
                          "--max-tokens", "5", "--token-ids", "1 2 3"], capture_output=True, text=True, timeout=100)
    assert run.returncode == 0 and len(run.stdout.split()) == 5, run.stderr


# ------------------------------------------------------------------ the retention alone
def retention_case(width, heads, d, dv, dims, base, decays, yarn=None):
    from tokenizer_amd.models.gafonex import _retention
    raw = {"heads": heads, "dim": d, "vdim": dv, "decay": list(decays), "rot": {"dims": dims, "base": base}}
    if yarn is not None:
        raw["rot"]["scaling"] = yarn
    return _retention(raw, width, 1e-6, 1 << 20), raw


def retention_tensors(gen, width, heads, d, dv, dtype, size=1.0):
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"q": rand(heads * d, width) * size / width ** 0.5, "k": rand(heads * d, width) * size / width ** 0.5,
         "v": rand(heads * dv, width) / width ** 0.5, "g": rand(heads * dv, width) * size / width ** 0.5,
         "o": rand(width, heads * dv) / (heads * dv) ** 0.5}
    return {name: rounded(t, dtype) for name, t in w.items()}


RETENTION_SIZES = [(48, 2, 16, 24, 8, 100.0, (0.97, 0.9)), (40, 3, 10, 14, 10, 300.0, (0.99, 0.5, 0.999)),
                   (32, 1, 2, 1, 2, 10.0, (0.95,)), (64, 2, 64, 64, 64, 10000.0, (0.99, 0.98)), (64, 1, 128, 128, 32, 500.0, (0.996,)),
                   (32, 2, 33, 70, 4, 50.0, (1.0, 0.0)), (64, 1, 256, 40, 0, 1.0, (0.98,)), (64, 1, 20, 256, 20, 60.0, (0.93,)),
                   (64, 5, 32, 48, 32, 1000.0, (0.9, 0.99, 0.96, 0.7, 0.998))]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("width,heads,d,dv,dims,base,decays", RETENTION_SIZES)
def test_retention_alone(backend, cut, width, heads, d, dv, dims, base, decays):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(heads * 100 + d + dv)
    n = 150
    w = retention_tensors(gen, width, heads, d, dv, dtype, size=1.5)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, m = retention_case(width, heads, d, dv, dims, base, decays)
    want = plain.retention(h, w, m, 1e-6)
    runner = PartRunner("retention", spec, w, backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:9] * 0.5)
    bound = tolerance(dtype, 5e-5, 6e-2)
    if heads * dv < 4:                      # (one value: its unit is its sign, which rounding tips where o passes zero)
        off = ((got - want).abs().amax(-1) > bound * max(1.0, float(want.abs().max())))
        assert int(off.sum()) <= (8 if dtype == torch.bfloat16 else 0)
        return
    assert float((got - want).abs().max()) <= bound * max(1.0, float(want.abs().max()))
    # The slot is given back and taken again: the next request starts from zeros, not from what the last one left.
    runner.end("main")
    runner.end("rider")
    again = runner.run(h[:30] * 0.7, [30], rid="next")
    fresh = plain.retention(h[:30] * 0.7, w, m, 1e-6)
    assert float((again - fresh).abs().max()) <= bound * max(1.0, float(fresh.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,heads,d,dv,dims", [(64, 2, 64, 64, 64), (40, 3, 20, 36, 12), (64, 1, 128, 80, 128)])
def test_long_portions_beside_short_ones(backend, width, heads, d, dv, dims):
    """Portions of hundreds of tokens (no multiples of a chunk) run in chunks side by side whose states are carried from
    one to the next; a second request's portion and a third's single token ride in the same step; then single tokens and
    another long portion go on from the states those left."""
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(d + dv)
    n = 560
    decays = [0.999, 0.99, 0.97][:heads]
    w = retention_tensors(gen, width, heads, d, dv, dtype, size=1.5)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    other = rounded(torch.randn(150, width, generator=gen, dtype=torch.float64), dtype)
    spec, m = retention_case(width, heads, d, dv, dims, 1000.0, decays)
    want, want_other = plain.retention(h, w, m, 1e-6), plain.retention(other, w, m, 1e-6)
    runner = PartRunner("retention", spec, w, backend, num_pages=80)
    runner.step([("third", other[:3])])
    first = runner.step([("other", other), ("third", other[3:4]), ("main", h[:299])])
    rest = runner.run(h[299:], [1, 2, 200, 17] + [1] * 41)
    got = torch.cat([first[2], rest])
    bound = tolerance(dtype, 5e-5, 6e-2)
    assert float((first[0] - want_other).abs().max()) <= bound * max(1.0, float(want_other.abs().max()))
    assert float((first[1] - want_other[3:4]).abs().max()) <= bound * max(1.0, float(want_other.abs().max()))
    assert float((got - want).abs().max()) <= bound * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
def test_a_write_that_is_read_two_hundred_tokens_later(backend, cut):
    """The first tokens' inputs are a hundred times larger than the later ones under decays of nearly one, so the late rows
    are mostly what the state carried all the way, through every cut of the sequence into steps."""
    ops, device, dtype = ops_for(backend)
    width, heads, d, dv, n = 32, 2, 16, 24, 230
    gen = torch.Generator().manual_seed(11)
    w = retention_tensors(gen, width, heads, d, dv, dtype, size=2.0)
    h = torch.randn(n, width, generator=gen, dtype=torch.float64) * 0.05
    h[:3] *= 100.0
    h = rounded(h, dtype)
    spec, m = retention_case(width, heads, d, dv, 16, 10000.0, (0.999, 0.9995))
    want = plain.retention(h, w, m, 1e-6)
    quiet = plain.retention(torch.cat([h[:3] * 0.001, h[3:]]), w, m, 1e-6)
    assert float((want[200:] - quiet[200:]).abs().max()) > 0.5 * float(quiet[200:].abs().max())
    runner = PartRunner("retention", spec, w, backend)
    got = runner.run(h, {"prompt": [n], "portions": [37, 2, 16, 1, 1, 29, 144], "decoded": [20] + [1] * 210}[cut], rider=h[:9])
    assert float((got[200:] - want[200:]).abs().max()) <= tolerance(dtype, 1e-4, 6e-2) * float(want[200:].abs().max())


# ------------------------------------------------------------------ the attention alone
def attention_case(width, heads, kv_heads, d, dv, dims, base, scale, yarn=None, mix=None):
    from tokenizer_amd.models.gafonex import _attention
    raw = {"heads": heads, "kv_heads": kv_heads, "dim": d, "vdim": dv, "scale": scale, "rot": {"dims": dims, "base": base}}
    if yarn is not None:
        raw["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), yarn))
    return _attention(raw, width, 1e-6, 1 << 20, mix), raw


def attention_tensors(gen, width, heads, kv_heads, d, dv, dtype):
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"q": rand(heads * d, width) / width ** 0.5, "k": rand(kv_heads * d, width) / width ** 0.5,
         "v": rand(kv_heads * dv, width) / width ** 0.5, "o": rand(width, heads * dv) / (heads * dv) ** 0.5,
         "q.norm": 1 + 0.3 * rand(d), "k.norm": 1 + 0.3 * rand(d),
         "talk": torch.eye(heads, dtype=torch.float64) * 0.6 + rand(heads, heads) * heads ** -0.5}
    return {name: (t.float().double() if t.dim() == 1 else rounded(t, dtype)) for name, t in w.items()}


def part_names(w):
    from tokenizer_amd.models.gafonex import _ATTENTION_NAMES
    theirs = {file: ours for ours, file in _ATTENTION_NAMES}
    return {theirs.get(name, name): t for name, t in w.items()}


ATTENTION_SIZES = [(48, 4, 2, 16, 24, 8, 10000.0, 0.7, None), (40, 3, 3, 10, 14, 6, 300.0, 0.9, (4.0, 30, 4.0, 1.0)),
                   (32, 1, 1, 24, 40, 2, 100.0, 0.5, None), (64, 4, 1, 64, 64, 32, 500000.0, 0.3, (8.0, 64, 16.0, 1.0)),
                   (64, 8, 2, 32, 32, 32, 10000.0, 0.4, None), (48, 6, 2, 6, 10, 0, 100.0, 0.9, None),
                   (64, 14, 2, 64, 64, 64, 1e6, 0.3, (4.0, 50, 8.0, 1.0)), (64, 6, 1, 48, 16, 48, 10000.0, 0.35, None),
                   (64, 2, 1, 128, 128, 64, 10000.0, 0.25, None), (48, 12, 2, 80, 96, 80, 1000.0, 0.3, None),
                   (64, 20, 4, 32, 48, 32, 100.0, 0.5, None), (64, 24, 4, 16, 128, 16, 100.0, 0.6, None),
                   (64, 16, 8, 32, 80, 32, 100.0, 0.5, None), (64, 40, 2, 16, 16, 16, 100.0, 0.6, None)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("width,heads,kv_heads,d,dv,dims,base,scale,yarn", ATTENTION_SIZES)
def test_talking_attention_alone(backend, cut, width, heads, kv_heads, d, dv, dims, base, scale, yarn):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(heads * 100 + d + dv)
    n = 120
    w = attention_tensors(gen, width, heads, kv_heads, d, dv, dtype)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, m = attention_case(width, heads, kv_heads, d, dv, dims, base, scale, yarn)
    want = plain.talking_attention(h, w, m, 1e-6, None)[0]
    runner = PartRunner("gqa_attention", spec, part_names(w), backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:9] * 0.5)
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 6e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("heads,kv_heads,d,dv", [(14, 2, 64, 64), (6, 3, 24, 20), (28, 4, 32, 32)])
def test_hundreds_of_keys_in_long_portions_and_single_tokens(backend, cut, heads, kv_heads, d, dv):
    """Several blocks of keys, several parts of a long context, portions of several tiles, two requests at a time."""
    ops, device, dtype = ops_for(backend)
    if backend == "cpu":
        pytest.skip("the long walks are for the device's kernels")
    gen = torch.Generator().manual_seed(heads + d)
    n, width = 700, 64
    w = attention_tensors(gen, width, heads, kv_heads, d, dv, dtype)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, m = attention_case(width, heads, kv_heads, d, dv, d // 4 * 2, 1000.0, 0.8 * d ** -0.25)
    want = plain.talking_attention(h, w, m, 1e-6, None)[0]
    cuts = {"prompt": [n], "portions": [150, 2, 333, 17, 1, 197], "decoded": [640] + [1] * 60}[cut]
    runner = PartRunner("gqa_attention", spec, part_names(w), backend, num_pages=100)
    got = runner.run(h, cuts, rider=h[:9] * 0.5)
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 6e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("heads,kv_heads,d,dv", [(2, 1, 16, 8), (4, 2, 32, 32), (3, 1, 24, 40)])
def test_one_key_made_to_stand_out_far_back_and_at_page_borders(backend, cut, heads, kv_heads, d, dv):
    """The mixer's input is [a query part | a key part]: the query projection reads the first half, the key projection
    the second, so a query whose first half is the second half of a chosen token scores that token far above all others
    in every head.  The chosen keys are, in turn: the second token of the sequence (hundreds of tokens back), the keys on
    either side of the last page border, the key before the query, the query itself and the very first token.  All heads'
    softmaxes then lie on that key, so head h's mixed weight is the sum of its row of the table, on that key alone."""
    ops, device, dtype = ops_for(backend)
    n = 230
    gen = torch.Generator().manual_seed(5 + d)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    keys = rand(n, d)
    target = []
    for i in range(n):
        j = [1, i - i % 16, i - i % 16 - 1, i - 1, i, 0][i % 6]
        target.append(j if 0 <= j <= i else i)
    h = rounded(torch.cat([keys[target], keys], dim=1), dtype)
    eye, zero = torch.eye(d, dtype=torch.float64), torch.zeros(d, d, dtype=torch.float64)
    w = {"q": torch.cat([torch.cat([eye, zero], dim=1)] * heads), "k": torch.cat([torch.cat([zero, eye], dim=1)] * kv_heads),
         "v": rounded(rand(kv_heads * dv, 2 * d), dtype), "o": rounded(rand(2 * d, heads * dv) / (heads * dv) ** 0.5, dtype),
         "q.norm": torch.ones(d, dtype=torch.float64), "k.norm": torch.ones(d, dtype=torch.float64),
         "talk": rounded(rand(heads, heads), dtype)}
    spec, m = attention_case(2 * d, heads, kv_heads, d, dv, 0, 100.0, 6.0)
    want = plain.talking_attention(h, w, m, 1e-6, None)[0]
    values = plain.unit_rms((h @ w["v"].T).reshape(n, kv_heads, dv), 1e-6)[target].repeat_interleave(heads // kv_heads, dim=1)
    alone = (values * w["talk"].sum(1)[None, :, None]).reshape(n, heads * dv) @ w["o"].T
    assert float((want - alone).abs().max()) < 1e-2 * float(want.abs().max())
    runner = PartRunner("gqa_attention", spec, part_names(w), backend)
    got = runner.run(h, {"prompt": [n], "portions": [37, 2, 16, 1, 1, 29, 144], "decoded": [160] + [1] * 70}[cut], rider=h[:9])
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 3e-2) * float(want.abs().max())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", ["prompt", "portions"])
def test_heads_that_take_only_from_one_other_head(backend, cut):
    """The mixing table is a permutation: head h's output is the other head's weights on head h's own values."""
    ops, device, dtype = ops_for(backend)
    width, heads, kv_heads, d, dv, n = 48, 6, 3, 16, 16, 90
    gen = torch.Generator().manual_seed(4)
    w = attention_tensors(gen, width, heads, kv_heads, d, dv, dtype)
    order = [3, 5, 0, 4, 1, 2]
    w["talk"] = torch.zeros(heads, heads, dtype=torch.float64)
    for row, column in enumerate(order):
        w["talk"][row, column] = 1.0
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, m = attention_case(width, heads, kv_heads, d, dv, 16, 100.0, 0.8)
    positions = torch.arange(n)
    q = plain.rotate(plain.unit_rms((h @ w["q"].T).reshape(n, heads, d), 1e-6) * w["q.norm"], positions, m["rot"])
    k = plain.rotate(plain.unit_rms((h @ w["k"].T).reshape(n, kv_heads, d), 1e-6) * w["k.norm"], positions, m["rot"])
    v = plain.unit_rms((h @ w["v"].T).reshape(n, kv_heads, dv), 1e-6)
    out = torch.zeros(n, heads, dv, dtype=torch.float64)
    for t in range(n):
        for head in range(heads):
            s = k[:t + 1, order[head] // 2] @ q[t, order[head]] * m["scale"]
            e = torch.exp(s - s.max())
            out[t, head] = (e / e.sum()) @ v[:t + 1, head // 2]
    want = out.reshape(n, heads * dv) @ w["o"].T
    got = PartRunner("gqa_attention", spec, part_names(w), backend).run(h, CUTS[cut](n), rider=h[:5])
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 5e-2) * max(1.0, float(want.abs().max()))


# ------------------------------------------------------------------ the store, the rotation, the norms, the gate
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n_q,n_kv,d,dv,dims", [(4, 2, 16, 24, 12), (3, 3, 10, 14, 10), (14, 2, 64, 64, 64), (1, 1, 2, 3, 2), (2, 1, 130, 300, 40),
                                                (5, 1, 12, 8, 0)])
@pytest.mark.parametrize("takes", [False, True])
def test_head_norms_rotation_and_values_on_their_way_into_the_pages(backend, n_q, n_kv, d, dv, dims, takes):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(d * 10 + dv)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    n, page_size, width = 21, 16, (n_q + n_kv) * d + n_kv * dv
    rows = rounded(rand(n, width + 8), dtype)
    positions = torch.tensor([(7 * i * i) % 3000 for i in range(n)])
    rot = {"dims": dims, "base": 300.0, "scaling": {"factor": 4.0, "original": 100, "fast": 8.0, "slow": 1.0}}
    q_w, k_w = (1 + 0.3 * rand(d)).float().double(), (1 + 0.3 * rand(d)).float().double()
    other, share = rounded(rand(n, n_kv * dv), dtype), torch.tensor([0.3], dtype=torch.float64)
    q = plain.rotate(plain.unit_rms(rows[:, :n_q * d].reshape(n, n_q, d), 1e-5) * q_w, positions, rot)
    k = plain.rotate(plain.unit_rms(rows[:, n_q * d:(n_q + n_kv) * d].reshape(n, n_kv, d), 1e-5) * k_w, positions, rot)
    v = plain.unit_rms(rows[:, (n_q + n_kv) * d:width].reshape(n, n_kv, dv), 1e-5)
    if takes:
        v = 0.7 * v + 0.3 * other.reshape(n, n_kv, dv)
    from tokenizer_amd.parts.position import yarn_rates
    stored = rows.to(dtype).to(device).contiguous()
    table = None
    if dims:
        rates, magnitude = yarn_rates(300.0, dims, rot["scaling"])
        table = ops.rotation_table(positions.to(torch.int32).to(device), rates.to(device), magnitude,
                                   torch.empty((n, dims), dtype=torch.float32, device=device))
    slots = torch.tensor([(5 * i) % 48 if i != 4 else -1 for i in range(n)], dtype=torch.int32)
    k_pages = torch.full((3, n_kv, page_size, d), float("nan"), dtype=dtype, device=device)
    v_pages = torch.full((3, n_kv, dv, page_size), float("nan"), dtype=dtype, device=device)
    wide = torch.zeros((n, n_kv * dv + 16), dtype=dtype, device=device)       # (rows that lie apart)
    wide[:, 8:8 + n_kv * dv] = other.to(dtype).to(device)
    ops.head_norm_rotate_store(stored, table, dims, slots.to(device), k_pages, v_pages, n_q, n_kv, n_kv, d, dv,
                               q_w.float().to(device), k_w.float().to(device), True,
                               wide[:, 8:8 + n_kv * dv] if takes else None, share.float().to(device) if takes else None, 1e-5)
    bound = tolerance(dtype, 2e-4, 3e-2) * 4        # (positions of thousands: an angle in float32 is good to 2e-4)
    got = stored.double().cpu()
    assert float((got[:, :n_q * d] - q.reshape(n, -1)).abs().max()) <= bound
    assert float((got[:, n_q * d:(n_q + n_kv) * d] - k.reshape(n, -1)).abs().max()) <= bound
    assert float((got[:, (n_q + n_kv) * d:width] - v.reshape(n, -1)).abs().max()) <= bound
    assert torch.equal(got[:, width:], rows[:, width:])
    for t in range(n):
        slot = int(slots[t])
        if slot >= 0:
            assert torch.equal(k_pages[slot // 16, :, slot % 16, :].double().cpu().reshape(-1), got[t, n_q * d:(n_q + n_kv) * d])
            assert torch.equal(v_pages[slot // 16, :, :, slot % 16].double().cpu().reshape(-1), got[t, (n_q + n_kv) * d:width])
    assert int(torch.isnan(k_pages[..., 0]).sum()) == n_kv * (48 - (n - 1))      # nothing else was written


@pytest.mark.parametrize("dims,base,yarn", [(40, 7000.0, (6.0, 1000, 24.0, 1.0)), (12, 400.0, (4.0, 40, 6.0, 1.0)), (2, 10.0, (3.0, 16, 2.0, 1.0)),
                                            (64, 500.0, (2.0, 8, 1.0, 1.0)), (16, 100.0, (32.0, 100000, 2.0, 1.0))])
def test_slowed_rates_against_the_oracle(dims, base, yarn):
    """Ramps inside the head, ramps cut at either end, and a ramp of no width."""
    from tokenizer_amd.parts.position import yarn_rates
    scaling = dict(zip(("factor", "original", "fast", "slow"), yarn))
    rates, magnitude = yarn_rates(base, dims, scaling)
    want, size = plain.rotation({"dims": dims, "base": base, "scaling": scaling})
    assert torch.allclose(rates.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-6) and abs(size - magnitude) < 1e-12
    assert abs(magnitude - (0.1 * math.log(yarn[0]) + 1.0)) < 1e-12


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("hidden,post_groups,groups", [(40, 2, 2), (54, 3, 1), (256, 1, 4), (1000, 5, 10), (2304, 2, 2), (5120, 4, 2),
                                                       (9000, 3, 5), (20, 20, 10), (4096, 1024, 2)])
def test_norms_over_groups_behind_a_sublayer_and_before_the_next(backend, hidden, post_groups, groups):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(hidden + groups)
    rows = 7
    stream = torch.randn(rows, hidden, generator=gen).to(device)
    term = (torch.randn(rows, hidden, generator=gen) * torch.linspace(0.2, 3.0, hidden)).to(dtype)     # groups of different size
    w1, w2 = 1 + 0.3 * torch.randn(hidden, generator=gen), 1 + 0.3 * torch.randn(hidden, generator=gen)
    x = stream.double().cpu() + plain.group_norm(term.double(), w1.double(), post_groups, 1e-5)
    y = plain.group_norm(x, w2.double(), groups, 1e-3)
    args = dict(post_groups=post_groups, groups=groups)
    bound = tolerance(dtype, 1e-5, 2e-2)
    kept, out = stream.clone(), torch.empty(rows, hidden, dtype=dtype, device=device)
    ops.norm_add_rmsnorm(kept, term.to(device), w1.to(device), 1e-5, w2.to(device), 1e-3, out, **args)
    assert float((kept.double().cpu() - x).abs().max()) <= 1e-5 * max(1.0, float(x.abs().max()))
    assert float((out.double().cpu() - y).abs().max()) <= bound * max(1.0, float(y.abs().max()))
    kept = stream.clone()
    ops.norm_add_rmsnorm(kept, term.to(device), w1.to(device), 1e-5, None, 0.0, out, **args)           # the sum itself
    assert float((out.double().cpu() - x).abs().max()) <= bound * max(1.0, float(x.abs().max()))
    pick = torch.tensor([6, 0, 3], dtype=torch.int32, device=device)                                   # some rows, nothing stored
    kept, some = stream.clone(), torch.empty(3, hidden, dtype=dtype, device=device)
    ops.norm_add_rmsnorm(kept, term.to(device), w1.to(device), 1e-5, w2.to(device), 1e-3, some, pick, store_residual=False, **args)
    assert torch.equal(kept, stream)
    assert float((some.double().cpu() - y[[6, 0, 3]]).abs().max()) <= bound * max(1.0, float(y.abs().max()))
    ops.norm_add_rmsnorm(kept, None, None, 0.0, w2.to(device), 1e-3, out, **args)                      # nothing to add
    want = plain.group_norm(stream.double().cpu(), w2.double(), groups, 1e-3)
    assert float((out.double().cpu() - want).abs().max()) <= bound * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,ff,rows", [(48, 40, 33), (52, 30, 5), (128, 96, 300), (64, 24, 1), (40, 50, 20)])
def test_the_relu_gated_layer(backend, width, ff, rows):
    from tokenizer_amd.models.gafonex import _FEED_FORWARD_NAMES
    from tokenizer_amd.parts import FEED_FORWARDS, FeedForwardSpec, Runtime
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(ff)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"gate": rounded(rand(ff, width) / width ** 0.5, dtype), "up": rounded(rand(ff, width) / width ** 0.5, dtype),
         "down": rounded(rand(width, ff) / ff ** 0.5, dtype)}
    h = rounded(rand(rows, width), dtype)
    want = plain.relu_gated(h, w)
    spec = FeedForwardSpec("gated_dense", hidden_size=width, intermediate_size=ff, activation="relu")
    stored = {ours: w[theirs].to(dtype).to(device).contiguous() for ours, theirs in _FEED_FORWARD_NAMES}
    part = FEED_FORWARDS.get("gated_dense")(spec, stored, Runtime(dtype, device, ops))
    got = part.forward(h.to(dtype).to(device).contiguous(), None).double().cpu()
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 3e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.gpu
def test_replayed_steps_compute_what_eager_steps_compute(folders):
    """The same decode and mixed steps with graphs (every shape several times, so that it is captured and replayed) and
    without: equal bit for bit."""
    from tokenizer_amd.engine import StepEntry
    got = {}
    for graphs in (False, True):
        eng = make_engine(folders["C"], "gpu-bfloat16", num_pages=60, max_requests=4)
        eng.use_graphs = graphs
        eng.model.decoder.runtime.ops.EAGER_LIBRARY_WORK, kept = 0, eng.model.decoder.runtime.ops.EAGER_LIBRARY_WORK
        try:
            rows = []
            for rid, n in (("a", 70), ("b", 33)):
                eng.add_request(rid)
                rows.append(eng.step([StepEntry(rid, random_ids(200, n, n), [n - 1])]).cpu())
            for k in range(12):
                ids = random_ids(200, 2, k)
                rows.append(eng.step([StepEntry("a", ids[:1], [0]), StepEntry("b", ids[1:], [0])]).cpu())
            eng.add_request("c")
            for k in range(8):
                ids = random_ids(200, 18, 100 + k)
                rows.append(eng.step([StepEntry("a", ids[:1], [0]), StepEntry("c", ids[1:], [16])]).cpu())
            got[graphs] = torch.cat(rows)
        finally:
            eng.model.decoder.runtime.ops.EAGER_LIBRARY_WORK = kept
    assert torch.equal(got[False], got[True])
