"""Zeridra through the framework against the plain implementation of tests/plain/zeridra_plain.py.

Every test runs on three backends: the engine on the CPU with the plain torch ops standing in for the kernel
library (the host side: tables, slots, borrowed pages, batching), and the engine on the GPU in float32 and in bfloat16
(the HIP kernels).  The models are the tiny ones of zeridra_configs.py with sharpened weights; the mechanisms alone
run as the framework's own parts (the registered mixers and feed-forward) over a cache manager and pools of their own.
"""
import copy

import pytest
import torch

import trace_tools as tt
from plain import zeridra_plain as plain
from test_bokulorn import BACKENDS, CUTS, PartRunner, make_engine, ops_for, rounded, tolerance
from tiny_configs import random_ids
from zeridra_configs import ZERIDRA, random_config, write_model

# float32: sums in another order.  bfloat16: the bound is on each row's root mean square error against the row's own
# spread; a lost key, a window one token off or a sink left out moves a row by a good part of its spread, and float32
# pins the same kernels' indexing to five digits.
TOL = {"cpu": 2e-5, "gpu-float32": 1e-4, "gpu-bfloat16": 0.15}


def close(got, want, backend, what=""):
    got = got.float().cpu()
    if backend == "gpu-bfloat16":
        spread = (want - want.mean(dim=-1, keepdim=True)).pow(2).mean(dim=-1).sqrt()
        off = (got - want).pow(2).mean(dim=-1).sqrt() / spread
        # (A router's scores for two experts are now and then nearly equal; bfloat16 rounding then picks the other
        # expert, and that row, and the rows behind it that read it through the cache, move by a good part of their
        # spread.  Such rows are few.)
        assert int((off > TOL[backend]).sum()) <= max(2, off.numel() // 10) and float(off.median()) <= TOL[backend] / 2, \
            f"{what}: rows are off by up to {float(off.max())} of their spread, {int((off > TOL[backend]).sum())} over the bound"
        return
    err = float((got - want).abs().max())
    bound = TOL[backend] * max(float(want.abs().max()), 1.0)
    assert err <= bound, f"{what}: max abs error {err} against a bound of {bound}"


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("zeridra")
    return {name: write_model(raw, seed, str(root / name)) for name, (raw, seed) in ZERIDRA.items()}


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
    vocab = ZERIDRA[name][0]["vocab"]
    return {f"r{i}": random_ids(vocab, n, 40 + i) for i, n in enumerate(lengths)}


def check_trace(folders, oracle, name, backend, steps, reqs, **kw):
    eng = make_engine(folders[name], backend, max_tokens=tt.peak_tokens(steps), max_requests=4, **kw)
    eng.pools.poison()          # pages that no request wrote read as NaN
    got = tt.run_in_process(eng, steps)
    for rid, ids in reqs.items():
        close(got[rid], oracle(name, ids), backend, rid)
    eng.cache.check_invariants()
    assert not eng.cache.requests
    return eng


NAMES = list(ZERIDRA)


# ------------------------------------------------------------------ whole models through the engine
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts_and_the_first_tokens(folders, oracle, name, backend):
    reqs = requests_for(name)
    check_trace(folders, oracle, name, backend, tt.whole(reqs), reqs)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(folders, oracle, name, backend):
    # The tail of 50 passes page borders of 16 and every window's edge; a request of 51 starts decoding behind its first token.
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
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_long_decoding(folders, oracle, name, backend):
    ids = random_ids(ZERIDRA[name][0]["vocab"], 230, 77)
    eng = check_trace(folders, oracle, name, backend, tt.decode_tail({"long": ids}, tail=227), {"long": ids})
    assert any(group.need.kind == "window" for group in eng.cache.groups)


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
@pytest.mark.parametrize("name", ["C", "A"])
def test_hundreds_of_tokens(folders, oracle, dtype, cut, name):
    """Prompts long enough for the prompt kernels' tiles and for routed layers over sorted tokens."""
    reqs = requests_for(name, (300, 17, 411, 130))
    steps = {"whole": lambda: tt.whole(reqs), "tail": lambda: tt.decode_tail(reqs, 40),
             "portions": lambda: tt.portions(reqs, 11), "mixed": lambda: tt.mixed(reqs, 12, max_live=4, tail=10)}[cut]()
    check_trace(folders, oracle, name, f"gpu-{dtype}", steps, reqs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cut", ["whole", "tail"])
def test_a_prompt_of_thirteen_hundred_tokens(folders, oracle, dtype, cut):
    reqs = requests_for("C", (1300,))
    steps = tt.whole(reqs) if cut == "whole" else tt.decode_tail(reqs, 20)
    check_trace(folders, oracle, "C", f"gpu-{dtype}", steps, reqs)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["A", "C"])
def test_replayed_steps_compute_what_eager_steps_compute(folders, name):
    """Every step recorded at first sight and replayed, bit for bit against an engine that records nothing."""
    reqs = requests_for(name, (40, 61, 18))
    steps = tt.mixed(reqs, 5, max_live=3, tail=12) + tt.decode_tail({"again": random_ids(ZERIDRA[name][0]["vocab"], 50, 3)}, 40)
    for at, step in enumerate(steps):
        step["step"] = at
    got = []
    for graphs in (False, True):
        eng = make_engine(folders[name], "gpu-bfloat16", num_pages=40, max_requests=4, use_graphs=graphs)
        eng.GRAPH_AFTER = 1
        eng.model.runtime.ops.EAGER_LIBRARY_WORK = 0        # (eager products of many rows take the route recorded ones take)
        try:
            got.append(tt.run_in_process(eng, steps))
        finally:
            del eng.model.runtime.ops.EAGER_LIBRARY_WORK
        assert eng.model.decoder.graph_safe and (eng.steps_replayed > 0) == graphs
    for rid in got[0]:
        assert torch.equal(got[0][rid], got[1][rid]), rid


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_replay_program_on_a_model_folder(folders, oracle, tmp_path, dtype):
    name = "B"
    reqs = requests_for(name, (40, 23, 5, 64, 31))
    steps = tt.mixed(reqs, 9, max_live=4, tail=6)
    got = tt.run_program(folders[name], dtype, steps, str(tmp_path / "out"), tt.peak_tokens(steps), ZERIDRA[name][0]["vocab"])
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
    """Each mechanism left out of the oracle, or one step off, moves its logits far beyond the tests' bounds."""
    cfg, tensors = plain.load_folder(folders["A"])
    ids = random_ids(cfg["vocab"], 60, 8)
    right = plain.forward(cfg, tensors, ids)
    spread = float((right - right.mean(-1, keepdim=True)).pow(2).mean().sqrt())

    def moved(change_cfg=None, change=None):
        c, t = copy.deepcopy(cfg), dict(tensors)
        if change_cfg:
            change_cfg(c)
        if change:
            t.update(change(t))
        return float((plain.forward(c, t, ids)[40:] - right[40:]).pow(2).mean().sqrt()) / spread
    assert moved(change=lambda t: {n: v - 30 for n, v in t.items() if n.endswith(".sink")}) > 0.02
    assert moved(change=lambda t: {n: 0 * v + 1 for n, v in t.items() if n.endswith((".ls1", ".ls2"))}) > 0.1
    assert moved(change=lambda t: {n: 0 * v + 1 for n, v in t.items() if n.endswith("dkv.norm")}) > 0.05
    assert moved(lambda c: [c["layers"][i]["mixer"]["mask"].update(size=c["layers"][i]["mixer"]["mask"]["size"] + 1)
                            for i in (1, 3, 4, 5)]) > 0.02
    assert moved(lambda c: c["layers"][0]["mixer"]["q_temp"].update(coef=0.0)) > 0.02
    assert moved(lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=12)) > 1e-3
    assert moved(lambda c: [c["layers"][i]["mixer"]["rot"].update(base=100.0) for i in (1, 3, 5)]) > 0.02
    assert moved(lambda c: c.pop("logit_softcap")) > 1e-3
    assert moved(lambda c: c.update(logit_scale=1.0)) > 0.1


# ------------------------------------------------------------------ configuration, registry
def test_the_spec_says_whose_latents_a_layer_reads_and_how_long_they_are_kept():
    from tokenizer_amd.config import ZeridraConfig
    from tokenizer_amd.models.zeridra import zeridra_spec
    from tokenizer_amd.parts import cache_needs, expected_tensors
    spec = zeridra_spec(ZeridraConfig.from_dict(ZERIDRA["A"][0]))
    assert [entry.cache_of for entry in spec.schedule] == [None, None, None, 1, None, 1]
    assert [layer.mixer.window for layer in spec.layers] == [None, 18, None, 36, 32, 4]
    needs = cache_needs(spec)
    assert [need.kind for need in needs] == ["full", "window", "full", "none", "window", "none"]
    assert needs[1].window == 36 and needs[1].head_dim == 48 and needs[4].window == 32     # layer 3 looks further back than layer 1
    names = set(expected_tensors(spec))
    assert {"l0.mix.q", "l0.mix.k", "l1.mix.dkv", "l1.mix.sink", "l3.mix.uk", "l3.mix.sink", "l2.ls1", "l0.ls2", "head"} <= names
    assert not {"l0.mix.v", "l3.mix.dkv", "l3.mix.dkv.norm", "l2.ls2", "l0.mix.sink", "l0.norm2", "l0.mlp.correction"} & names


def test_a_config_with_a_missing_or_misfitting_key_is_refused():
    from tokenizer_amd.config import ConfigError, ZeridraConfig
    raw = ZERIDRA["A"][0]
    ZeridraConfig.from_dict(raw)

    def broken(change):
        bad = copy.deepcopy(raw)
        change(bad)
        with pytest.raises(ConfigError):
            ZeridraConfig.from_dict(bad)
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][0]["mixer"].update(vdim=8))
    broken(lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=0))
    broken(lambda c: c["layers"][1]["mixer"].pop("q_rank"))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6))
    broken(lambda c: c["layers"][1]["mixer"]["mask"].update(size=0))
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=3))
    broken(lambda c: c["layers"][3]["mixer"].update(kv_from=0))                # an attention layer keeps no latents
    broken(lambda c: c["layers"][5]["mixer"].update(kv_from=3))                # layer 3 keeps none of its own
    broken(lambda c: c["layers"][3]["mixer"].update(kv_rank=32))
    broken(lambda c: c["layers"][3]["mixer"]["rot"].update(base=99.0))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda c: c["layers"][2].update(type="retention"))
    broken(lambda c: c["norm"].pop("eps"))
    broken(lambda c: c.update(logit_softcap=-1.0))


def test_the_registry_picks_the_design_by_its_config(folders):
    from tokenizer_amd.config import get_architecture, load_config
    cfg = load_config(folders["D"])
    assert cfg.architecture == "Zeridra" and cfg.logit_softcap is None and len(cfg.layers) == 4
    assert get_architecture("Zeridra").config_class is type(cfg)


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


# ------------------------------------------------------------------ the latent attention alone
def latent_case(width, heads, d, e, dv, q_rank, kv_rank, window, scale, base, eps, own=True, kept_window=None):
    from tokenizer_amd.parts import MixerSpec
    raw = {"heads": heads, "dim": d, "rot_dim": e, "vdim": dv, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
           "mask": {"size": window}, "rot": {"dims": e, "base": base}}
    spec = MixerSpec("latent_attention", hidden_size=width, n_heads=heads, n_kv_heads=1, head_dim=d, value_dim=dv, scale=scale,
                     q_rank=q_rank, kv_rank=kv_rank, rot_dim=e, window=window - 1, sink=True, own_kv=own, eps=eps,
                     options={"rot_base": base, "rot_pairs": "neighbours",
                              "kept_window": window - 1 if kept_window is None else kept_window})
    return spec, raw


def latent_tensors(gen, width, heads, d, e, dv, q_rank, kv_rank, dtype, size=1.0, own=True):
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"dq": rand(q_rank, width) * size / width ** 0.5, "dq.norm": 1 + 0.3 * rand(q_rank),
         "uq": rand(heads * (d + e), q_rank) * size / q_rank ** 0.5,
         "uk": rand(heads * d, kv_rank) * size / kv_rank ** 0.5, "uv": rand(heads * dv, kv_rank) / kv_rank ** 0.5,
         "sink": 1.5 * rand(heads), "o": rand(width, heads * dv) / (heads * dv) ** 0.5}
    if own:
        w.update({"dkv": rand(kv_rank + e, width) * size / width ** 0.5, "dkv.norm": 1 + 0.3 * rand(kv_rank)})
    return {name: (t.float().double() if t.dim() == 1 else rounded(t, dtype)) for name, t in w.items()}


LATENT_SIZES = [(48, 4, 16, 8, 24, 24, 40, 33, 0.3, 10000.0), (40, 3, 10, 6, 14, 20, 22, 7, 0.35, 300.0), (32, 1, 24, 2, 40, 16, 30, 1, 0.2, 100.0),
                (64, 2, 32, 16, 32, 48, 112, 64, 0.18, 500000.0), (64, 2, 16, 32, 16, 32, 288, 50, 0.2, 10000.0),
                (64, 16, 16, 16, 16, 40, 48, 96, 0.25, 1000.0), (64, 20, 8, 8, 8, 24, 24, 17, 0.4, 5000.0),
                (64, 2, 16, 16, 16, 32, 48, 500, 0.3, 100.0)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("width,heads,d,e,dv,q_rank,kv_rank,window,scale,base", LATENT_SIZES)
def test_latent_attention_with_a_window_and_a_sink_alone(backend, cut, width, heads, d, e, dv, q_rank, kv_rank, window, scale, base):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(heads * 100 + d + kv_rank)
    n, eps = 150, 1e-5
    w = latent_tensors(gen, width, heads, d, e, dv, q_rank, kv_rank, dtype, size=2.0)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, raw = latent_case(width, heads, d, e, dv, q_rank, kv_rank, window, scale, base, eps)
    want = plain.latent_attention(h, raw, w, eps, plain.latent_pair(h, raw, w, eps))
    runner = PartRunner("latent_attention", spec, w, backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:9] * 0.5)
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 5e-2) * max(1.0, float(want.abs().max()))
    # The sink takes part, and so do the positions where a query sees more than itself.
    w["sink"] = w["sink"] - 40
    assert float((plain.latent_attention(h, raw, w, eps, plain.latent_pair(h, raw, w, eps)) - want).abs().max()) > 0.05


class BorrowedRunner(PartRunner):
    """A latent mixer that keeps its rows and one that reads them, run one after the other on the same step."""

    def __init__(self, owner, owner_tensors, reader, reader_tensors, backend, **kw):
        from tokenizer_amd.parts import MIXERS, LayerCache, Runtime
        super().__init__("latent_attention", owner, owner_tensors, backend, **kw)
        assert MIXERS.get("latent_attention").cache_need(reader).kind == "none"
        stored = {n: t.to(torch.float32 if t.dim() == 1 else self.dtype).to(self.device).contiguous() for n, t in reader_tensors.items()}
        first, second = self.part, MIXERS.get("latent_attention")(reader, stored, Runtime(self.dtype, self.device, self.ops))
        theirs = LayerCache(group=self.cache.group, k_pages=self.cache.k_pages, v_pages=self.cache.v_pages, writes=False)

        class Both:
            @staticmethod
            def forward(x, ctx, cache):
                first.forward(x, ctx, cache)
                return second.forward(x, ctx, theirs)
        self.part = Both


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("own_window,window", [(9, 40), (33, 12), (1, 64), (500, 17)])
def test_a_layer_that_reads_anothers_latents(backend, cut, own_window, window):
    """Other heads, sizes and another window than the layer that keeps them; pages behind the wider window are given back."""
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(own_window + window)
    width, e, kv_rank, base, n, eps = 48, 8, 40, 2000.0, 150, 1e-6
    kept = max(own_window, window) - 1
    first, first_raw = latent_case(width, 3, 16, e, 8, 24, kv_rank, own_window, 0.3, base, eps, kept_window=kept)
    second, second_raw = latent_case(width, 4, 12, e, 20, 32, kv_rank, window, 0.35, base, eps, own=False)
    w1 = latent_tensors(gen, width, 3, 16, e, 8, 24, kv_rank, dtype, size=2.0)
    w2 = latent_tensors(gen, width, 4, 12, e, 20, 32, kv_rank, dtype, size=2.0, own=False)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    want = plain.latent_attention(h, second_raw, w2, eps, plain.latent_pair(h, first_raw, w1, eps))
    runner = BorrowedRunner(first, w1, second, w2, backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:9] * 0.5)
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 5e-2) * max(1.0, float(want.abs().max()))
    given_back = sum(1 for page in runner.manager.table("main", 0) if page < 0)
    assert (given_back > 0) == (kept < 130)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("window", [2, 16, 17, 31, 64, 81])
def test_one_latent_made_to_stand_out_just_inside_and_just_outside_the_window(backend, cut, window):
    """The mixer's input is [a query part | a key part]: the query latent reads the first half, the key latent the
    second, and both go up through the same matrix, so a query whose first half is the second half of a chosen token
    scores that token far above all others.  The chosen tokens are, in turn: the last one inside the window, the first
    one outside it, the query itself, the keys on either side of the last page border."""
    ops, device, dtype = ops_for(backend)
    half, heads, dv, e, n, eps = 16, 2, 8, 4, 230, 1e-6
    gen = torch.Generator().manual_seed(5 + window)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    keys = rand(n, half)
    keys = keys / keys.norm(dim=-1, keepdim=True)
    target = []
    for i in range(n):
        j = [i - window + 1, i - window, i, i - window + 1, i - window, i - i % 16, i - i % 16 - 1][i % 7]
        target.append(j if 0 <= j <= i else i)
    h = rounded(torch.cat([keys[target], keys], dim=1), dtype)
    up = torch.linalg.qr(rand(half, half))[0]
    eye, zero = torch.eye(half, dtype=torch.float64), torch.zeros(half, half, dtype=torch.float64)
    w = {"dq": torch.cat([eye, zero], dim=1), "dq.norm": torch.ones(half, dtype=torch.float64),
         "uq": torch.cat([torch.cat([up, 0.02 * rand(e, half)]) for _ in range(heads)]),
         "dkv": torch.cat([torch.cat([zero, eye], dim=1), 0.3 * rand(e, 2 * half)]), "dkv.norm": torch.ones(half, dtype=torch.float64),
         "uk": torch.cat([up] * heads), "uv": rand(heads * dv, half), "sink": torch.tensor([3.0, -2.0], dtype=torch.float64),
         "o": torch.cat([torch.eye(heads * dv, dtype=torch.float64), torch.zeros(2 * half - heads * dv, heads * dv, dtype=torch.float64)])}
    w = {name: (t if t.dim() == 1 else rounded(t, dtype)) for name, t in w.items()}
    spec, raw = latent_case(2 * half, heads, half, e, dv, half, half, window, 1.5, 100.0, eps)
    want = plain.latent_attention(h, raw, w, eps, plain.latent_pair(h, raw, w, eps))
    runner = PartRunner("latent_attention", spec, w, backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:7])
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 5e-2) * float(want.abs().max())
    # A window that is one token off, either way, moves the rows that chose the token at its edge by far more.
    for other, chosen in ((window - 1, 1), (window + 1, 0)):
        off = plain.latent_attention(h, dict(raw, mask={"size": other}), w, eps, plain.latent_pair(h, raw, w, eps))
        rows = [i for i in range(window + 8, n) if target[i] == i - window + chosen]
        assert len(rows) > 20 and float((off[rows] - want[rows]).abs().max(dim=-1).values.median()) > 0.2


# ------------------------------------------------------------------ the attention whose values are the keys alone
def attention_case(width, heads, kv_heads, d, scale, coef, every, eps=1e-6):
    from tokenizer_amd.models.zeridra import _attention
    raw = {"heads": heads, "kv_heads": kv_heads, "dim": d, "vdim": d, "scale": scale, "q_temp": {"coef": coef, "every": every}}
    return _attention(raw, width, eps), raw


def attention_tensors(gen, width, heads, kv_heads, d, dtype, size=1.0):
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"q": rand(heads * d, width) * size / width ** 0.5, "k": rand(kv_heads * d, width) * size / width ** 0.5,
         "o": rand(width, heads * d) / (heads * d) ** 0.5}
    return {name: rounded(t, dtype) for name, t in w.items()}


def named(w):
    return {{"q": "q_proj.weight", "k": "k_proj.weight", "o": "o_proj.weight"}[name]: t for name, t in w.items()}


ATTENTION_SIZES = [(48, 4, 2, 16, 0.3, 0.4, 11), (40, 3, 3, 10, 0.4, 0.5, 7), (32, 1, 1, 20, 0.3, 0.2, 1), (64, 12, 2, 64, 0.12, 0.3, 50),
                   (64, 8, 1, 128, 0.09, 0.1, 16), (64, 5, 1, 80, 0.1, 1.0, 100), (64, 20, 1, 48, 0.15, 0.3, 33), (64, 2, 2, 256, 0.06, 0.0, 8),
                   (64, 4, 2, 300, 0.05, 0.3, 20), (56, 6, 3, 12, 0.3, 0.7, 3)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("width,heads,kv_heads,d,scale,coef,every", ATTENTION_SIZES)
def test_attention_whose_values_are_the_keys_alone(backend, cut, width, heads, kv_heads, d, scale, coef, every):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(heads * 100 + d)
    n = 150
    w = attention_tensors(gen, width, heads, kv_heads, d, dtype, size=1.5)
    h = rounded(torch.randn(n, width, generator=gen, dtype=torch.float64), dtype)
    spec, raw = attention_case(width, heads, kv_heads, d, scale, coef, every)
    want = plain.attention(h, raw, w)
    runner = PartRunner("gqa_attention", spec, named(w), backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:9] * 0.5)
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 5e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("d,every", [(16, 16), (64, 30), (128, 61)])
def test_one_key_made_to_stand_out_far_back_and_the_one_in_the_denominator(backend, cut, d, every):
    """Keys are scaled unit vectors and queries point at a chosen one: the second token, the keys on either side of the last page
    border, the key before, the query itself; every fifth query points away from every key (all scores far below 0, so
    nearly all of its weight goes to the one that the denominator has and its output is near zero)."""
    ops, device, dtype = ops_for(backend)
    heads, kv_heads, n = 2, 1, 230
    gen = torch.Generator().manual_seed(d)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    keys = rand(n, d)
    keys = 2.0 * keys / keys.norm(dim=-1, keepdim=True) + 0.8 / d ** 0.5 * torch.ones(d, dtype=torch.float64)
    target, sign = [], []
    for i in range(n):
        j = [1, i - i % 16, 0, i - i % 16 - 1, i - 1, i][i % 6]
        target.append(j if 0 <= j <= i else i)
        sign.append(1.0)
    q = keys[target].clone()
    away = list(range(4, n, 5))
    q[away] = -4.0 / d ** 0.5
    h = rounded(torch.cat([q, keys], dim=1), dtype)
    eye, zero = torch.eye(d, dtype=torch.float64), torch.zeros(d, d, dtype=torch.float64)
    w = {"q": torch.cat([torch.cat([eye, zero], dim=1), torch.cat([0.5 * eye, zero], dim=1)]), "k": torch.cat([zero, eye], dim=1),
         "o": torch.eye(2 * d, dtype=torch.float64)}
    spec, raw = attention_case(2 * d, heads, kv_heads, d, 2.5, 0.35, every)
    want = plain.attention(h, raw, w)
    runner = PartRunner("gqa_attention", spec, named(w), backend)
    got = runner.run(h, CUTS[cut](n), rider=h[:7])
    assert float((got - want).abs().max()) <= tolerance(dtype, 3e-5, 4e-2) * float(want.abs().max())
    # The second token's key does carry the rows that chose it, and the denominator's one the rows that look away.
    blind = h.clone()
    blind[1, d:] = -blind[1, d:]
    rows = [i for i in range(40, n) if target[i] == 1 and i not in away]
    assert len(rows) > 15 and float((plain.attention(blind, raw, w)[rows] - want[rows]).abs().max(dim=-1).values.min()) > 0.2
    T = h.shape[0]
    with_sink = plain.softmax_with_sink(torch.full((1, T, T), -6.0, dtype=torch.float64), torch.zeros(1, dtype=torch.float64), plain.visible(T))
    assert float(with_sink[0, 0, 0]) < 0.01 and float(want[away].abs().max()) < 0.5 * float(want.abs().max())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n_q,n_k,d,dv,tied,stride", [(4, 2, 16, 16, True, 0), (3, 3, 10, 10, True, 2), (5, 1, 64, 64, True, 0), (2, 2, 24, 40, False, 8),
                                                       (40, 8, 64, 64, True, 0), (3, 1, 12, 20, False, 0)])
@pytest.mark.parametrize("coef,every", [(0.3, 5), (0.0, 1), (1.5, 1), (-0.1, 1000)])
def test_the_query_temperature_and_the_store(backend, n_q, n_k, d, dv, tied, stride, coef, every):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(n_q * 10 + d)
    n, page_size = 23, 16
    used = (n_q + n_k) * d + (0 if tied else n_k * dv)
    x = torch.randn(n, used + stride, generator=gen).to(dtype)
    positions = torch.tensor([0, 1, every - 1, every, 2 * every - 2, 2 * every - 1, 4095, 70000] + list(range(100, 115)), dtype=torch.int32)
    slots = torch.randperm(64, generator=gen)[:n].to(torch.int32)
    slots[3] = -1
    k_pages = torch.full((4, n_k, page_size, d), 7.0, dtype=dtype, device=device)
    v_pages = torch.full((4, n_k, dv, page_size), 7.0, dtype=dtype, device=device)
    qkv = x.clone().to(device)
    ops.temper_store(qkv, positions.to(device), coef, every, slots.to(device), k_pages, v_pages, n_q, n_k, d, dv, tied)
    factor = plain.temperature(positions.long(), coef, every)
    want_q = x[:, :n_q * d].double() * factor[:, None]
    got = qkv.double().cpu()
    assert float((got[:, :n_q * d] - want_q).abs().max()) <= (1e-5 if dtype == torch.float32 else 2 ** -8) * float(want_q.abs().max())
    assert torch.equal(got[:, n_q * d:], x[:, n_q * d:].double())                        # everything behind the queries stays
    keys = x[:, n_q * d:(n_q + n_k) * d].reshape(n, n_k, d)
    values = keys if tied else x[:, (n_q + n_k) * d:used].reshape(n, n_k, dv)
    want_k, want_v = torch.full((4, n_k, page_size, d), 7.0, dtype=dtype), torch.full((4, n_k, dv, page_size), 7.0, dtype=dtype)
    for t, slot in enumerate(slots.tolist()):
        if slot >= 0:
            want_k[slot // page_size, :, slot % page_size] = keys[t]
            want_v[slot // page_size, :, :, slot % page_size] = values[t]
    assert torch.equal(k_pages.cpu(), want_k) and torch.equal(v_pages.cpu(), want_v)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("rot,heads", [(2, 1), (6, 3), (16, 5), (64, 2)])
def test_the_rotation_of_neighbours(backend, rot, heads):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(rot)
    n, head_width, plain_dims = 11, rot + 5, 5
    q = torch.randn(n, heads * head_width, generator=gen).to(dtype)
    positions = torch.tensor([0, 1, 2, 3, 15, 16, 17, 100, 1000, 5000, 100000], dtype=torch.int32)
    rates = torch.tensor([300.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float()
    out = torch.zeros(n, heads * (rot + 3), dtype=dtype, device=device)
    ops.rotate_tails(q.to(device), heads, head_width, plain_dims, rot, rates.to(device), positions.to(device), out, rot + 3, 3, neighbours=True)
    x = q.reshape(n, heads, head_width)[..., plain_dims:].double()
    want = plain.turn_neighbours(x, positions.long(), 300.0)
    got = out.double().cpu().reshape(n, heads, rot + 3)
    assert float(got[..., :3].abs().max()) == 0.0
    # (Angles are float32 products: at position 100,000 that is an error of 2^-8 of a radian at most.)
    assert float((got[:, :, 3:] - want)[:9].abs().max()) <= (1e-3 if dtype == torch.float32 else 3e-2)
    assert float((got[:, :, 3:] - want).abs().max()) <= 6e-2


# ------------------------------------------------------------------ router and experts alone
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width,tokens", [(6, 2, 64, 37), (1, 1, 40, 5), (12, 1, 52, 80), (64, 6, 128, 70), (300, 4, 64, 9), (9, 9, 48, 20)])
def test_the_router_whose_scores_are_the_weights(backend, experts, top, width, tokens):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(experts + top)
    x = rounded(torch.randn(tokens, width, generator=gen, dtype=torch.float64), dtype)
    router = rounded(torch.randn(experts, width, generator=gen, dtype=torch.float64) * 0.4, dtype)
    s = torch.sigmoid(x @ router.T)
    best = torch.topk(s, top, dim=-1)
    on = lambda t: t.to(dtype).to(device).contiguous()

    def check(chosen, weights):
        chosen, weights = chosen.long().cpu(), weights.double().cpu()
        picked = torch.gather(s, 1, chosen)
        assert all(len(set(row)) == top for row in chosen.tolist())
        assert float((picked - best.values).abs().max()) <= 1e-5                     # (near ties may come in either order)
        assert float((weights - picked).abs().max()) <= 1e-5
    chosen = torch.empty((tokens, top), dtype=torch.int32, device=device)
    weights = torch.empty((tokens, top), dtype=torch.float32, device=device)
    ops.route_scores(ops.linear(on(x), on(router), out_dtype=torch.float32), None, experts, 0, 0, chosen, weights, renormalize=False)
    check(chosen, weights)
    fused = getattr(ops, "route_rows_scores", None)
    if fused is not None:
        chosen.fill_(-1)
        if fused(on(x), on(router), None, experts, 0, 0, chosen, weights, renormalize=False):
            check(chosen, weights)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,inner,width,tokens", [(6, 2, 24, 64, 37), (1, 1, 10, 52, 9), (12, 1, 32, 128, 50), (8, 3, 16, 64, 3), (16, 1, 40, 64, 600),
                                                            (8, 4, 32, 64, 300), (24, 1, 16, 64, 1), (24, 2, 48, 64, 16), (5, 2, 12, 40, 200),
                                                            (12, 1, 24, 64, 44)])
def test_the_routed_experts_with_weighted_inputs(backend, experts, top, inner, width, tokens):
    """In the form that multiplies every expert, over sorted tokens, and for few rows; a weight on the output instead of the input
    would give other rows (checked in the oracle)."""
    from tokenizer_amd.parts import FEED_FORWARDS, FeedForwardSpec, Runtime
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(experts * 10 + tokens)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    w = {"router": rand(experts, width) * 0.12}
    for j in range(experts):
        w.update({f"e{j}.gate": 2 * rand(inner, width) / width ** 0.5, f"e{j}.up": 2 * rand(inner, width) / width ** 0.5,
                  f"e{j}.down": rand(width, inner) / inner ** 0.5})
    w = {name: rounded(t, dtype) for name, t in w.items()}
    x = rounded(rand(tokens, width), dtype)
    mlp = {"router": {"experts": experts, "top": top}}
    want = plain.routed_feed_forward(x, mlp, w)
    spec = FeedForwardSpec("routed_experts", hidden_size=width, intermediate_size=inner, n_experts=experts, top_k=top,
                           router="sigmoid", correction=False, renormalize=False, weigh_input=True)
    part = FEED_FORWARDS.get("routed_experts")(spec, {n: t.to(dtype).to(device) for n, t in w.items()}, Runtime(dtype, device, ops))
    got = part.forward(x.to(dtype).to(device), None).double().cpu()
    # (A near tie between the last chosen and the first passed over may go either way under rounding: such rows are left out.)
    z = torch.sort(x @ w["router"].T, dim=-1, descending=True).values
    sure = torch.ones(tokens, dtype=torch.bool) if top == experts else (z[:, top - 1] - z[:, top]) > 1e-4
    assert int(sure.sum()) >= tokens - 2
    assert float((got - want)[sure].abs().max()) <= tolerance(dtype, 3e-5, 3e-2) * max(1.0, float(want.abs().max()))
    chosen, weights = plain.route(x, mlp["router"], w)
    on_output = sum(weights[0, k] * (w[f"e{e}.down"] @ (plain.silu(w[f"e{e}.gate"] @ x[0]) * (w[f"e{e}.up"] @ x[0])))
                    for k, e in enumerate(chosen[0].tolist()))
    assert float((on_output - want[0]).abs().max()) > 1e-3


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("layer_scale,second", [(True, True), (True, False), (False, True)])
def test_one_norm_for_both_sub_layers_with_scales_on_their_outputs(backend, layer_scale, second):
    from tokenizer_amd.parts import BLOCKS, NORMS, FeedForwardSpec, LayerSpec, MixerSpec, NormSpec, Runtime
    ops, device, dtype = ops_for(backend)
    width, n = 48, 9
    gen = torch.Generator().manual_seed(3)
    runtime = Runtime(dtype, device, ops)
    norm_spec = NormSpec("rmsnorm", width, 1e-5, options={"tensor_name": ""})
    vector = lambda: (1 + 0.4 * torch.randn(width, generator=gen)).to(device)
    g, ls1, ls2, final = vector(), vector(), vector(), vector()
    norm = NORMS.get("rmsnorm")(norm_spec, {"": g}, runtime)

    class Sub:
        def __init__(self, factor):
            self.factor, self.seen = factor, None

        def forward(self, x, ctx, cache=None):
            self.seen = x
            return (x.float() * self.factor).to(x.dtype)
    mixer, ff = Sub(2.0), Sub(-0.5)
    layer = LayerSpec("parallel_scaled", MixerSpec("gqa_attention", width), FeedForwardSpec("gated_dense", width), norm_spec, norm_spec,
                      options={"width": width, "layer_scale": layer_scale, "one_norm": True})
    block = BLOCKS.get("parallel_scaled")(norm, mixer, norm if second else None, ff if second else None, layer,
                                          {"ls1": ls1, "ls2": ls2}, runtime)
    residual = torch.randn(n, width, generator=gen).to(device)
    start = residual.clone()
    delta = block.forward(residual, None, None, None)
    out = NORMS.get("rmsnorm")(norm_spec, {"": final}, runtime).apply(residual, delta)
    h = plain.norm(start.double(), g.double(), 1e-5)
    one = torch.ones(width, dtype=torch.float64, device=device)
    want = start.double() + 2.0 * h * (ls1.double() if layer_scale else one)
    if second:
        assert ff.seen.data_ptr() == mixer.seen.data_ptr()
        want = want - 0.5 * h * (ls2.double() if layer_scale else one)
    bound = 1e-5 if dtype == torch.float32 else 2e-2
    assert float((residual.double() - want).abs().max()) <= bound * float(want.abs().max())
    assert float((out.double() - plain.norm(want, final.double(), 1e-5)).abs().max()) <= bound * 4


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [40, 64, 52, 200, 1028, 2056, 4096, 4100])
@pytest.mark.parametrize("count,scaled", [(1, False), (1, True), (2, True), (2, False), (3, True), (4, True)])
def test_weighted_terms_onto_the_stream_and_the_norm(backend, width, count, scaled):
    ops, device, dtype = ops_for(backend)
    gen = torch.Generator().manual_seed(width + count)
    n = 11
    residual = torch.randn(n, width, generator=gen)
    vectors = [1 + 0.4 * torch.randn(width, generator=gen) for _ in range(count + 2)]
    terms = [(torch.randn(n, width, generator=gen).to(dtype), 0.5 + k, vectors[k] if scaled else None) for k in range(count)]
    want = residual.double()
    for rows, factor, scale in terms:
        want = want + rows.double() * factor * (1.0 if scale is None else scale.double())
    on = [(rows.to(device), factor, None if scale is None else scale.to(device)) for rows, factor, scale in terms]
    bound = 2e-6 if dtype == torch.float32 else 1e-2
    for rows_picked in (None, [3, 0, 10]):
        stream = residual.clone().to(device)
        out = torch.empty((n if rows_picked is None else 3, width), dtype=dtype, device=device)
        second = torch.empty_like(out)
        pick = None if rows_picked is None else torch.tensor(rows_picked, dtype=torch.int32, device=device)
        ops.add_terms_rmsnorm(stream, on, vectors[-1].to(device), 1e-5, out, pick, store_residual=pick is None,
                              weight2=vectors[-2].to(device), eps2=1e-3, out2=second)
        x = want if rows_picked is None else want[rows_picked]
        for got, weight, eps in ((out, vectors[-1], 1e-5), (second, vectors[-2], 1e-3)):
            normed = plain.norm(x, weight.double(), eps)
            assert float((got.double().cpu() - normed).abs().max()) <= bound * float(normed.abs().max())
        kept = stream.double().cpu()
        assert float((kept - (want if pick is None else residual.double())).abs().max()) <= 2e-6 * float(want.abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("width", [64, 1024, 1028, 3584, 4096, 4104])
@pytest.mark.parametrize("parts", [1, 3, 4, 5, 8, 13])
@pytest.mark.parametrize("scaled", [True, False])
def test_a_term_that_is_a_product_still_in_parts(width, parts, scaled):
    from tokenizer_amd.kernels import PendingSum, get_ops
    ops, device = get_ops(), torch.device("cuda:0")
    gen = torch.Generator().manual_seed(width + parts)
    n = 9
    residual, rows = torch.randn(n, width, generator=gen), torch.randn(n, width, generator=gen).to(torch.bfloat16)
    slabs = torch.randn(parts, n, width, generator=gen)
    weight, one, two = (1 + 0.4 * torch.randn(width, generator=gen) for _ in range(3))
    want = residual.double() + rows.double() * (one.double() if scaled else 1.0) + slabs.double().sum(0) * (two.double() if scaled else 1.0)
    for rows_picked in (None, [8, 2]):
        stream = residual.clone().to(device)
        out = torch.empty((n if rows_picked is None else 2, width), dtype=torch.bfloat16, device=device)
        terms = [(rows.to(device), 1.0, one.to(device) if scaled else None),
                 (PendingSum(ops, slabs.to(device), None, torch.bfloat16), 1.0, two.to(device) if scaled else None)]
        pick = None if rows_picked is None else torch.tensor(rows_picked, dtype=torch.int32, device=device)
        ops.add_terms_rmsnorm(stream, terms, weight.to(device), 1e-5, out, pick, store_residual=pick is None)
        normed = plain.norm(want if pick is None else want[rows_picked], weight.double(), 1e-5)
        assert float((out.double().cpu() - normed).abs().max()) <= 1e-2 * float(normed.abs().max())
        rough = 2e-6 if width <= 4096 else 1e-2              # (rows too long for that kernel: the parts are added into bfloat16 first)
        assert pick is not None or float((stream.double().cpu() - want).abs().max()) <= rough * float(want.abs().max())


@pytest.mark.gpu
@pytest.mark.parametrize("d", [16, 32, 48, 64, 80, 96, 112, 128, 160, 192, 224, 256])
@pytest.mark.parametrize("n_q,n_kv,window,sink,page_size", [(6, 2, None, True, 16), (5, 1, 40, True, 16), (20, 1, None, False, 32), (3, 3, 16, True, 48)])
def test_single_tokens_over_values_that_are_the_keys_read_once(d, n_q, n_kv, window, sink, page_size):
    """The kernel that reads keys alone against the one that reads both pages and against the plain op, at every head size;
    slots that no token wrote hold NaN."""
    from kernel_refs import PlainOps
    from tokenizer_amd.kernels import get_ops
    ops, device, dtype = get_ops(), torch.device("cuda:0"), torch.bfloat16
    gen = torch.Generator().manual_seed(d + n_q)
    lengths = [1, 2, 16, 17, 31, 32, 33, 64, 200, 700]
    pages = [-(-n // page_size) for n in lengths]
    total = sum(pages) + 3
    order = torch.randperm(total, generator=gen).tolist()
    k_pages = torch.full((total, n_kv, page_size, d), float("nan"), dtype=dtype)
    v_pages = torch.full((total, n_kv, d, page_size), float("nan"), dtype=dtype)
    table = torch.full((len(lengths), max(pages)), -1, dtype=torch.int32)
    at = 0
    for e, n in enumerate(lengths):
        keys = torch.randn(n, n_kv, d, generator=gen).to(dtype)
        for j in range(n):
            page = order[at + j // page_size]
            table[e, j // page_size] = page
            k_pages[page, :, j % page_size] = keys[j]
            v_pages[page, :, :, j % page_size] = keys[j]
        at += pages[e]
        if window is not None:                              # pages wholly behind the window are given back
            for i in range(max(0, n - 1 - window) // page_size):
                table[e, i] = -1
    q = torch.randn(len(lengths), n_q * d, generator=gen).to(dtype)
    positions = torch.tensor([n - 1 for n in lengths], dtype=torch.int32)
    entries = torch.arange(len(lengths), dtype=torch.int32)
    sinks = torch.randn(n_q, generator=gen) if sink else None
    want = torch.empty_like(q)
    PlainOps(torch.float64).paged_attention(q, want, k_pages, v_pages, positions, entries, table, n_q, n_kv, d, window, 0.2, sinks=sinks)
    on = lambda t: None if t is None else t.to(device)
    got = {}
    before = ops.use_tied_values
    try:
        for tied in (False, True):
            ops.use_tied_values = tied
            out = torch.empty_like(q, device=device)
            ops.paged_attention(on(q), out, on(k_pages), on(v_pages), on(positions), on(entries), on(table), n_q, n_kv, d, window, 0.2,
                                max_position=max(lengths) - 1, sinks=on(sinks), tied_values=True)
            got[tied] = out.float().cpu()
    finally:
        ops.use_tied_values = before
    for out in got.values():
        assert float((out - want.float()).abs().max()) <= 2e-2
    assert float((got[True] - got[False]).abs().max()) <= 2e-2


@pytest.mark.gpu
@pytest.mark.parametrize("d", [16, 32, 48, 64, 80, 96, 112, 128, 160, 192, 224, 256, 20, 300])
@pytest.mark.parametrize("n_q,n_kv,window,sink,page_size", [(6, 2, None, True, 16), (5, 1, 40, True, 16), (12, 2, None, False, 32), (3, 3, 100, True, 48)])
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_portions_over_values_that_are_the_keys(d, n_q, n_kv, window, sink, page_size, dtype):
    """Ragged portions and single tokens over key pages alone, in every prompt kernel and shape, against the plain op; slots
    that no token wrote, and pages that were given back and hold another request's keys, hold NaN."""
    from kernel_refs import PlainOps
    from tokenizer_amd.cache import CacheManager
    from tokenizer_amd.engine.batch import StepEntry, build_context
    from tokenizer_amd.kernels import get_ops
    from tokenizer_amd.parts import CacheNeed
    dtype = getattr(torch, dtype)
    ops, device = get_ops(), torch.device("cuda:0")
    gen = torch.Generator().manual_seed(d + n_q)
    need = CacheNeed(kind="full" if window is None else "window", n_kv_heads=n_kv, head_dim=d, window=window, tied_values=True)
    manager = CacheManager([need], num_pages=60, page_size=page_size, max_requests=5)
    k_pages = torch.full((60, n_kv, page_size, d), float("nan"), dtype=dtype)
    counts = {"a": (0, 90), "b": (130, 37), "c": (60, 1), "d": (0, 1), "e": (33, 2)}
    keys = {rid: torch.randn(before + new, n_kv, d, generator=gen).to(dtype) for rid, (before, new) in counts.items()}
    entries = []
    for rid, (before, new) in counts.items():
        manager.add_request(rid)
        if before:
            assert manager.reserve(rid, before)
            manager.advance(rid, before)
        assert manager.reserve(rid, before + new)
        entries.append(StepEntry(rid, [0] * new, []))
        table = manager.table(rid, 0)
        for j in range(before + new):
            if table[j // page_size] >= 0:
                k_pages[table[j // page_size], :, j % page_size] = keys[rid][j]
    ctx = build_context(entries, manager, device)
    n = ctx.n_tokens
    q = torch.randn(n, n_q * d, generator=gen).to(dtype)
    sinks = torch.randn(n_q, generator=gen) if sink else None
    want = torch.zeros_like(q)
    PlainOps(torch.float64).paged_attention(q, want, k_pages, None, ctx.positions.cpu(), ctx.entry_of_token.cpu(), ctx.block_tables[0].cpu(),
                                            n_q, n_kv, d, window, 0.2, sinks=sinks, tied_values=True)
    k_dev, q_dev, sinks_dev = k_pages.to(device), q.to(device), None if sinks is None else sinks.to(device)
    before = ops.prefill_shared, ops.prefill_shape, ops.prefill_waves
    shapes = [(0, 0, 0)]
    if dtype == torch.bfloat16:
        shapes += [(-1, 0, waves) for waves in (1, 2, 4, 8)] + [(1, shape, 0) for shape in (1, 2, 11, 12)]
    try:
        for shape in shapes:
            ops.prefill_shared, ops.prefill_shape, ops.prefill_waves = shape
            out = torch.zeros_like(q_dev)
            ops.paged_attention(q_dev, out, k_dev, None, ctx.positions, ctx.entry_of_token, ctx.block_tables[0], n_q, n_kv, d, window, 0.2,
                                max_position=ctx.max_position, batch=ctx, sinks=sinks_dev, tied_values=True)
            real = ctx.entry_of_token >= 0
            err = (out[real].float().cpu() - want[real.cpu()].float()).abs().max()
            assert float(err) <= (2e-5 if dtype == torch.float32 else 2e-2), shape
    finally:
        ops.prefill_shared, ops.prefill_shape, ops.prefill_waves = before


@pytest.mark.gpu
@pytest.mark.parametrize("n_q,n_kv,d,new,cached,window", [(14, 2, 64, 40, 4000, None), (14, 1, 128, 30, 3000, None), (28, 4, 128, 16, 6500, None), (14, 1, 128, 20, 3000, 2300)])
def test_short_portions_far_into_a_request_with_their_keys_in_parts(n_q, n_kv, d, new, cached, window):
    """A few tiles behind a long context: the tiles' keys are cut over workgroups, and the sink joins one of the parts."""
    from tokenizer_amd.cache import CacheManager
    from tokenizer_amd.engine.batch import StepEntry, build_context
    from tokenizer_amd.kernels import get_ops
    from tokenizer_amd.parts import CacheNeed
    ops, device = get_ops(), torch.device("cuda:0")
    gen = torch.Generator().manual_seed(d + new)
    need = CacheNeed(kind="full" if window is None else "window", n_kv_heads=n_kv, head_dim=d, window=window, tied_values=True)
    manager = CacheManager([need], num_pages=420, page_size=16, max_requests=1)
    manager.add_request("a")
    manager.reserve("a", cached)
    manager.advance("a", cached)
    assert manager.reserve("a", cached + new)
    ctx = build_context([StepEntry("a", [0] * new, [])], manager, device)
    keys = torch.randn(cached + new, n_kv, d, generator=gen).to(torch.bfloat16)
    k_pages = torch.full((420, n_kv, 16, d), float("nan"), dtype=torch.bfloat16)
    table = manager.table("a", 0)
    for j in range(cached + new):
        if table[j // 16] >= 0:
            k_pages[table[j // 16], :, j % 16] = keys[j]
    q = torch.randn(ctx.n_tokens, n_q * d, generator=gen).to(torch.bfloat16)
    sinks = 3.0 + torch.randn(n_q, generator=gen)
    out = torch.zeros_like(q, device=device)
    reach = ctx.max_position + 1
    args = (ctx.q_tiles.shape[0], n_q, n_kv, d, -1 if window is None else window, 0, reach, 0, 0)
    assert ops.lib.ta_prefill_attention_key_splits(*args) > 1
    ops.paged_attention(q.to(device), out, k_pages.to(device), None, ctx.positions, ctx.entry_of_token, ctx.block_tables[0], n_q, n_kv, d,
                        window, d ** -0.5, max_position=ctx.max_position, batch=ctx, sinks=sinks.to(device), tied_values=True)
    k = keys.double().repeat_interleave(n_q // n_kv, dim=1)
    for i in range(new):
        pos = cached + i
        lo = 0 if window is None else max(0, pos - window)
        scores = torch.einsum("hd,khd->hk", q[i].double().reshape(n_q, d), k[lo:pos + 1]) * d ** -0.5
        e = torch.exp(scores)
        want = torch.einsum("hk,khd->hd", e / (e.sum(-1, keepdim=True) + torch.exp(sinks.double())[:, None]), k[lo:pos + 1]).reshape(-1)
        assert float((out[i].double().cpu() - want).abs().max()) <= 1e-2


@pytest.mark.gpu
@pytest.mark.parametrize("gated,weigh_input", [(True, True), (True, False), (False, False)])
@pytest.mark.parametrize("experts,top,inner,width,tokens", [(8, 2, 48, 64, 1), (2, 1, 40, 1032, 50), (3, 3, 1032, 72, 40), (64, 4, 16, 128, 16),
                                                            (300, 1, 8, 8, 200), (5, 2, 24, 4096, 9), (1, 1, 104, 40, 33)])
def test_the_chosen_experts_of_few_rows(experts, top, inner, width, tokens, gated, weigh_input):
    """Experts that nobody chose hold NaN; more rows than one block choose the same expert; a row that names one expert twice
    (as a row of NaN does that only fills a batch up) stays a row of its own."""
    from tokenizer_amd.kernels import get_ops
    ops, device, dtype = get_ops(), torch.device("cuda:0"), torch.bfloat16
    gen = torch.Generator().manual_seed(experts * 10 + tokens)
    rand = lambda *shape: torch.randn(*shape, generator=gen, dtype=torch.float64)
    halves = 2 if gated else 1
    first = rounded(rand(experts, halves, inner, width) / width ** 0.5 * 2, dtype)
    second = rounded(rand(width, experts, inner) / inner ** 0.5, dtype)
    x = rounded(rand(tokens, width), dtype)
    chosen = torch.stack([torch.randperm(experts, generator=gen)[:top] for _ in range(tokens)]).to(torch.int32)
    if experts > 40:
        chosen = chosen % 40
    if top > 1:
        chosen[-1] = chosen[-1, 0]
    weights = (0.2 + torch.rand(tokens, top, generator=gen)).float()
    for e in range(experts):
        if not bool((chosen == e).any()):
            first[e], second[:, e] = float("nan"), float("nan")
    want = torch.zeros(top, tokens, width, dtype=torch.float64)
    for t in range(tokens):
        for k in range(top):
            e, w = int(chosen[t, k]), float(weights[t, k])
            row = w * x[t] if weigh_input else x[t]
            if gated:
                inside = plain.silu(first[e, 0] @ row) * (first[e, 1] @ row) * (1.0 if weigh_input else w)
            else:
                inside = w * torch.relu(first[e, 0] @ row) ** 2
            want[k, t] = second[:, e] @ inside
    on = lambda t: t.to(dtype).to(device).contiguous()
    fill = torch.full((width, 8), float("nan"), dtype=torch.float64)                   # columns behind the experts' own
    parts = ops.experts_few(on(x), chosen.to(device), weights.to(device), experts, on(first.reshape(-1, width)), gated, inner,
                            on(torch.cat([second.reshape(width, -1), fill], dim=1)), weigh_input=weigh_input)
    assert parts is not None and tuple(parts.partial.shape) == (top, tokens, width)
    bound = 1.5e-2 * float(want.abs().max())
    assert float((parts.partial.double().cpu() - want).abs().max()) <= bound
    assert float((parts.resolve().double().cpu() - want.sum(0)).abs().max()) <= 2 * bound


@pytest.mark.gpu
@pytest.mark.parametrize("n_q,n_kv,d,width,rows", [(4, 2, 32, 64, 8), (14, 2, 64, 896, 1), (5, 1, 96, 72, 16), (3, 3, 128, 1032, 3), (28, 4, 128, 3584, 8),
                                                   (2, 1, 256, 40, 16)])
@pytest.mark.parametrize("coef,every", [(0.4, 7), (0.0, 3), (1.2, 1)])
def test_the_projection_with_the_temperature_and_the_store_in_its_epilogue(n_q, n_kv, d, width, rows, coef, every):
    from tokenizer_amd.kernels import get_ops
    ops, device, dtype = get_ops(), torch.device("cuda:0"), torch.bfloat16
    gen = torch.Generator().manual_seed(n_q * 100 + d + rows)
    x = torch.randn(rows, width, generator=gen).to(dtype)
    weight = (torch.randn((n_q + n_kv) * d, width, generator=gen) / width ** 0.5).to(dtype)
    positions = torch.randint(0, 5000, (rows,), generator=gen, dtype=torch.int32)
    positions[0] = every - 1
    slots = torch.randperm(64, generator=gen)[:rows].to(torch.int32)
    if rows > 2:
        slots[2] = -1
    k_pages = torch.full((4, n_kv, 16, d), 7.0, dtype=dtype, device=device)
    q = ops.fused_qk_temper(x.to(device), weight.to(device), positions.to(device), coef, every, slots.to(device), k_pages, n_q, n_kv, d)
    both = x.double() @ weight.double().T
    want_q = both[:, :n_q * d] * plain.temperature(positions.long(), coef, every)[:, None]
    assert float((q.double().cpu() - want_q).abs().max()) <= 6e-3 * float(want_q.abs().max())
    want_k = torch.full((4, n_kv, 16, d), 7.0, dtype=torch.float64)
    for t, slot in enumerate(slots.tolist()):
        if slot >= 0:
            want_k[slot // 16, :, slot % 16] = both[t, n_q * d:].reshape(n_kv, d)
    assert float((k_pages.double().cpu() - want_k).abs().max()) <= 6e-3 * float(want_k.abs().max())
    untouched = want_k == 7.0
    assert torch.equal(k_pages.double().cpu()[untouched], want_k[untouched])
