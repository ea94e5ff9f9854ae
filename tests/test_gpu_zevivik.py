"""The Zevivik design through the engine against the plain implementation (`plain_zevivik.py`): whole prompts, last tokens
one by one (past every chunk's edge), portions of changing size down to two tokens, mixed batches with few pages, in
float32 and in bfloat16, on tiny configurations that differ in every size and option; requests alone against in a batch;
pages that others left dirty, pages of passed chunks kept against given back; long decoding (from graphs, bit-equal to
kernel by kernel); other page sizes; keys made to stand out through the whole model; greedy generation through `LLMEngine`
and the command lines."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_zevivik as pz
import replay_util as ru
import tiny_zevivik as tz
from test_gpu_bibevik import ChosenExperts

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = {"A": (5, 17, 33, 70), "B": (6, 34, 40, 75), "C": (1, 2, 33, 70), "D": (3, 64, 210), "E": (4, 19, 45), "F": (2, 57, 113)}
# relative to the largest |logit| of the expected rows; fixed before the first run
TOL = {"float32": ru.FP32_TOL, "bfloat16": ru.BF16_TOL}
NAMES = sorted(tz.CONFIGS)
NEAR_TIE_16 = 5e-2  # how far apart two experts' logits may lie for a 16-bit run to take either


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    out = {}
    for name, cfg in tz.CONFIGS.items():
        for dtype in ("float32", "bfloat16"):
            d = tmp_path_factory.mktemp(f"zevivik_{name}_{dtype}")
            tz.make_folder(cfg, seed=53, out_dir=str(d), dtype=dtype)
            out[(name, dtype)] = str(d)
    return out


def prompts_for(name):
    return {f"r{i}": tz.random_tokens(n, tz.CONFIGS[name]["vocab"], seed=900 + i) for i, n in enumerate(LENGTHS[name])}


def make_runner(folders, name, dtype, num_pages=64, page_size=16, max_requests=4, **kw):
    from inferx_amd.engine.runner import ModelRunner
    return ModelRunner.from_directory(folders[(name, dtype)], dtype=dtype, page_size=page_size, num_pages=num_pages,
                                      max_requests=max_requests, max_seq_len=num_pages * page_size, **kw)


def routed_runs(cfg):
    return [i for i, _ in pz.run_order(cfg) if (cfg["layers"][i].get("mlp") or {}).get("kind") == "moe"]


def expected_for(folders, name, dtype, prompts, chosen, what):
    """The plain logits of every request, and for bfloat16 how far rounding every stored activation to 16 bits moves each
    position's (relative to the largest logit; the largest of five samples).  bfloat16: with the engine's choice of experts,
    which may differ from the plain one at near ties only."""
    cfg, weights = tz.read_folder(folders[(name, dtype)])
    runs = len(routed_runs(cfg))
    out, gap = {}, {}
    for rid, toks in prompts.items():
        theirs = None
        if chosen is not None and runs:
            theirs = [torch.tensor([chosen.by_place[(rid, pos)][call] for pos in range(len(toks))]) for call in range(runs)]
        own, logits_of = [], []
        logits = pz.forward(cfg, weights, toks, experts_of=theirs, chosen=own, scores=logits_of)
        for call in range(runs if theirs is not None else 0):
            for pos in range(len(toks)):  # with the engine's experts upstream, every choice is the plain one or a near tie
                mine, other = set(own[call][pos].tolist()), set(theirs[call][pos].tolist())
                if mine != other:
                    z = logits_of[call][pos]
                    lost, taken = max(float(z[e]) for e in mine - other), min(float(z[e]) for e in other - mine)
                    assert lost - taken < NEAR_TIE_16, \
                        f"{what}: request {rid} position {pos} routed run {call}: the engine chose {sorted(other)}, " \
                        f"the plain implementation {sorted(mine)}: no near tie"
        if dtype == "bfloat16":
            used = theirs if theirs is not None else own
            exact = logits if theirs is not None else pz.forward(cfg, weights, toks, experts_of=own)
            for store in [pz.bfloat16] + [pz.jittered(s) for s in range(4)]:
                stored = pz.forward(cfg, weights, toks, experts_of=used, store=store)
                for pos, g in enumerate((stored - exact).abs().max(dim=1).values.tolist()):
                    gap[(rid, pos)] = max(g, gap.get((rid, pos), 0.0))
        out[rid] = logits
    scale = max(float(l.abs().max()) for l in out.values())
    return out, {place: g / scale for place, g in gap.items()}


def run_and_check(folders, name, dtype, steps, monkeypatch, what, prompts=None, only=None, **runner_kw):
    if dtype == "bfloat16":
        runner_kw.setdefault("use_graphs", False)
    runner = make_runner(folders, name, dtype, **runner_kw)
    chosen = ChosenExperts(runner, monkeypatch) if dtype == "bfloat16" else None
    got = ru.replay(runner, steps)
    every = prompts or prompts_for(name)
    expected, gap = expected_for(folders, name, dtype, {r: every[r] for r in (only or every)}, chosen, what)
    # bfloat16: a position that 16-bit storage alone moves by more than a third of the fixed tolerance may differ by
    # three times what that storage costs there; every position is compared in float32 with the fixed tolerance
    tol = TOL[dtype]
    touchy = {place: 3 * g for place, g in gap.items() if 3 * g > tol}
    worst = ru.compare(got, expected, tol, what, skip=touchy)
    scale = max(float(e.abs().max()) for e in expected.values())
    for (rid, pos), limit in touchy.items():
        err = float((got[(rid, pos)].double() - expected[rid][pos]).abs().max()) / scale
        assert err <= limit, f"{what}: request {rid} position {pos}: error {err:.3e}, 16-bit storage alone {limit / 3:.1e}"
    print(f"{what}: worst {worst:.2e} (tolerance {tol:.1e}; {len(touchy)} positions by their own)")
    return runner, got


WAYS = {"whole": lambda p: ru.whole(p), "tail": lambda p: ru.tail_decoded(p, 45), "portions": lambda p: ru.chunked(p)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("way", ["whole", "tail", "portions"])
def test_each_request_alone(folders, name, dtype, way, monkeypatch):
    """(`tail`: the last 45 tokens one by one, across edges of the configurations' chunks, whose pages are given back while
    decoding.)"""
    run_and_check(folders, name, dtype, WAYS[way](prompts_for(name)), monkeypatch, f"{way} {name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_with_few_pages(folders, name, dtype, monkeypatch):
    """Up to four live requests, portions of some beside single tokens of others, in a pool with room for about two of the
    longer ones: pages are given back and used again."""
    prompts = prompts_for(name)
    for i in range(4):  # more requests than slots
        prompts[f"x{i}"] = tz.random_tokens(11 + 7 * i, tz.CONFIGS[name]["vocab"], seed=950 + i)
    max_tokens = 256
    steps = ru.mixed(prompts, seed=8, max_tokens=max_tokens)
    assert any(len(s["entries"]) > 1 and {len(e[1]) for e in s["entries"]} & {1} and
               max(len(e[1]) for e in s["entries"]) > 1 for s in steps), "no step mixes a portion with a single token"
    run_and_check(folders, name, dtype, steps, monkeypatch, f"mixed {name} {dtype}", prompts, num_pages=max_tokens // 16)
    owners = {}
    runner = make_runner(folders, name, dtype, num_pages=max_tokens // 16)
    ru.replay(runner, steps, page_owners=owners)
    assert any(len(who) > 1 for who in owners.values()), "no physical page was used by two requests"


@pytest.mark.parametrize("name", ["A", "B", "D", "F"])
def test_a_batch_gives_what_each_request_gives_alone(folders, name):
    """float32: the logits of a request in a batch of unequal requests, cut into unequal portions, equal the logits of the
    same request run alone and whole, to rounding."""
    prompts = prompts_for(name)
    alone = ru.replay(make_runner(folders, name, "float32"), ru.whole(prompts))
    together = ru.replay(make_runner(folders, name, "float32"), ru.mixed(prompts, seed=5))
    scale = max(float(v.abs().max()) for v in alone.values())
    for key, row in alone.items():
        assert float((row - together[key]).abs().max()) <= 1e-5 * scale, f"{key} differs between alone and in a batch"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_pages_that_others_left_dirty(folders, name, dtype, monkeypatch):
    """A request that starts on pages that hold leftovers (not-a-number here) gives the same logits: nobody reads a place
    of a page before it is written."""
    from inferx_amd.engine.runner import ModelRunner
    prompts = prompts_for(name)
    made = ModelRunner.from_directory

    def dirty(*a, **kw):
        runner = made(*a, **kw)
        for arrays in runner.pages:
            for t in arrays.values():
                t.fill_(float("nan"))
        return runner
    monkeypatch.setattr(ModelRunner, "from_directory", dirty)
    second = {r: prompts[r] for r in sorted(prompts, reverse=True)[:3]}  # one after the other
    run_and_check(folders, name, dtype, ru.chunked(second, sizes=(3, 2, 5)), monkeypatch, f"dirty pages {name} {dtype}",
                  only=second, num_pages=16, max_requests=1)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_giving_passed_chunks_back_changes_no_logit(folders, dtype):
    """The pages of passed chunks kept until the request ends against given back: the same bits, with fewer pages in use."""
    prompts = prompts_for("A")
    steps = ru.tail_decoded(prompts, 45)
    got, held = {}, {}
    for release in (True, False):
        runner = make_runner(folders, "A", dtype, release_window_pages=release)
        groups = [g for g, n in enumerate(runner.group_needs) if n.chunk]
        assert len(groups) == 2
        held[release], real = 0, runner.run_entries

        def run_entries(entries, runner=runner, real=real, release=release):
            out = real(entries)
            held[release] = max(held[release], sum(runner.cache.pools[g].used_pages for g in groups))
            return out
        runner.run_entries = run_entries
        got[release] = ru.replay(runner, steps)
    assert held[True] < held[False]
    for key, row in got[True].items():
        assert torch.equal(row, got[False][key]), f"{key} depends on whether passed pages are given back"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "D", "F"])
def test_long_decoding(folders, name, dtype, monkeypatch):
    """A short prompt and 150 tokens one by one, two requests side by side that started at different times: kernel by
    kernel against the plain implementation, then replayed from graphs with the same bits."""
    vocab = tz.CONFIGS[name]["vocab"]
    prompts = {"a": tz.random_tokens(156, vocab, 1), "b": tz.random_tokens(140, vocab, 2)}
    steps = [{"entries": [("a", prompts["a"][:6], list(range(6)))], "end": []},
             {"entries": [("a", prompts["a"][6:16], list(range(10)))], "end": []},
             {"entries": [("a", prompts["a"][16:17], [0]), ("b", prompts["b"][:1], [0])], "end": []}]
    for i in range(1, 140):
        steps.append({"entries": [("a", prompts["a"][16 + i:17 + i], [0]), ("b", prompts["b"][i:i + 1], [0])],
                      "end": ["a", "b"] if i == 139 else []})
    _, plainly = run_and_check(folders, name, dtype, steps, monkeypatch, f"long decoding {name} {dtype}", prompts, use_graphs=False)
    runner = make_runner(folders, name, dtype)
    got = ru.replay(runner, steps)
    assert runner._graphs, "no step was replayed from a graph"
    for key, row in plainly.items():
        assert torch.equal(row, got[key]), f"{key}: replayed from a graph differs from kernel by kernel"


@pytest.mark.parametrize("page_size", [8, 48])
def test_other_page_sizes(folders, page_size, monkeypatch):
    for dtype in ("float32", "bfloat16"):
        run_and_check(folders, "A", dtype, ru.chunked(prompts_for("A")), monkeypatch, f"pages of {page_size} {dtype}", num_pages=24,
                      page_size=page_size)


def standing_out(cfg, weights, length, key):
    """Weights whose first attention layer answers the last token's query with the key of one token of the prompt, wherever
    that lies: two tokens of the vocabulary whose embeddings point two ways, found by Wq and Wk of every head in the same
    direction (nothing of it is rotated); and the prompt."""
    w = {k: v.clone().double() for k, v in weights.items()}
    mark, ask = 0, 1
    toks = [2 + t % (cfg["vocab"] - 2) for t in tz.random_tokens(length, cfg["vocab"], 77)]
    toks[key], toks[-1] = mark, ask
    W, m = cfg["width"], cfg["layers"][0]["mixer"]
    w["embed"][:, :2] = 0.0
    for t, c in ((mark, 0), (ask, 1)):
        w["embed"][t] = 0.0
        w["embed"][t, c] = 1.0
    w["l0.norm1"] = torch.ones(W, dtype=torch.float64)
    for n, heads, c in (("q", m["heads"], 1), ("k", m["kv_heads"], 0)):
        rows = w[f"l0.mix.{n}"].view(heads, m["dim"], W)
        rows[:, :, :2] = 0.0
        rows[:, m["dim"] - 1, c] = (8.0 / m["scale"] / W) ** 0.5 * 2  # (a marked row is sqrt(W) long after the norm)
    return {k: v.to(weights[k].dtype) for k, v in w.items()}, toks


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("length,key", [(110, 80), (110, 79), (110, 81), (110, 95), (110, 96), (110, 108), (81, 80), (82, 80), (81, 79), (120, 80),
                                        (120, 40)])
def test_a_key_inside_and_outside_the_chunk_through_the_model(tmp_path, length, key, dtype):
    """Configuration D's chunks of 40: a marked token just inside and just outside the last query's chunk, at page borders
    and far back, found by a prompt's last token, by the last token alone, and after portions whose cuts lie around it."""
    from inferx_amd.engine.runner import ModelRunner
    from safetensors.torch import load_file, save_file
    cfg = dict(tz.D, layers=tz.D["layers"][:2])
    folder = tz.make_folder(cfg, seed=5, out_dir=str(tmp_path), dtype=dtype)
    path = os.path.join(folder, "model.safetensors")
    weights, toks = standing_out(cfg, load_file(path), length, key)
    save_file({k: v.contiguous() for k, v in weights.items()}, path)
    want = pz.forward(cfg, weights, toks)
    other = list(toks)
    other[key] = 2  # without the mark the answer differs clearly where the key is seen
    scale = float(want.abs().max())
    moved = float((pz.forward(cfg, weights, other)[-1] - want[-1]).abs().max()) / scale
    runner = ModelRunner.from_directory(folder, dtype=dtype, page_size=16, num_pages=16, max_requests=2, max_seq_len=256)
    tol = {"float32": 5e-5, "bfloat16": 3e-2}[dtype]
    if (length - 1) // 40 == key // 40 and key != length - 1:
        assert moved > 3 * tol, "the marked key does not show in the logits"
    for cuts in ([length], [length - 1, 1], [key, 1, length - key - 1], [key + 1, length - key - 1], [key - 1, 2, length - key - 1]):
        cuts = [c for c in cuts if c]
        runner.add_request("x")
        at = 0
        for n in cuts:
            got = runner.run_entries([("x", toks[at:at + n], [n - 1])])
            at += n
        runner.end_request("x")
        err = float((got.cpu()[-1].double() - want[-1]).abs().max()) / scale
        assert err <= tol, f"portions {cuts}: {err:.2e}"


def greedy_agrees(cfg, weights, prompt, out, what):
    seq = list(prompt)
    for i, token in enumerate(out):
        want = int(torch.argmax(pz.forward(cfg, weights, seq)[-1]))
        assert token == want, f"{what}: token {i} is {token}, the plain implementation says {want}"
        seq.append(token)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_engine(folders, name, dtype):
    from inferx_amd.engine.engine import LLMEngine
    from inferx_amd.sampling import SamplingParams
    cfg, weights = tz.read_folder(folders[(name, dtype)])
    prompts = [tz.random_tokens(n, cfg["vocab"], seed=n) for n in (5, 9, 17, 30, 3, 12)]
    # a token budget below the longest prompt: prompts come in portions beside decoding requests; four at a time
    engine = LLMEngine(folders[(name, dtype)], dtype, max_num_seqs=4, max_model_len=96, max_num_batched_tokens=16,
                       num_gpu_blocks_override=20)
    outs = engine.generate(prompts, SamplingParams(max_tokens=12))
    for prompt, out in zip(prompts, outs):
        assert len(out) == 12
        if dtype == "float32":
            greedy_agrees(cfg, weights, prompt, out, f"{name} {dtype}")


def test_command_lines(folders, tmp_path):
    """`bin/inferx-generate` and `bin/trace_run` choose the model class by config.json."""
    folder = folders[("A", "float32")]
    cfg, weights = tz.read_folder(folder)
    prompt = tz.random_tokens(7, cfg["vocab"], 4)
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "inferx-generate"), "--model", folder, "--dtype",
                        "float32", "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "5", "--max-model-len",
                        "64", "--num-gpu-blocks-override", "8"], capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    tokens = json.loads(p.stdout.strip().splitlines()[-1])["output_token_ids"]
    assert len(tokens) == 5
    greedy_agrees(cfg, weights, prompt, list(tokens), "inferx-generate")

    steps = [{"step": 0, "entries": [{"id": "a", "tokens": prompt[:4], "want": [0, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": prompt[4:], "want": [2]},
                                     {"id": "b", "tokens": prompt[:2], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": prompt[2:3], "want": [0]}], "end": ["b"]}]
    out_dir = tmp_path / "logits"
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out",
                        str(out_dir), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = pz.forward(cfg, weights, prompt).numpy()
    scale = float(np.abs(want).max())
    for step, rows in ((0, [0, 3]), (1, [6]), (2, [2])):
        got = np.fromfile(out_dir / f"{step}.f32", dtype="<f4").reshape(len(rows), -1)
        assert float(np.abs(got - want[rows]).max()) <= ru.FP32_TOL * scale
