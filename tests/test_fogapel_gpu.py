"""Fogapel in the engine against the plain implementation (tests/plain_fogapel.py): every way of
cutting the work, both precisions, small configurations that differ in every size and branch, and
some drawn at random; chunk edges in prompts and in decoding; a sharp key among many; far tokens that
only the time mixers carry; state and pages used again; recorded steps; generation through the entry
points."""
import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import cuttings
import plain_fogapel
from fogapel_configs import drawn, fogapel
from engine_helpers import (TOL, first_mismatch, first_wrong_row, load_graph_runner, load_runner,
                            random_sequences, replay, replay_wanted)

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = {"F1": [5, 9, 33, 70, 130, 47], "F2": [3, 17, 40, 65, 31], "F3": [12, 50, 90, 20, 2],
           "F4": [7, 30, 64, 97], "F4c": [2, 50, 97], "F5": [9, 170, 66, 35], "F6": [4, 40, 100, 21]}
DTYPES = [torch.float32, torch.bfloat16]
NAMES = ["F1", "F2", "F3", "F4", "F4c", "F5", "F6"]
ROUTER_GAIN = 8.0       # routers this much larger than the other matrices: few choices that rounding turns
CLOSE_CALL = 0.01       # gap of two router logits, as a share of the logits' spread, that rounding may turn


def matrix_names(cfg):
    """The tensors an engine holds in its own dtype (the others stay float32)."""
    from pytriton_llama_amd.config import build_model
    return {n for n, (_, src) in build_model(copy.deepcopy(cfg)).expected_tensors().items() if src.kind == "matrix"}


def read_folder(folder, weights_as=None):
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    w = load_file(os.path.join(folder, "model.safetensors"))
    if weights_as is not None:      # the values an engine of that dtype holds: matrices are rounded
        rounded = matrix_names(cfg)
        w = {k: (v.to(weights_as).float() if k in rounded else v) for k, v in w.items()}
    return cfg, w


def write_folder(tmp_path_factory, cfg, std, seed, edit=None, tame=False):
    """A model folder of random weights. ``edit``: called with the tensors before they are stored.
    ``tame``: the time mixers' keys are their receptances and the bonus is positive, so that what a head
    reads behind few tokens is never the small rest of a cancellation whose sign the rounding of bfloat16
    decides and the norm of the heads blows up, and routers are decisive. The float32 tests run on the untamed
    weights (but for the configurations drawn at random, where rounding to float32 alone may be blown up to
    the tolerance)."""
    from safetensors.torch import load_file, save_file
    from pytriton_llama_amd.weights import write_random_model
    folder = str(tmp_path_factory.mktemp("fogapel"))
    write_random_model(cfg, folder, seed=seed, dtype=torch.float32, norm_std=0.1, std=std)
    if edit is not None or tame:
        path = os.path.join(folder, "model.safetensors")
        w = load_file(path)
        for k in list(w):
            if tame and k.endswith(".mix.u"):
                pre = k[:-1]
                w[pre + "k"], w[pre + "mu.k"] = w[pre + "r"].clone(), w[pre + "mu.r"].clone()
                w[k] = w[k].abs() + 0.3
            if tame and k.endswith(".mlp.router"):
                w[k] = w[k] * ROUTER_GAIN
        if edit is not None:
            edit(w)
        save_file(w, path)
    return folder


def plain_logits(folder, seqs, weights_as=None, touchy=None):
    """``weights_as``: the plain model with matrices and stored results rounded as an engine of that
    dtype rounds them. ``touchy``: a dict that receives, per request, the positions at which a comparison
    says nothing: those that rounding alone moves by more than half the tolerance in the plain model,
    and those at which a router's choice is a close call that rounding may turn."""
    cfg, w = read_folder(folder, weights_as)
    out = {}
    routed = plain_fogapel.routed
    with torch.no_grad():
        for rid, toks in seqs.items():
            close = torch.zeros(len(toks), dtype=torch.bool)

            def watched(h, mlp, t, pre):
                z = plain_fogapel.lin(h, t[pre + "router"], t[pre + "router.b"])
                top = mlp["router"]["top"]
                if top < z.shape[1]:
                    order = z.sort(-1, descending=True).values
                    close.logical_or_(order[:, top - 1] - order[:, top] < CLOSE_CALL * (order[:, 0] - order[:, -1]))
                return routed(h, mlp, t, pre)
            try:
                plain_fogapel.routed = watched if touchy is not None else routed
                out[rid] = plain_fogapel.forward(cfg, w, toks, round_inputs=weights_as).float()
            finally:
                plain_fogapel.routed = routed
            if touchy is not None:
                exact = plain_fogapel.forward(cfg, w, toks).float()
                touchy[rid] = close | ((out[rid] - exact).abs().amax(dim=-1) / exact.abs().max() > 0.5 * TOL[weights_as])
    return out


def wrong_places(got, want, dtype):
    """None, or a text that says what is wrong. float32: no place may differ by more than the
    tolerance. bfloat16: a router's choice that rounding turns in the engine and not in the plain
    model (one that the plain model's own margins did not give away) moves a position by any amount
    and those behind it a little, so a few positions may lie beyond the tolerance: at most one in
    thirty, and none by more than four times the tolerance. A key lost, a chunk off by one, a state that is
    not carried or a sink left out moves many positions and does not pass."""
    tol = TOL[dtype]
    if dtype == torch.float32:
        bad = first_mismatch(got, want, tol)
        return None if bad is None else f"first wrong place (request, position, error) = {bad}"
    errs = []
    for rid in want:
        e = (got[rid] - want[rid]).abs().amax(dim=-1) / float(want[rid].abs().max())
        errs += [(float("inf") if x != x else x, rid, p) for p, x in enumerate(e.tolist())]
    over = [e for e in errs if e[0] > tol]
    if len(over) * 30 <= len(errs) and (not over or max(over)[0] <= 4 * tol):
        return None
    return f"{len(over)} of {len(errs)} places beyond the tolerance, the worst (error, request, position) = {max(over)}"


def skip_touchy(got, want, touchy):
    for rid, t in touchy.items():
        if rid in got:
            got[rid][t] = want[rid][t]


def make_case(tmp_path_factory, cfg, std, page, lengths, seed, tame_both=False):
    tamed = write_folder(tmp_path_factory, cfg, std, seed, tame=True)
    folder = tamed if tame_both else write_folder(tmp_path_factory, cfg, std, seed)
    seqs = random_sequences(cfg["vocab"], lengths, seed=seed + 3)
    touchy = {}
    want = {torch.float32: plain_logits(folder, seqs),
            torch.bfloat16: plain_logits(tamed, seqs, torch.bfloat16, touchy), "touchy": touchy}
    assert sum(int(c.sum()) for c in touchy.values()) * 4 < sum(len(c) for c in touchy.values())
    return {torch.float32: folder, torch.bfloat16: tamed}, page, seqs, want


@pytest.fixture(scope="module")
def cases(tmp_path_factory, gpu_device):
    out = {}
    for i, name in enumerate(NAMES):
        cfg, std, page = fogapel(name)
        out[name] = make_case(tmp_path_factory, cfg, std, page, LENGTHS[name], 61 + i)
    return out


def run_steps(case, dtype, steps, num_pages=None):
    folders, page, seqs, want = case
    if num_pages is None:
        num_pages = -(-cuttings.max_live_tokens(steps, round_to=page) // page)
    runner = load_runner(folders[dtype], dtype, page, num_pages, max_num_seqs=4)
    got = replay(runner, steps, seqs)
    if dtype == torch.bfloat16:
        skip_touchy(got, want[dtype], want["touchy"])
    bad = wrong_places(got, want[dtype], dtype)
    assert bad is None, f"{dtype}: {bad}"
    assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.paged)
    assert runner.manager.num_free_slots == 4


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", NAMES)
def test_whole(cases, name, dtype):
    run_steps(cases[name], dtype, cuttings.whole(cases[name][2]))


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", NAMES)
def test_last_tokens_one_by_one(cases, name, dtype):
    run_steps(cases[name], dtype, cuttings.tail_decode(cases[name][2], 40))


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", NAMES)
def test_portions_down_to_two_tokens(cases, name, dtype):
    run_steps(cases[name], dtype, cuttings.portions(cases[name][2]))


@pytest.mark.parametrize("name", NAMES)
def test_first_tokens_one_by_one_then_portions(cases, name):
    """The first tokens of a sequence alone: convolutions that reach before the start, states that
    start from zero."""
    run_steps(cases[name], torch.float32,
              cuttings.portions(cases[name][2], sizes=(1, 1, 2, 1, 3, 16, 1, 15, 2, 32)))


@pytest.mark.parametrize("name", NAMES)
def test_every_token_alone(cases, name):
    """Token-by-token decoding from the first token on against the whole prompt."""
    folders, page, seqs, want = cases[name]
    short = {r: t for r, t in seqs.items() if len(t) <= 70}
    runner = load_runner(folders[torch.float32], torch.float32, page, 32, max_num_seqs=4)
    got = replay(runner, cuttings.portions(short, sizes=(1,)), short)
    assert first_mismatch(got, {r: want[torch.float32][r] for r in short}, TOL[torch.float32]) is None


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_with_pages_and_slots_used_again(cases, name, dtype):
    _, page, seqs, _ = cases[name]
    steps = cuttings.mixed(seqs, seed=5, max_live=3)
    need = cuttings.max_live_tokens(steps, round_to=page) // page
    assert need < sum(-(-len(t) // page) for t in seqs.values())
    run_steps(cases[name], dtype, steps, need)


@pytest.mark.parametrize("name", NAMES)
def test_a_slot_that_is_used_again_starts_from_zero(cases, name):
    """Two state slots for all requests, one after the other: every request but the first two
    gets a slot (and pages) that another one has filled."""
    folders, page, seqs, want = cases[name]
    runner = load_runner(folders[torch.float32], torch.float32, page, 48, max_num_seqs=2)
    got = replay(runner, cuttings.portions(seqs, sizes=(9, 1, 30)), seqs)
    assert first_mismatch(got, want[torch.float32], TOL[torch.float32]) is None
    got = replay(runner, cuttings.whole(seqs), seqs)          # and once more, on used slots throughout
    assert first_mismatch(got, want[torch.float32], TOL[torch.float32]) is None


@pytest.mark.parametrize("name", NAMES)
def test_a_batch_gives_what_each_request_gives_alone(cases, name):
    """Unequal requests in one step against each alone (float32: the differences are those of
    the order of sums only)."""
    folders, page, seqs, _ = cases[name]
    runner = load_runner(folders[torch.float32], torch.float32, page, 128, max_num_seqs=8)
    alone = replay(runner, cuttings.whole(seqs), seqs)
    together = [{"step": 0, "end": list(seqs),
                 "entries": [{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in seqs.items()]}]
    batch = replay(runner, together, seqs)
    assert first_mismatch(batch, alone, 5e-6) is None


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path_factory, gpu_device, seed, dtype):
    cfg, std, page = drawn(seed)
    case = make_case(tmp_path_factory, cfg, std, page, [3, 40, 101, 18], 300 + seed, tame_both=True)
    for steps in (cuttings.tail_decode(case[2], 30), cuttings.portions(case[2], sizes=(19, 2, 33, 1, 5)),
                  cuttings.mixed(case[2], seed=seed, max_live=3)):
        run_steps(case, dtype, steps)


# ---- chunk edges, sharp keys and far tokens ------------------------------------------------------
def changed(toks, at, vocab):
    return toks[:at] + [(toks[at] + 1) % vocab] + toks[at + 1:]


def cut(seqs, sizes, decode_from):
    steps = []
    for rid, t in seqs.items():
        lo, k = 0, 0
        while lo < len(t):
            n = 1 if lo >= decode_from else sizes[k % len(sizes)]
            hi = min(len(t), lo + n, decode_from if lo < decode_from else len(t))
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": t[lo:hi], "want": list(range(hi - lo))}],
                          "end": [rid] if hi == len(t) else []})
            lo, k = hi, k + 1
    return steps


@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", ["F4", "F4c"])
def test_chunk_edges_in_prompts_and_in_decoding(tmp_path_factory, gpu_device, name, dtype):
    """A model whose tokens meet through the attention alone, its scores scaled up so that the softmax
    picks few keys. The first token of a query's chunk moves its logits by far more than the tolerance;
    the one in front of the chunk not at all, or, with convolutions, those that no tap of the chunk's
    first token reaches: in the plain model first, so that the comparison with the engine (over portions
    that end at, in front of and behind the edges, and over tokens decoded across them) means
    something."""
    cfg, std, page = fogapel(name)
    if name == "F4c":                        # (through a second layer's taps, a whole chunk reaches over the edge)
        cfg["layers"] = cfg["layers"][:1]
    for l in cfg["layers"]:
        l["mixer"]["scale"] *= 2.0
    m = cfg["layers"][0]["mixer"]
    size, taps = m["mask"]["size"], m["conv"]
    folder = write_folder(tmp_path_factory, cfg, std, 77)
    seqs = random_sequences(200, [7 * size + 5, size + 1], seed=3)
    toks = seqs["r0"]
    rounded = None if dtype == torch.float32 else dtype
    touchy = {}
    want = plain_logits(folder, seqs, rounded, touchy if rounded else None)
    scale = float(want["r0"].abs().max())
    edge = 5 * size
    inside = plain_logits(folder, {"r": changed(toks, edge, 200)}, rounded)["r"]
    moved = lambda other, rows: (other[rows] - want["r0"][rows]).abs().amax(-1) / scale
    rows = slice(edge + 1, edge + size)
    assert float(moved(inside, rows).median()) > (1.0 if rounded else 100.0) * TOL[dtype]
    outside = plain_logits(folder, {"r": changed(toks, edge - taps, 200)}, rounded)["r"]
    assert float(moved(outside, slice(edge, len(toks))).max()) == 0.0
    if taps > 1:                             # (a convolution reaches over the edge)
        near = plain_logits(folder, {"r": changed(toks, edge - 1, 200)}, rounded)["r"]
        assert float(moved(near, slice(edge, edge + taps)).max()) > TOL[dtype]
    # without the added term, and without the cap, the logits are others
    import torch.nn.functional as F
    for attr, other in (("softmax_with_one", lambda s, seen: F.softmax(s.masked_fill(~seen, float("-inf")), -1)),
                        ("softcap", lambda s, cap: s)):
        keep = getattr(plain_fogapel, attr)
        try:
            setattr(plain_fogapel, attr, other)
            bare = plain_logits(folder, {"r": toks}, rounded)["r"]
        finally:
            setattr(plain_fogapel, attr, keep)
        assert float(moved(bare, slice(0, len(toks))).max()) > 2 * TOL[dtype], attr
    for steps in (cut(seqs, (size,), 10 ** 6), cut(seqs, (size - 1, 2), 4 * size + 3), cut(seqs, (size + 1, 61, 2), 3 * size - 1),
                  cut(seqs, (10 ** 6,), 10 ** 6), cut(seqs, (130, 33, 2, 17), 5 * size - 2)):
        runner = load_runner(folder, dtype, page, 32, max_num_seqs=2)
        got = replay(runner, steps, seqs)
        if rounded:
            skip_touchy(got, want, touchy)
        bad = first_mismatch(got, want, TOL[dtype])
        assert bad is None, bad


def test_far_tokens_that_the_time_mixers_carry(tmp_path_factory, gpu_device):
    """Slow decays in every time mixer: the third token of a 500-token sequence still moves the last
    logits by far more than the tolerance, through the state alone (chunks are over long before)."""
    cfg, std, page = fogapel("F1")

    def edit(w):
        for k in w:
            if k.endswith("w0"):
                w[k] = w[k] * 0.0 - 9.0
    folder = write_folder(tmp_path_factory, cfg, std, 12, edit)
    seqs = random_sequences(200, [500], seed=8)
    want = plain_logits(folder, seqs)
    other = plain_logits(folder, {"r0": changed(seqs["r0"], 2, 200)})["r0"]
    shift = (other[-60:] - want["r0"][-60:]).abs().max() / want["r0"].abs().max()
    assert float(shift) > 20 * TOL[torch.float32], float(shift)
    for steps in (cuttings.whole(seqs), cuttings.tail_decode(seqs, 120), cuttings.portions(seqs, sizes=(65, 2, 190, 31))):
        runner = load_runner(folder, torch.float32, page, 40, max_num_seqs=2)
        assert first_mismatch(replay(runner, steps, seqs), want, TOL[torch.float32]) is None


def test_a_pool_too_small_unless_chunks_give_their_pages_back(cases):
    """F4's chunks of 48 positions in pages of 16: a request of 97 tokens decodes on four pages."""
    folders, page, seqs, want = cases["F4"]
    seqs = {"r3": seqs["r3"]}
    assert len(seqs["r3"]) > 4 * page
    runner = load_runner(folders[torch.float32], torch.float32, page, 4, max_num_seqs=1)
    got = replay(runner, cuttings.portions(seqs, sizes=(16, 1, 1, 9)), seqs)
    assert first_mismatch(got, {"r3": want[torch.float32]["r3"]}, TOL[torch.float32]) is None


def test_long_decoding_keeps_the_state(cases):
    """300 tokens one by one behind a short prompt: the matrices, the rows in front and the
    convolutions' inputs are carried through every step."""
    folder, page = cases["F1"][0][torch.float32], cases["F1"][1]
    seqs = random_sequences(200, [320], seed=9)
    want = plain_logits(folder, seqs)
    runner = load_runner(folder, torch.float32, page, 24, max_num_seqs=2)
    got = replay(runner, cuttings.tail_decode(seqs, 300), seqs)
    assert first_mismatch(got, want, TOL[torch.float32]) is None


# ---- recorded steps ----------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES, ids=["fp32", "bf16"])
@pytest.mark.parametrize("name", ["F1", "F2", "F5", "F6"])
def test_cuttings_replayed_as_graphs(cases, name, dtype):
    """Decode steps and single portions replayed as HIP graphs (padded layouts: rows that belong
    to nobody, the padding state slot) against the plain model."""
    folders, page, seqs, want = cases[name]
    for steps in (cuttings.tail_decode(seqs, 24), cuttings.mixed(seqs, seed=9, max_live=3)):
        for st in steps:
            for e in st["entries"]:
                e["want"] = e["want"][-1:]
        places = cuttings.wanted_places(steps)
        runner = load_graph_runner(folders[dtype], dtype, page, 64, max_model_len=200, max_num_seqs=4)
        got = replay_wanted(runner, steps)
        rows = {r: want[dtype][r][torch.as_tensor(places[r])] for r in got}
        if dtype == torch.bfloat16:
            skip_touchy(got, rows, {r: want["touchy"][r][torch.as_tensor(places[r])] for r in got})
        bad = wrong_places(got, rows, dtype)
        assert bad is None, f"{name} {dtype}: {bad}"


@pytest.mark.parametrize("graphs", [False, True], ids=["eager", "graphs"])
def test_long_portions_take_the_recurrences_in_segments(cases, graphs):
    """Portions of 900 and 300 tokens (walked in segments side by side), the first followed by portions
    that start inside a segment and by tokens one by one from the state the segments left; launched
    kernel by kernel and replayed as graphs."""
    from pytriton_llama_amd import ops
    folders, page, _, _ = cases["F5"]
    folder = folders[torch.bfloat16]            # (the tamed weights; the engine is float32)
    assert ops.linear_segment(1, 900, 2, 64, 256) < 300
    seqs = random_sequences(184, [1240, 310], seed=21)
    want = plain_logits(folder, seqs)
    steps, at = [], {"r0": 0, "r1": 0}
    for rid, n in (("r0", 900), ("r1", 300), ("r0", 330), ("r1", 1), ("r1", 1)) + (("r0", 1),) * 10 + (("r1", 8),):
        lo = at[rid]
        at[rid] = hi = lo + n
        steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": seqs[rid][lo:hi], "want": [n - 1]}],
                      "end": [rid] if hi == len(seqs[rid]) else []})
    assert at == {r: len(t) for r, t in seqs.items()}
    places = cuttings.wanted_places(steps)
    if graphs:
        runner = load_graph_runner(folder, torch.float32, page, 128, max_model_len=1280, max_num_seqs=2)
    else:
        runner = load_runner(folder, torch.float32, page, 128, max_num_seqs=2)
    got = replay_wanted(runner, steps)
    rows = {r: want[r][torch.as_tensor(places[r])] for r in got}
    bad = first_wrong_row(got, rows, places, TOL[torch.float32])
    assert bad is None, bad


# ---- generation ----------------------------------------------------------------------------------
def plain_greedy(folder, prompt, n):
    cfg, w = read_folder(folder)
    toks = list(prompt)
    with torch.no_grad():
        for _ in range(n):
            toks.append(int(plain_fogapel.forward(cfg, w, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["F1", "F6"])
def test_greedy_generation_through_the_entry_point(cases, name):
    from pytriton_llama_amd.generate import GenerateText
    folder, page = cases[name][0][torch.float32], cases[name][1]
    vocab = fogapel(name)[0]["vocab"]
    g = torch.Generator().manual_seed(4)
    prompts = [torch.randint(0, vocab, (n,), generator=g).tolist() for n in (4, 11, 19, 26)]
    want = [plain_greedy(folder, p, 10) for p in prompts]
    gen = GenerateText(folder, max_seq_len=64, max_gpu_num_blocks=16, dtype="float32", page_size=page,
                       max_batch_size=4)
    got, _ = gen.generate(prompts, max_gen_len=10, temperature=0.0)
    assert got == want


def test_scheduler_with_few_pages_preempts_and_gives_the_same_tokens(cases):
    from pytriton_llama_amd.config import EngineConfig
    from pytriton_llama_amd.engine import Engine, SamplingParams
    folder, page = cases["F3"][0][torch.float32], cases["F3"][1]
    g = torch.Generator().manual_seed(6)
    prompts = [torch.randint(0, 120, (n,), generator=g).tolist() for n in (6, 9, 14, 17)]
    sp = SamplingParams(temperature=0.0, max_new_tokens=12)
    want = [plain_greedy(folder, p, 12) for p in prompts]
    tight = Engine(folder, EngineConfig(dtype="float32", page_size=page, num_pages=8, max_num_seqs=4,
                                        max_model_len=64, max_num_batched_tokens=16, prefill_chunk=6))
    got = tight.generate(prompts, sp)
    assert tight.scheduler.num_preemptions > 0
    assert got == want
    tight.runner.manager.check()
    assert tight.runner.manager.num_free_slots == 4


def test_command_line_and_trace_replay(cases, tmp_path):
    folders, page, seqs, want = cases["F2"]
    folder = folders[torch.float32]
    prompt = seqs["r1"]
    out = subprocess.run(
        [sys.executable, os.path.join(ROOT, "cli.py"), "--checkpoints_dir", folder, "--dtype", "float32",
         "--temperature", "0", "--max_gen_len", "4", "--max_seq_len", "64", "--max_gpu_num_blocks", "16",
         "--page_size", str(page), "--prompt_ids", ",".join(map(str, prompt))],
        capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert " ".join(map(str, plain_greedy(folder, prompt, 4))) in " ".join(out.stdout.split())
    steps = cuttings.mixed(seqs, seed=2, max_live=4)
    lines = "\n".join(json.dumps(s) for s in steps) + "\n"
    run = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
         "--out", str(tmp_path), "--max-tokens", str(cuttings.max_live_tokens(steps))],
        input=lines, capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [l for l in run.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    import numpy as np
    fed = {r: 0 for r in seqs}
    for s in steps:
        got = torch.from_numpy(np.fromfile(str(tmp_path / f"{s['step']}.f32"), dtype="<f4")).view(-1, 151)
        row = 0
        for e in s["entries"]:
            n = len(e["tokens"])
            ref = want[torch.float32][e["id"]][fed[e["id"]]:fed[e["id"]] + n]
            assert float((got[row:row + n] - ref).abs().max() / ref.abs().max()) < TOL[torch.float32]
            row, fed[e["id"]] = row + n, fed[e["id"]] + n
