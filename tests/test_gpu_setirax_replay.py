"""Setirax in the engine against the plain model under every way of cutting the same requests: whole, last tokens one by
one (through graphs and without), portions of changing size down to two tokens, mixed with other requests on so few pages
and slots that they are used again; float32 and bfloat16; small configurations that differ in every size and option, and
configurations drawn at random; and greedy generation through the engine's own entry point and scheduler."""
import numpy as np
import pytest
import torch

import trace_tools
from helpers import BF16_FLOOR, TOL_F32, rel_err, write_model_dir
from plain import setirax_plain as plain
from setirax_helpers import (SET, as_f64, dense, latent, make_weights, model, parallel, plain_logits, plain_logits_bf16,
                             plain_logits_f32, random_config, random_tokens, sharpened, stored_config, unit)

pytestmark = pytest.mark.gpu

NAMES = ["A", "B", "C", "D", "E", "F", "G"]
LENGTHS = {"A": [70, 5, 45, 21, 33, 2], "B": [88, 40, 66, 3, 58], "C": [150, 17, 140, 49], "D": [50, 36, 77, 1],
           "E": [40, 3, 65], "F": [90, 26, 25, 61], "G": [33, 70, 4, 129]}
PAGE = {"A": 16, "B": 8, "C": 16, "D": 16, "E": 16, "F": 8, "G": 32}
GAINS = {"sharp": 2.0, "mild": 1.0}


def bounds(dtype, moved):
    """(most of one row, most of the mean) for errors of the engine's rows, from the errors ``moved`` that the type's
    arithmetic alone makes in the plain model's rows. A state or an output that nearly cancels before it is divided by its
    root mean square amplifies rounding many times, in other rows with every order of the same sums: the worst row may be a
    few times the plain model's worst, the mean over many rows may not."""
    if dtype == "float32":
        return max(TOL_F32, 8 * max(moved)), None
    return 3 * max(moved) + BF16_FLOOR, 1.3 * float(np.mean(moved)) + 1e-3


def judge(errors, dtype, moved, what):
    most, mean = bounds(dtype, moved)
    worst, average = max(errors), float(np.mean(errors))
    print(f"{what} [{dtype}]: {len(errors)} rows, worst relative error {worst:.3e} (allowed {most:.3e}), mean {average:.3e} "
          f"({'not judged' if mean is None else f'allowed {mean:.3e}'})")
    assert worst <= most, f"{what}: relative error {worst:.3e} exceeds {most:.1e}"
    assert mean is None or len(errors) < 60 or average <= mean, f"{what}: mean relative error {average:.3e} exceeds {mean:.1e}"


def moved_by(dtype, cfg, weights, tokens, want, rows=None):
    other = (plain_logits_f32 if dtype == "float32" else plain_logits_bf16)(cfg, weights, tokens)
    return [rel_err(other[p], want[p]) for p in (rows if rows is not None else range(len(tokens)))]


class Case:
    def __init__(self, name, tmp, kind):
        self.name, self.kind, self.cfg, self.page = name, kind, sharpened(SET[name], GAINS[kind]), PAGE[name]
        self.weights = make_weights(self.cfg, seed=sum(map(ord, name)) + 1)
        self.dir = write_model_dir(str(tmp / f"set{name}_{kind}"), stored_config(self.cfg), self.weights)
        self.reqs = {f"r{i}": random_tokens(self.cfg, n, seed=100 + i) for i, n in enumerate(LENGTHS[name])}
        self.want = {rid: plain_logits(self.cfg, self.weights, toks) for rid, toks in self.reqs.items()}
        self.moved = {dtype: [e for rid, toks in self.reqs.items() for e in moved_by(dtype, self.cfg, self.weights, toks, self.want[rid])]
                      for dtype in ("float32", "bfloat16")}

    def check(self, got, dtype, what):
        judge([rel_err(row, self.want[rid][pos]) for (rid, pos), row in got.items()], dtype, self.moved[dtype], what)
        return sum(len(t) for t in self.reqs.values())


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("setirax")
    made = {}

    def case(name, kind="sharp"):
        if (name, kind) not in made:
            made[(name, kind)] = Case(name, tmp, kind)
        return made[(name, kind)]
    return case


def runner_for(case, dtype, steps, page_size=None, use_graph=True, **kw):
    from minivllm_amd.engine.trace import TraceRunner
    return TraceRunner(case.dir, dtype, trace_tools.max_live_tokens(steps), page_size=page_size or case.page,
                       use_graph=use_graph, **kw)


def prompt_lens_of(case):
    return {rid: max(2, len(t) - 12) if len(t) > 3 else len(t) for rid, t in case.reqs.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_whole(cases, name, dtype):
    for case in (cases(name, kind) for kind in GAINS):
        steps = trace_tools.whole(case.reqs)
        got = trace_tools.collect(steps, runner_for(case, dtype, steps).run_step)
        assert len(got) == case.check(got, dtype, f"{name} {case.kind} whole")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("use_graph", [True, False])
def test_tail_decode(cases, name, dtype, use_graph):
    """The last 40 tokens one by one, from the states and the caches that the prompt left, every run of a layer with its own."""
    case = cases(name)
    steps = trace_tools.tail_decode(case.reqs, tail=40)
    got = trace_tools.collect(steps, runner_for(case, dtype, steps, use_graph=use_graph).run_step)
    case.check(got, dtype, f"{name} last 40 one by one (graph={use_graph})")
    assert all((rid, len(toks) - 1) in got for rid, toks in case.reqs.items())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("page_size", ["own", 4])
def test_portions(cases, name, dtype, page_size):
    """Portions of 7, 5, 3, 2, 11, 2, 17, 2, 4 tokens: shorter than the convolutions reach back, across pages."""
    case = cases(name)
    steps = trace_tools.portions(case.reqs)
    ps = case.page if page_size == "own" else page_size
    got = trace_tools.collect(steps, runner_for(case, dtype, steps, page_size=ps).run_step)
    assert len(got) == case.check(got, dtype, f"{name} portions (page {ps})")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_mixed(cases, name, dtype):
    """Up to three live requests on three state slots and pages for exactly the live tokens: slots and pages change hands,
    and what the request before left in a slot must not leak."""
    for case in (cases(name, kind) for kind in GAINS):
        for seed in (0, 1):
            steps = trace_tools.mixed(case.reqs, prompt_lens_of(case), max_live=3, seed=seed)
            runner = runner_for(case, dtype, steps, max_live=3)
            got = trace_tools.collect(steps, runner.run_step)
            assert len(got) == case.check(got, dtype, f"{name} {case.kind} mixed seed {seed}")
            runner.manager.check_invariants()
            assert not runner.manager.seqs and runner.manager.slots.num_free == 3
            for pool in runner.manager.pools:
                assert pool.num_free == pool.num_pages


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_steps_with_prompt_portions_from_graphs(cases, name, dtype):
    """Every entry wants its last row only, as generation does: such steps are replayed from graphs per size class, padded
    with inert rows and sequences that must leave every state alone."""
    case = cases(name)
    cuttings = {"portions": trace_tools.portions(case.reqs),
                "mixed": trace_tools.mixed(case.reqs, prompt_lens_of(case), max_live=4, seed=4)}
    for what, steps in cuttings.items():
        steps = trace_tools.only_last_rows(steps)
        runner = runner_for(case, dtype, steps)
        got = trace_tools.collect(steps, runner.run_step)
        case.check(got, dtype, f"{name} {what} from graphs")
        assert len(got) == sum(len(st["entries"]) for st in steps)
        assert runner.executor.model.graph_safe and list(runner.executor._mixed_graphs)
        eager = trace_tools.collect(steps, runner_for(case, dtype, steps, use_graph=False).run_step)
        worst = max(rel_err(got[k], eager[k]) for k in got)
        assert worst <= (TOL_F32 if dtype == "float32" else bounds(dtype, case.moved[dtype])[0]), f"graphs against eager steps: {worst:.3e}"


@pytest.mark.parametrize("name", ["A", "B", "C", "E"])
def test_decode_graph_recorded_with_fewer_requests(cases, name):
    """The graph for four sequences, recorded by a step of three, serves a later step of four (sizes whose single tokens no
    one-launch kernel serves among them)."""
    case = cases(name, "mild")
    toks = [random_tokens(case.cfg, 30, seed=70 + i) for i in range(4)]
    want = [plain_logits(case.cfg, case.weights, t) for t in toks]
    steps = [{"step": 0, "entries": [{"id": f"r{i}", "tokens": t[:20], "want": [19]} for i, t in enumerate(toks)], "end": []}]
    for k, who in enumerate([(0, 1, 2), (0, 1, 2, 3), (3, 1, 0), (2, 3, 1, 0), (3, 2), (0, 1, 2, 3)]):
        had = [sum(e["id"] == f"r{i}" for st in steps[1:] for e in st["entries"]) for i in range(4)]
        steps.append({"step": k + 1, "entries": [{"id": f"r{i}", "tokens": [toks[i][20 + had[i]]], "want": [0]} for i in who], "end": []})
    got = trace_tools.collect(steps, runner_for(case, "float32", steps).run_step)
    judge([rel_err(row, want[int(rid[1:])][pos]) for (rid, pos), row in got.items()], "float32", case.moved["float32"], "graph of four")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "F", "G"])
def test_mixed_with_poisoned_pages(cases, name, dtype):
    """Pages are filled with NaN when they change hands: a kernel that reads a slot nobody has written since puts NaN into
    the logits."""
    case = cases(name)
    steps = trace_tools.mixed(case.reqs, prompt_lens_of(case), max_live=4, seed=2)
    runner = runner_for(case, dtype, steps, poison_pages=True)
    got = trace_tools.collect(steps, runner.run_step)
    assert len(got) == case.check(got, dtype, f"{name} mixed on poisoned pages")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_first_tokens_and_short_requests(cases, name, dtype):
    case = cases(name)
    reqs = {"one": case.reqs["r0"][:1], "two": case.reqs["r0"][:2], "three": case.reqs["r1"][:3]}
    steps = trace_tools.whole(reqs) + [dict(st, step=st["step"] + 3) for st in trace_tools.tail_decode(
        {"again": case.reqs["r0"][:6]}, tail=5)]
    got = trace_tools.collect(steps, runner_for(case, dtype, steps).run_step)
    assert len(got) == 1 + 2 + 3 + 6
    judge([rel_err(row, case.want["r1" if rid == "three" else "r0"][pos]) for (rid, pos), row in got.items()], dtype, case.moved[dtype],
          "first tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_long_decoding(cases, name, dtype):
    """Four tokens of prompt, then 250 tokens one by one: windows and many pages pass, the states run on."""
    case = cases(name, "mild")
    toks = random_tokens(case.cfg, 254, seed=9)
    want = plain_logits(case.cfg, case.weights, toks)
    steps = trace_tools.tail_decode({"long": toks}, tail=250)
    got = trace_tools.collect(steps, runner_for(case, dtype, steps).run_step)
    assert len(got) == 251
    judge([rel_err(row, want[pos]) for (_, pos), row in got.items()], dtype, moved_by(dtype, case.cfg, case.weights, toks, want), "long decoding")


def edge_model(window):
    """One softmax layer of each kind with a window, sizes that the MFMA kernels serve in bfloat16, and scores so steep that a
    key a query looks for takes nearly all of the weight."""
    cfg = model(256, 128, 1e-6, 20.0, [
        latent(4, 64, 64, 64, 0.6, window, None),
        parallel((4, 2, 64, 64, 0.9, 50.0, window, 1, (16, 1e6, (8.0, 1.0, 4.0, 64.0))), (2, 32, 32, 1.0, 8), dense(96), (1.0, 0.1))])
    w = make_weights(cfg, seed=12)
    # queries read one half of a row and keys the other: token 255 looks for token 254
    basis = torch.linalg.qr(torch.randn(128, 128, generator=torch.Generator().manual_seed(1)))[0]
    ask, tell = basis[:64], basis[64:]
    w["l0.mix.dkv"], w["l0.mix.uk"], w["l0.mix.q"] = tell, torch.eye(64).repeat(4, 1), ask.repeat(4, 1)
    w["l1.mix.left.q"], w["l1.mix.left.k"] = ask.repeat(4, 1), tell.repeat(2, 1)
    for side in "qk":
        w[f"l1.mix.left.{side}.conv"] = torch.ones_like(w[f"l1.mix.left.{side}.conv"])
    mark = torch.randn(64, generator=torch.Generator().manual_seed(2))
    w["embed"][255], w["embed"][254] = 2.0 * mark @ ask, 2.0 * mark @ tell
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    return cfg, w


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [16, 31, 64])
def test_keys_just_inside_and_just_outside_a_window(tmp_path, dtype, window):
    """The key a query singles out ``window - 1`` positions before it (just inside), ``window`` positions before it
    (just outside) and far before it, at places around pages' borders; in a prompt, in a portion of two tokens, and decoded."""
    cfg, weights = edge_model(window)
    path = write_model_dir(str(tmp_path / "model"), stored_config(cfg), weights)
    from minivllm_amd.engine.trace import TraceRunner
    w = as_f64(weights)
    reqs, marks = {}, {}
    for i, back in enumerate((window - 1, window, window + 1, 4 * window)):
        for at in (5 * window, 5 * window + 1):
            toks = random_tokens(cfg, at + 3, seed=50 + i)
            toks = [t % 254 for t in toks]
            toks[at - back], toks[at] = 254, 255
            reqs[f"{back}.{at}"], marks[f"{back}.{at}"] = toks, at
    want = {rid: plain.forward(cfg, w, toks)[0].numpy() for rid, toks in reqs.items()}
    wider = {rid: plain.forward(edge_model(window + 1)[0], w, toks)[0].numpy() for rid, toks in reqs.items()}
    narrower = {rid: plain.forward(edge_model(window - 1)[0], w, toks)[0].numpy() for rid, toks in reqs.items()}
    moved = [e for rid, toks in reqs.items() for e in moved_by(dtype, cfg, weights, toks, want[rid])]
    most = bounds(dtype, moved)[0]
    for rid, at in marks.items():                      # the mistake of one key would show in the marked row
        back = int(rid.split(".")[0])
        other = narrower if back == window - 1 else wider
        if back in (window - 1, window):
            assert rel_err(other[rid][at], want[rid][at]) > 1.5 * most, (rid, rel_err(other[rid][at], want[rid][at]), most)
    steps, n = [], 0
    for rid, toks in reqs.items():
        at, rows = marks[rid], list(range(len(toks)))
        cuts = {"whole": [len(toks)], "two": [at - 1, 2, 2], "one": [at, 1, 1, 1]}
        for how, sizes in cuts.items():
            p = 0
            for k in sizes:
                steps.append({"step": n, "entries": [{"id": f"{how}:{rid}", "tokens": toks[p:p + k], "want": rows[:k]}],
                              "end": [f"{how}:{rid}"] if p + k == len(toks) else []})
                p, n = p + k, n + 1
            assert p == len(toks)
    got = trace_tools.collect(steps, TraceRunner(path, dtype, trace_tools.max_live_tokens(steps), page_size=16).run_step)
    assert len(got) == 3 * sum(len(t) for t in reqs.values())
    judge([rel_err(row, want[rid.split(":")[1]][pos]) for (rid, pos), row in got.items()], dtype, moved, f"edges of a window of {window}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompt(tmp_path, dtype):
    """A prompt of 1,100 tokens through sizes that the MFMA kernels serve, one softmax layer without a window: whole, and the
    last 40 tokens one by one behind a prompt fed in two portions. A token of the first page is repeated at the end."""
    cfg = model(400, 128, 1e-6, 20.0, [
        latent(6, 32, 64, 160, 0.3, None, dense(256)),
        parallel((8, 2, 64, 64, 0.3, 25.0, 200, 3, (32, 1e5, (8.0, 1.0, 4.0, 512.0))), (3, 64, 64, 16.0, 24), dense(128)),
        unit(96, 3, 4, None)])
    cfg["layers"].append(dict(cfg["layers"][1], weights_of=1))
    weights = make_weights(cfg, seed=8)
    path = write_model_dir(str(tmp_path / "model"), stored_config(cfg), weights)
    toks = random_tokens(cfg, 1100, seed=77)
    toks[1070] = toks[15]
    w = as_f64(weights)
    want = plain.forward(cfg, w, toks)[0].numpy()
    rows = [0, 1, 15, 16, 47, 48, 199, 200, 201, 511, 512, 1023, 1024, 1059, 1060, 1070, 1099]
    moved = moved_by(dtype, cfg, weights, toks, want, rows=rows + list(range(1000, 1100)))
    steps = [{"step": 0, "entries": [{"id": "w", "tokens": toks, "want": rows}], "end": ["w"]},
             {"step": 1, "entries": [{"id": "d", "tokens": toks[:1000], "want": [999]}], "end": []},
             {"step": 2, "entries": [{"id": "d", "tokens": toks[1000:1060], "want": [59]}], "end": []}]
    steps += [{"step": 3 + i, "entries": [{"id": "d", "tokens": [toks[1060 + i]], "want": [0]}],
               "end": ["d"] if i == 39 else []} for i in range(40)]
    from minivllm_amd.engine.trace import TraceRunner
    got = trace_tools.collect(steps, TraceRunner(path, dtype, trace_tools.max_live_tokens(steps)).run_step)
    assert len(got) == len(rows) + 2 + 40
    judge([rel_err(row, want[pos]) for (_, pos), row in got.items()], dtype, moved, "1,100 tokens")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_residual_after_every_layer(cases, dtype):
    """The residual stream behind each run of a layer, in one prompt step, against the plain model's."""
    case = cases("A")
    toks = case.reqs["r0"]
    want = plain.forward(case.cfg, as_f64(case.weights), toks, keep_layers=True)[2]
    steps = trace_tools.whole({"r": toks})
    runner = runner_for(case, dtype, steps, use_graph=False)
    kept = []
    for block in {id(b): b for b in runner.executor.model.blocks}.values():
        def forward(stream, ctx, call, *a, _run=block.forward, **kw):
            _run(stream, ctx, call, *a, **kw)
            assert stream.delta is None
            kept.append(stream.resid.clone())
        block.forward = forward
    runner.run_step(steps[0])
    assert len(kept) == len(want)
    for i, (x, y) in enumerate(zip(kept, want)):
        err = float((x[:len(toks)].double().cpu() - y).abs().max() / y.abs().max())
        assert err <= (2e-5 if dtype == "float32" else 6e-2), f"after run {i}: {err:.2e}"


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Sizes, orders of layers, shared tensors and options drawn at random (every second time sizes that the MFMA kernels serve),
    mixed steps on few pages, through both types."""
    from minivllm_amd.engine.trace import TraceRunner
    rng = np.random.default_rng(500 + seed)
    cfg = random_config(rng, fast_sizes=seed % 2 == 0)
    weights = make_weights(cfg, seed=seed)
    path = write_model_dir(str(tmp_path / "model"), stored_config(cfg), weights)
    reqs = {f"r{i}": random_tokens(cfg, int(n), seed=10 * seed + i) for i, n in enumerate(rng.integers(2, 90, size=4))}
    want = {rid: plain_logits(cfg, weights, toks) for rid, toks in reqs.items()}
    prompt_lens = {rid: max(2, len(t) - 9) if len(t) > 3 else len(t) for rid, t in reqs.items()}
    steps = trace_tools.mixed(reqs, prompt_lens, max_live=3, seed=seed, max_portion=40)
    for dtype in ("float32", "bfloat16"):
        moved = [e for rid, toks in reqs.items() for e in moved_by(dtype, cfg, weights, toks, want[rid])]
        runner = TraceRunner(path, dtype, trace_tools.max_live_tokens(steps), page_size=int(rng.choice([4, 8, 16, 32, 64])))
        got = trace_tools.collect(steps, runner.run_step)
        assert len(got) == sum(len(t) for t in reqs.values())
        judge([rel_err(row, want[rid][pos]) for (rid, pos), row in got.items()], dtype, moved,
              f"seed {seed}, {[l['type'] for l in cfg['layers']]}")
        runner.manager.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation(cases, name, dtype):
    """Through LLM.generate: the scheduler cuts prompts into portions of at most 24 tokens, batches them with decoding
    requests, runs decode steps in rows from graphs, and preempts when pages run out."""
    from minivllm_amd import LLM, SamplingParams
    case = cases(name, "mild")
    llm = LLM(model=case.dir, dtype=dtype, kv_cache_block_size=case.page, kv_cache_num_blocks=40, max_model_len=320,
              max_num_batched_tokens=48, max_num_batched_seqs=4, prefill_chunk=24)
    prompts = [random_tokens(case.cfg, n, seed=n) for n in (5, 61, 33, 1, 90, 18)]
    sp = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    outs = llm.generate(prompts, sp, use_tqdm=False)
    assert [o.prompt_token_ids for o in outs] == prompts and all(len(o.token_ids) == 40 for o in outs)
    clear = near = 0
    for out in outs:
        seq = list(out.prompt_token_ids) + list(out.token_ids)
        logits = plain_logits(case.cfg, case.weights, seq)
        tol = bounds(dtype, moved_by(dtype, case.cfg, case.weights, seq, logits))[0]
        for t, tok in enumerate(out.token_ids):
            row = logits[len(out.prompt_token_ids) + t - 1]
            slack = 2 * tol * float(np.abs(row).max())
            assert row[tok] >= row.max() - slack, f"token {t}: {tok} scores {row[tok]}, the best {row.max()}"
            if row.max() - np.partition(row, -2)[-2] > slack:
                assert tok == int(row.argmax())
                clear += 1
            else:
                near += 1
    print(f"greedy {name} [{dtype}]: {clear} tokens decided by a clear margin, {near} near ties")
    assert clear > near if dtype == "float32" else True
    llm.manager.check_invariants()


def test_command_lines(cases, tmp_path):
    """``run.py --random-model setirax-tiny`` prints completions, and ``bin/trace_run`` as a program, fed a trace on its
    standard input, writes the logits the plain model gives (four state slots by default)."""
    import ast
    import json
    import os
    import re
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, os.path.join(root, "run.py"), "--random-model", "setirax-tiny", "--seed", "3",
                           "--prompt-ids", "5,17,3", "--prompt-ids", "200", "--max-tokens", "5", "--temperature", "0",
                           "--ignore-eos", "--max-model-len", "64", "--kv-cache-num-blocks", "16",
                           "--max-num-batched-tokens", "64", "--max-num-batched-seqs", "4"],
                          capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    completions = re.findall(r"Completion:\s*(\[.*?\])", proc.stdout, re.S)
    assert len(completions) == 2 and all(len(ast.literal_eval(c)) == 5 for c in completions)

    case = cases("D", "mild")
    steps = trace_tools.mixed(case.reqs, prompt_lens_of(case), max_live=4, seed=7)
    out = tmp_path / "logits"
    proc = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", case.dir, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", str(trace_tools.max_live_tokens(steps))],
                          input="".join(json.dumps(st) + "\n" for st in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done ")] == [f"done {st['step']}" for st in steps]
    got = trace_tools.collect(steps, lambda st: (np.fromfile(out / f"{st['step']}.f32", dtype="<f4").reshape(
        -1, case.cfg["vocab"]) if any(e["want"] for e in st["entries"]) else None))
    case.check(got, "float32", "D mixed through bin/trace_run")
