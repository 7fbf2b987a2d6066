"""The Vebusun design served by the engine against its plain restatement (oracle/vebusun.py): whole prompts, portions,
token-by-token decoding, mixed batches, reused cache blocks and state slots, window borders, graphs, generation, replay.

Tolerances: row error relative to the logits' spread.  float32 5e-5; bfloat16 8e-2 (sharp attention on random weights,
16-bit operands); a key too many or too few, or a state that is lost, costs 0.1 .. 1 on the rows it touches."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from .test_dagupel_gpu import _engine, _feed, _run, _seq, row_errors_at
from .vebusun_common import CONFIGS, as_f64, config, delta, lightning, parallel, row_errors, weights, window, write_model
from oracle import vebusun as ref

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 5e-5, torch.bfloat16: 8e-2}
BOTH = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
_cache = {}


def _model(name):
    """(config, tensors, tokens, reference logits) of a named configuration, computed once."""
    if name not in _cache:
        cfg = CONFIGS[name]
        t = weights(cfg, 11)
        n = {"tiny": 70, "large": 90}.get(name, 230)
        tokens = np.random.default_rng(5).integers(0, cfg["vocab"], n).tolist()
        _cache[name] = cfg, t, tokens, ref.forward(cfg, as_f64(t), tokens)
    return _cache[name]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_portions_and_decoding(name, dtype):
    cfg, t, tokens, want = _model(name)
    engine = _engine(cfg, t, dtype)
    for cuts in ([len(tokens)], [37, 2, 16, 5, 64], [17, 1], [2], [130, 3, 2, 1], [1]):
        n = 60 if cuts in ([2], [1]) else len(tokens)
        err = row_errors(_feed(engine, tokens[:n], cuts), want[:n])
        assert err.max() < TOL[dtype], (cuts, int(err.argmax()), err.max())
        assert engine.allocator.n_free == engine.allocator.n_blocks and engine.allocator.n_free_states == engine.allocator.n_states


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_residual_stream_after_every_layer_run(name):
    cfg, t, tokens, _ = _model(name)
    want, got = [], []
    ref.forward(cfg, as_f64(t), tokens[:40], want)
    engine = _engine(cfg, t, torch.float32)
    engine.model.on_layer = lambda i, x: got.append((i, x.cpu().numpy().copy()))
    _run(engine, [(_seq("s", tokens[:40]), 40)])
    assert [i for i, _ in got] == list(range(len(ref.layer_runs(cfg)))) and len(got) == len(want)
    for (i, g), w in zip(got, want):
        np.testing.assert_allclose(g, w, atol=3e-5 * np.abs(w).max(), err_msg=f"layer run {i}")


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_mixed_batches_reused_blocks_and_states(name, dtype):
    """Portions of some beside single tokens of others, sequences that pause, end and come back on blocks and state slots
    others held: every row as if its sequence were alone."""
    cfg, t, _, _ = _model(name)
    rng = np.random.default_rng(8)
    streams = {k: rng.integers(0, cfg["vocab"], n).tolist() for k, n in (("a", 150), ("b", 90), ("c", 33), ("d", 118), ("e", 61))}
    want = {k: ref.forward(cfg, as_f64(t), s) for k, s in streams.items()}
    engine = _engine(cfg, t, dtype, n_blocks=24, block_size=16, n_states=3)
    live, waiting, worst = {}, list(streams) * 2, 0.0
    while live or waiting:
        while waiting and len(live) < 3 and waiting[0] not in live:
            k = waiting.pop(0)
            live[k] = _seq(k, streams[k])
        entries = []
        for k in rng.permutation(sorted(live)):
            if len(entries) and rng.random() < 0.25:
                continue   # (left out of this step)
            left = len(streams[k]) - live[k].n_cached
            n = 1 if rng.random() < 0.5 else int(rng.integers(2, 60))
            entries.append((live[k], min(n, left)))
        at = [s.n_cached for s, _ in entries]
        for (s, n), c, got in zip(entries, at, _run(engine, entries)):
            worst = max(worst, float(row_errors_at(got, want[s.id], c, n).max()))
        for s, _ in entries:
            if s.n_cached == len(streams[s.id]):
                live.pop(s.id).release(engine.allocator)
    assert worst < TOL[dtype], worst
    assert engine.allocator.n_free == 24 and engine.allocator.n_free_states == 3


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("size,keep", [(5, 3), (16, 1), (17, 0), (64, 6), (65, 16), (130, 17)])
def test_window_and_kept_token_edges(size, keep, dtype):
    """A key that takes nearly all of the soft-max, met by queries at every distance: one marked token writes a key the
    others' queries point at.  Kept tokens are seen for ever, others last at distance size - 1."""
    W, D = 64, 16
    left = window(2, 1, D, D, 4, size, keep, softcap=50.0, scale=1.0)
    cfg = config(W, [(parallel(left, lightning(8, 8, (0.9,)), 1.0, 0.0), None)], vocab=20, embedding_scale=1.0, residual_mult=1.0)
    t = weights(cfg, 3, sharp=1.0)
    t["embed"][:, :2] = 0
    t["embed"][7, 0] = t["embed"][8:, 1] = 8.0                 # the marked token alone on one axis, the others on the next
    for n in ("l0.norm1", "l0.norm1.b"):
        t[n].fill_(1.0 if n.endswith("norm1") else 0.0)
    t["l0.norm1.alpha"].fill_(1.0)
    q, k = t["l0.mix.left.q"].view(2, D, W), t["l0.mix.left.k"].view(1, D, W)
    for x, axis in ((q, 1), (k, 0)):                           # (the last dimension is not rotated)
        x.mul_(0.05)
        x[:, D - 1] = 0
        x[:, D - 1, axis] = 4.0
    t["l0.mix.left.q.norm"].fill_(1.0)
    t["l0.mix.left.k.norm"].fill_(1.0)
    tokens = np.random.default_rng(1).integers(8, 20, 200)
    base = ref.forward(cfg, as_f64(t), tokens.tolist())
    for place in sorted({0, max(keep - 1, 0), keep, 15, 16, 17, 40}):
        seq = tokens.copy()
        seq[place] = 7
        want = ref.forward(cfg, as_f64(t), seq.tolist())
        moved = row_errors(base, want)
        last = 199 if place < keep else min(place + size - 1, 199)
        if place < last:                                       # (the construction shows the edge)
            assert moved[place + 1:last + 1].min() > 0.1
        assert last == 199 or moved[last + 1:].max() < 1e-9
        engine = _engine(cfg, t, dtype, block_size=16)
        for cuts in ([200], [place + 1, max(size - 2, 1), 1], [64, 1], [2, 30]):
            err = row_errors(_feed(engine, seq.tolist(), cuts), want)
            assert err.max() < TOL[dtype], (place, cuts, int(err.argmax()), err.max())


@pytest.mark.parametrize("dtype", BOTH)
def test_a_first_token_is_remembered_by_the_recurrences(dtype):
    """Slow decays: what the first token wrote shows hundreds of tokens later, through portions and decoding."""
    cfg = config(48, [(delta(2, 1, 16, 16, 4), None), (parallel(window(1, 1, 8, 8, 4, 3, 0), lightning(8, 8, (0.999, 0.9995)), 0.0, 1.0), None)],
                 vocab=30, residual_mult=1.0)
    t = weights(cfg, 6)
    t["l0.mix.dt_bias"].fill_(-9.0)
    t["l0.mix.b"].mul_(0.1)
    t["l0.mix.b"][:, 0] = 8.0      # the first token writes with a step size near 1, the others hardly at all
    t["embed"][:, 0] = -4.0
    t["embed"][0, 0] = 4.0
    rng = np.random.default_rng(2)
    tokens = rng.integers(1, 30, 400).tolist()
    other = [0] + tokens[1:]
    want, plain = ref.forward(cfg, as_f64(t), other), ref.forward(cfg, as_f64(t), tokens)
    assert row_errors(plain, want)[300:].mean() > 0.2   # (it shows)
    engine = _engine(cfg, t, dtype, n_blocks=32)
    for cuts in ([400], [1], [100, 3, 290, 1]):
        err = row_errors(_feed(engine, other, cuts), want)
        # (a read-out near zero is blown up by its norm, roundings included: the 16-bit rows are taken together)
        assert err[300:].mean() < TOL[dtype] / 4 and (dtype == torch.bfloat16 or err.max() < TOL[dtype]), cuts


@pytest.mark.parametrize("dtype", BOTH)
def test_rows_do_not_depend_on_the_batch(dtype):
    """The same sequence alone and beside many others, on other blocks and slots: equal up to rounding."""
    cfg, t, tokens, want = _model("wide")
    engine = _engine(cfg, t, dtype, n_blocks=80, block_size=16)
    others = [_seq(i, np.random.default_rng(i).integers(0, cfg["vocab"], 20 + 3 * i)) for i in range(12)]
    s = _seq("s", tokens)
    _run(engine, [(o, len(o.tokens) - 3) for o in others[:6]] + [(s, 120)] + [(o, len(o.tokens) - 3) for o in others[6:]])
    for k in range(3):
        got = _run(engine, [(o, 1) for o in others] + [(s, 1)])[-1]
        assert row_errors_at(got, want, 120 + k, 1).max() < TOL[dtype]


def _greedy(cfg, t, prompt, n):
    t64, out = as_f64(t), list(prompt)
    margins = []
    for _ in range(n):
        logits = ref.forward(cfg, t64, out)[-1]
        top = np.sort(logits)[-2:]
        margins.append((top[1] - top[0]) / logits.std())
        out.append(int(logits.argmax()))
    return out[len(prompt):], margins


@pytest.mark.parametrize("graphs", [[], [1, 2, 3]])
def test_greedy_generation_through_the_scheduler(graphs):
    """Prompts longer than the step budget, more requests than blocks and state slots hold at once, decode batches from
    captured graphs or eager: token ids equal the restatement's (float32)."""
    cfg, t, _, _ = _model("odd")
    from scalellm_amd.sampling import SamplingParams
    rng = np.random.default_rng(3)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (30, 3, 47, 1, 12)]
    engine = _engine(cfg, t, torch.float32, n_blocks=16, block_size=8, n_states=3, max_seqs=4, max_step_tokens=24, graph_batch_sizes=graphs,
                     graph_max_seq_len=128)
    engine.capture_graphs()
    out = engine.generate(prompts, SamplingParams(max_tokens=9))
    for p, got in zip(prompts, out):
        want, margins = _greedy(cfg, t, p, 9)
        assert min(margins) > 1e-3
        assert got == want
    assert engine.allocator.n_free == 16 and engine.allocator.n_free_states == 3
    assert (engine.runner.num_graph_replayed > 0) == bool(graphs)


@pytest.mark.parametrize("batch", [2, 40])
def test_graph_replays_equal_eager_steps(batch):
    """bf16 decode batches through ModelRunner graphs, replays with eager steps between them (40 rows: vendor products)."""
    cfg, t, tokens, _ = _model("wide")
    rng = np.random.default_rng(2)
    prompts = [rng.integers(0, cfg["vocab"], 100 + k % 7).tolist() for k in range(batch)]
    steps, outs = 60 if batch == 2 else 8, []
    for graphs in ([], [batch]):
        engine = _engine(cfg, t, torch.bfloat16, n_blocks=8 * batch + 8, block_size=16, graph_batch_sizes=graphs, graph_max_seq_len=256)
        engine.capture_graphs()
        seqs = [_seq(k, p) for k, p in enumerate(prompts)]
        rows = _run(engine, [(s, len(s.tokens) - steps) for s in seqs])
        c = _seq("c", tokens)
        for k in range(steps):
            rows.append(engine.run_entries([(s, 1) for s in seqs])[1].float().cpu().numpy())
            if k % 5 == 3:
                rows += _run(engine, [(c, 11)])
        outs.append(np.concatenate(rows))
        assert engine.runner.num_graph_replayed == (steps if graphs else 0)
    assert row_errors(outs[1], outs[0].astype(np.float64)).max() < 1e-2


def test_preempted_sequences_start_over():
    cfg, t, _, _ = _model("tiny")
    from scalellm_amd.sampling import SamplingParams
    rng = np.random.default_rng(4)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (14, 15, 9)]
    engine = _engine(cfg, t, torch.float32, n_blocks=7, block_size=8, max_seqs=3, max_step_tokens=64)
    out = engine.generate(prompts, SamplingParams(max_tokens=20))
    for p, got in zip(prompts, out):
        assert got == _greedy(cfg, t, p, 20)[0]
    assert engine.allocator.n_free == 7


def test_long_decoding():
    """Hundreds of decoded tokens, every one through the step kernels (float32)."""
    cfg, t, _, _ = _model("odd")
    tokens = np.random.default_rng(9).integers(0, cfg["vocab"], 420).tolist()
    want = ref.forward(cfg, as_f64(t), tokens)
    got = _feed(_engine(cfg, t, torch.float32, n_blocks=32), tokens, [3, 1])
    assert row_errors(got, want).max() < TOL[torch.float32]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program(tmp_path, dtype):
    cfg, t, tokens, want = _model("odd")
    write_model(tmp_path / "m", cfg, t)
    (tmp_path / "out").mkdir()
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": tokens[:50], "want": [0, 49]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": tokens[:20], "want": []}, {"id": "a", "tokens": tokens[50:51], "want": [0]}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": tokens[51:55], "want": []}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "c", "tokens": tokens[:90], "want": [89, 3]}, {"id": "b", "tokens": tokens[20:21], "want": [0]}],
         "end": ["b", "c"]}]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out",
                        str(tmp_path / "out"), "--max-tokens", "192"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    tol = TOL[getattr(torch, dtype)]
    for step, places in ((0, [0, 49]), (1, [50]), (3, [89, 3, 20])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(len(places), cfg["vocab"])
        for row, p_ in zip(got, places):
            assert row_errors_at(row[None], want, p_, 1).max() < tol, (step, p_)


def test_command_line_generates(tmp_path):
    cfg, t, _, _ = _model("odd")
    write_model(tmp_path / "m", cfg, t)
    p = subprocess.run([sys.executable, "-m", "scalellm_amd.generate", "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--prompt", "1,2,3", "--prompt", "9,8", "--max-tokens", "5"], cwd=ROOT, capture_output=True, text=True,
                       timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    got = [json.loads(ln)["tokens"] for ln in p.stdout.splitlines() if ln.startswith("{")]
    assert got == [_greedy(cfg, t, q, 5)[0] for q in ([1, 2, 3], [9, 8])]
