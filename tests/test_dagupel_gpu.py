"""The Dagupel design served by the engine against its plain restatement (oracle/dagupel.py): whole prompts, portions,
token-by-token decoding, mixed batches, reused cache blocks, window and block borders, graphs, generation, trace replay.

Tolerances: row error relative to the logits' spread.  float32 2e-5; bfloat16 6e-2 (sharp attention on random weights,
16-bit operands); a key too many or too few costs 0.1 .. 1 on the rows it touches."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from .dagupel_common import CONFIGS, as_f64, config, mixer, row_errors, weights, write_model
from oracle import dagupel as ref

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 2e-5, torch.bfloat16: 6e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
_cache = {}


def _model(name):
    """(config, tensors, tokens, reference logits) of a named configuration, computed once."""
    if name not in _cache:
        cfg, sharp = CONFIGS[name]
        t = weights(cfg, 11, sharp)
        n = {"tiny": 70, "large": 60}.get(name, 200)
        tokens = np.random.default_rng(5).integers(0, cfg["vocab"], n).tolist()
        _cache[name] = cfg, t, tokens, ref.forward(cfg, as_f64(t), tokens)
    return _cache[name]


def row_errors_at(got, want, start, n):
    d = got - want[start:start + n]
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())


def _engine(cfg, tensors, dtype, n_blocks=16, block_size=16, n_states=64, **options):
    from scalellm_amd.checkpoint import Checkpoint
    from scalellm_amd.engine import EngineOptions, LLMEngine
    from scalellm_amd.registry import ModelLimits, model_class
    cls = model_class(cfg["architecture"])
    model = cls.from_checkpoint(cfg, Checkpoint(dict(tensors)), ModelLimits(n_blocks, block_size, dtype, "cuda", n_states))
    return LLMEngine(model, n_blocks, block_size, "cuda", EngineOptions(**options))


def _run(engine, entries):
    """entries: [(sequence, n)] -> logits of every new token, per entry."""
    _, logits = engine.run_entries(entries, {i: range(n) for i, (_, n) in enumerate(entries)})
    out = logits.float().cpu().numpy()
    ends = np.cumsum([0] + [n for _, n in entries])
    return [out[a:b] for a, b in zip(ends, ends[1:])]


def _seq(name, tokens):
    from scalellm_amd.engine import Sequence
    return Sequence(name, list(tokens))


def _feed(engine, tokens, cuts):
    """A sequence alone, in portions of the given sizes (the last size repeats)."""
    s, out, k = _seq("s", tokens), [], 0
    while s.n_cached < len(tokens):
        n = min(cuts[min(k, len(cuts) - 1)], len(tokens) - s.n_cached)
        out.append(_run(engine, [(s, n)])[0])
        k += 1
    s.release(engine.allocator)
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_portions_and_decoding(name, dtype):
    cfg, t, tokens, want = _model(name)
    engine = _engine(cfg, t, dtype)
    for cuts in ([len(tokens)], [37, 2, 16, 5, 64], [17, 1], [2], [1]):
        if cuts == [2]:
            tokens_, want_ = tokens[:60], want[:60]
        else:
            tokens_, want_ = tokens, want
        err = row_errors(_feed(engine, tokens_, cuts), want_)
        assert err.max() < TOL[dtype], (cuts, int(err.argmax()), err.max())
        assert engine.allocator.n_free == engine.allocator.n_blocks


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_residual_stream_after_every_layer(name):
    cfg, t, tokens, _ = _model(name)
    want, got = [], []
    ref.forward(cfg, as_f64(t), tokens[:40], want)
    engine = _engine(cfg, t, torch.float32)
    engine.model.on_layer = lambda i, x: got.append((i, x.cpu().numpy().copy()))
    _run(engine, [(_seq("s", tokens[:40]), 40)])
    assert [i for i, _ in got] == list(range(len(cfg["layers"])))
    for (i, g), w in zip(got, want):
        np.testing.assert_allclose(g, w, atol=2e-5 * np.abs(w).max(), err_msg=f"layer {i}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", ["odd", "wide", "deep"])
def test_mixed_batches_and_reused_blocks(name, dtype):
    """Portions of some beside single tokens of others, sequences that pause, end and come back on blocks others held:
    every row as if its sequence were alone."""
    cfg, t, tokens, _ = _model(name)
    rng = np.random.default_rng(8)
    streams = {k: rng.integers(0, cfg["vocab"], n).tolist() for k, n in (("a", 150), ("b", 90), ("c", 33), ("d", 118), ("e", 61))}
    want = {k: ref.forward(cfg, as_f64(t), s) for k, s in streams.items()}
    engine = _engine(cfg, t, dtype, n_blocks=24, block_size=16)
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
    assert engine.allocator.n_free == 24


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window", [5, 16, 17, 64, 65, 130])
def test_window_edges_around_block_borders(window, dtype):
    """A key that takes nearly all of the soft-max, met by queries at every distance around the window's edge: one
    marked token writes a key the others' queries point at.  Seen last at distance window - 1."""
    W, K = 64, 64
    m = mixer(2, 16, 4, 16, K, window, scale=1.0, base=1e9)
    cfg = config(W, [(m, None, 0)], vocab=20, max_positions=256)
    t = weights(cfg, 3)
    t["pos"].zero_()
    t["embed"][7] = 0
    t["embed"][7, 0] = 8.0            # the marked token is alone on its axis
    t["embed"][:7, 0] = t["embed"][8:, 0] = 0
    t["l0.norm1"].fill_(1.0)
    t["l0.mix.dkv"][:, 0] = 0
    t["l0.mix.dkv"][0] = 0
    t["l0.mix.dkv"][0, 0] = 1.0       # its latent has one big entry, which no other token's has
    t["l0.mix.uk"].zero_()
    t["l0.mix.uk"].view(2, 16, K)[:, 0, 0] = 1.0
    t["l0.mix.q"].view(2, 20, W)[:, 0] = 0
    t["l0.mix.q"].view(2, 20, W)[:, 0, 1] = 1.0    # every other token's query looks that way
    t["l0.mix.g"].zero_()
    for other in range(20):
        if other != 7:
            t["embed"][other, 1] = 6.0 + float(t["embed"][other, 1])
    tokens = np.random.default_rng(1).integers(8, 20, 200)
    for place in (0, 3, 15, 16, 17, 31, 40):
        seq = tokens.copy()
        seq[place] = 7
        plain = ref.forward(cfg, as_f64(t), tokens.tolist())
        want = ref.forward(cfg, as_f64(t), seq.tolist())
        moved = row_errors(plain, want)
        last = min(place + window - 1, 199)
        if place < last < 199:        # (the construction shows the edge)
            assert moved[place + 1:last + 1].min() > 0.1 and moved[last + 1:].max() < 1e-9
        engine = _engine(cfg, t, dtype, block_size=16)
        for cuts in ([200], [place + 1, max(window - 2, 1), 1], [64, 1]):
            err = row_errors(_feed(engine, seq.tolist(), cuts), want)
            assert err.max() < TOL[dtype], (place, cuts, int(err.argmax()), err.max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_rows_do_not_depend_on_the_batch(dtype):
    """The same sequence alone and beside many others, on other blocks: equal up to rounding."""
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
    """Prompts longer than the step budget, more requests than fit at once, decode batches from captured graphs or eager:
    token ids equal the restatement's (float32)."""
    cfg, t, _, _ = _model("odd")
    from scalellm_amd.sampling import SamplingParams
    rng = np.random.default_rng(3)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (30, 3, 47, 1, 12)]
    engine = _engine(cfg, t, torch.float32, n_blocks=16, block_size=8, max_seqs=3, max_step_tokens=24, graph_batch_sizes=graphs,
                     graph_max_seq_len=128)
    engine.capture_graphs()
    out = engine.generate(prompts, SamplingParams(max_tokens=9))
    for p, got in zip(prompts, out):
        want, margins = _greedy(cfg, t, p, 9)
        assert min(margins) > 1e-3
        assert got == want
    assert engine.allocator.n_free == 16
    assert (engine.runner.num_graph_replayed > 0) == bool(graphs)


def test_graph_replays_equal_eager_steps():
    """bf16 decode batches through ModelRunner graphs, several replays with eager steps between them, long decoding."""
    cfg, t, tokens, _ = _model("wide")
    outs = []
    for graphs in ([], [2]):
        engine = _engine(cfg, t, torch.bfloat16, n_blocks=40, block_size=16, graph_batch_sizes=graphs, graph_max_seq_len=256)
        engine.capture_graphs()
        a, b, c = _seq("a", tokens), _seq("b", tokens[::-1]), _seq("c", tokens[5:])
        rows = [_run(engine, [(a, 60)])[0], _run(engine, [(b, 33)])[0]]
        for k in range(100):
            _, logits = engine.run_entries([(a, 1), (b, 1)])
            rows.append(logits.float().cpu().numpy())
            if k % 10 == 3:
                rows += _run(engine, [(c, 18)])
        outs.append(np.concatenate(rows))
        assert engine.runner.num_graph_replayed == (100 if graphs else 0)
    assert row_errors(outs[1], outs[0].astype(np.float64)).max() < 1e-2


def test_graph_replays_of_a_batch_the_vendor_products_serve():
    """40 decode rows: the projections are library products inside the graph; every replay equals the eager step."""
    cfg, t, _, _ = _model("wide")
    rng = np.random.default_rng(2)
    prompts = [rng.integers(0, cfg["vocab"], 20 + k).tolist() for k in range(40)]
    outs = []
    for graphs in ([], [40]):
        engine = _engine(cfg, t, torch.bfloat16, n_blocks=200, block_size=16, graph_batch_sizes=graphs, graph_max_seq_len=128)
        engine.capture_graphs()
        seqs = [_seq(k, p) for k, p in enumerate(prompts)]
        _run(engine, [(s, len(s.tokens) - 9) for s in seqs])
        rows = []
        for k in range(9):
            rows.append(engine.run_entries([(s, 1) for s in seqs])[1].float().cpu().numpy())
            if k % 3 == 1:
                _run(engine, [(_seq("x", prompts[3]), 5)])
        outs.append(np.concatenate(rows))
        assert engine.runner.num_graph_replayed == (9 if graphs else 0)
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


def test_llama_step_through_the_same_engine():
    """The engine serves the other step model as well: generation equals stepping it by hand."""
    from scalellm_amd.decode import LlamaDecodeStep, LlamaShape
    from scalellm_amd.engine import EngineOptions, LLMEngine
    from scalellm_amd.sampling import SamplingParams
    shape = LlamaShape.tiny()
    outs = []
    for budget in (64, 8):
        model = LlamaDecodeStep(shape, 64, 32, 16, dtype=torch.bfloat16, device="cuda", seed=0, group_size=128)
        engine = LLMEngine(model, 32, 16, "cuda", EngineOptions(max_seqs=4, max_step_tokens=budget))
        outs.append(engine.generate([[1, 2, 3, 4, 5, 6, 7, 8, 9, 10, 11], [400, 5]], SamplingParams(max_tokens=6)))
    assert all(len(x) == 6 and 0 <= min(x) and max(x) < shape.vocab for o in outs for x in o)
    # (other batches, other kernels and roundings: the first tokens agree, later ones may part at a near tie)
    assert [x[0] for x in outs[0]] == [x[0] for x in outs[1]]


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
    assert sorted(os.listdir(tmp_path / "out")) == ["0.f32", "1.f32", "3.f32"]
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
