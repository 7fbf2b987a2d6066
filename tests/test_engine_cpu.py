"""Host logic around a step model, without a GPU: checkpoint reader, registry and configuration, rotary tables, block
allocation, step building, portion plans, scheduling, sampling."""
import json
import struct

import numpy as np
import pytest
import torch

from oracle import dagupel as ref
from scalellm_amd.checkpoint import Checkpoint, CheckpointError
from scalellm_amd.dagupel import DagupelConfig
from scalellm_amd.engine import BlockAllocator, EngineOptions, LLMEngine, OutOfBlocks, Scheduler, Sequence, StepBuilder
from scalellm_amd.latent_layers import LatentPlan, YarnScaling, rotary_table
from scalellm_amd.layers import Portion
from scalellm_amd.registry import ModelLimits, architecture_of, load_model, model_class
from scalellm_amd.sampling import Sampler, SamplingParams

from .dagupel_common import CONFIGS, config, mixer, weights, write_model


# ---- checkpoint, registry, configuration --------------------------------------------------------
def test_safetensors_round_trip_and_errors(tmp_path):
    t = {"a": torch.arange(6, dtype=torch.bfloat16).view(2, 3), "b": torch.tensor([3, -1], dtype=torch.int32),
         "c": torch.tensor([[0.5]], dtype=torch.float32)}
    write_model(tmp_path, {"architecture": "x"}, t)
    ck = Checkpoint.open(str(tmp_path / "model.safetensors"))
    assert sorted(ck.names()) == ["a", "b", "c"]
    for k, v in t.items():
        assert torch.equal(ck.take(k, tuple(v.shape)), v) and ck.take(k).dtype == v.dtype
    ck.finish()
    ck = Checkpoint.open(str(tmp_path / "model.safetensors"))
    with pytest.raises(CheckpointError, match="not in the checkpoint"):
        ck.take("z")
    with pytest.raises(CheckpointError, match="expected"):
        ck.take("a", (3, 2))
    with pytest.raises(CheckpointError, match="does not use"):
        ck.finish()
    head = json.dumps({"a": {"dtype": "F32", "shape": [4], "data_offsets": [0, 8]}}).encode()
    (tmp_path / "bad").write_bytes(struct.pack("<Q", len(head)) + head + b"\0" * 8)
    with pytest.raises(CheckpointError, match="data_offsets"):
        Checkpoint.open(str(tmp_path / "bad"))


def test_registry_and_configuration_errors():
    assert model_class("Dagupel").__name__ == "DagupelStep"
    with pytest.raises(ValueError, match="unknown architecture"):
        model_class("nothing")
    with pytest.raises(ValueError):
        architecture_of({})
    cfg, _ = CONFIGS["odd"]
    c = DagupelConfig.parse(cfg)
    assert [c.weight_layer(i) for i in range(3)] == [0, 0, 2] and c.layers[2].mlp is None
    assert c.layers[0].mixer.rot_scaling == YarnScaling(4.0, 64, 8.0, 1.0) and c.layers[2].mixer.rot_scaling is None
    for change in (lambda d: d["layers"][0].update(type="other"), lambda d: d["layers"][0]["mlp"].update(kind="other"),
                   lambda d: d["layers"][1].update(weights_of=9), lambda d: d["layers"][0]["mixer"]["rot"].update(dims=4)):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError):
            DagupelConfig.parse(bad)
    circle = json.loads(json.dumps(cfg))
    circle["layers"][0]["weights_of"], circle["layers"][1]["weights_of"] = 1, 0
    with pytest.raises(ValueError, match="circle"):
        DagupelConfig.parse(circle).weight_layer(0)


def test_weights_load_shared_layers_once_and_differences_are_errors(tmp_path):
    cfg, _ = CONFIGS["tiny"]
    t = weights(cfg, 1)
    write_model(tmp_path, cfg, t)
    limits = ModelLimits(4, 16, torch.bfloat16, "cpu")
    m = load_model(str(tmp_path), limits)
    assert m.layers[0] is not m.layers[1] and m.layers[2] is m.layers[1] and m.layers[3] is m.layers[1]
    assert len({id(c.rows) for c in m.caches}) == 4        # a cache of its own for every layer
    with pytest.raises(CheckpointError, match="does not use"):
        type(m).from_checkpoint(cfg, Checkpoint(dict(t, extra=t["embed"])), limits)
    bad = json.loads(json.dumps(cfg))
    bad["layers"][2]["mixer"]["mask"]["size"] = 3
    with pytest.raises(ValueError, match="differs"):
        type(m).from_checkpoint(bad, Checkpoint(t), limits)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_padded_weights_compute_the_plain_products(name):
    """The merged, padded matrices of the layer against the checkpoint's, on the CPU in double."""
    from scalellm_amd.dagupel import DagupelStep
    cfg, _ = CONFIGS[name]
    t = weights(cfg, 2)
    m = DagupelStep.from_checkpoint(cfg, Checkpoint(t), ModelLimits(1, 16, torch.float32, "cpu"))
    rng = np.random.default_rng(0)
    for i, e in enumerate(cfg["layers"]):
        x, pre = e["mixer"], f"l{ref.weight_layer(cfg, i)}.mix."
        a, H, W = m.layers[i].attn, x["heads"], cfg["width"]
        w = {k[len(pre):]: v.double().numpy() for k, v in t.items() if k.startswith(pre)}
        h = np.zeros(a.w_in.size(1))
        h[:W] = rng.standard_normal(W)
        proj = a.w_in.double().numpy() @ h
        q = proj[:a.off_c].reshape(H, a.head_w)
        want = (w["q"] @ h[:W]).reshape(H, -1)
        np.testing.assert_allclose(q[:, :x["dim"]], want[:, :x["dim"]])
        np.testing.assert_allclose(q[:, a.q_dim:a.q_dim + x["rot_dim"]], want[:, x["dim"]:])
        down = w["dkv"] @ h[:W]
        np.testing.assert_allclose(proj[a.off_c:a.off_c + x["kv_rank"]], down[:x["kv_rank"]])
        np.testing.assert_allclose(proj[a.off_r:a.off_r + x["rot_dim"]], down[x["kv_rank"]:])
        np.testing.assert_allclose(proj[a.off_g:a.off_g + H], w["g"] @ h[:W])
        # absorbed: (W_uk^T q) . c == q . (W_uk c)
        c = np.zeros(a.c_pad)
        c[:x["kv_rank"]] = rng.standard_normal(x["kv_rank"])
        k = (w["uk"] @ c[:x["kv_rank"]]).reshape(H, -1)
        flat = np.zeros(H * a.head_w + 64)
        flat[:H * a.head_w] = q.reshape(-1)
        for head in range(H):
            lo = head * a.head_w
            qa = a.w_abs[head].double().numpy() @ flat[lo:lo + a.w_abs.size(2)]
            np.testing.assert_allclose(qa @ c, k[head] @ want[head, :x["dim"]], atol=1e-9)
        out = np.zeros(a.o_k)
        v = (a.w_uv.double().numpy() @ c)
        out[:H * a.v_pad] = v.reshape(-1)
        want_o = w["o"] @ (w["uv"] @ c[:x["kv_rank"]])
        np.testing.assert_allclose((a.w_o.double().numpy() @ out)[:W], want_o, atol=1e-9)


@pytest.mark.parametrize("rot", [
    {"base": 10000.0, "dims": 64}, {"base": 50.0, "dims": 2}, {"base": 500.0, "dims": 34, "scaling": dict(factor=4.0, original=128, fast=16.0, slow=2.0)},
    {"base": 1e6, "dims": 32, "scaling": dict(factor=1.0, original=64, fast=8.0, slow=1.0)},
    {"base": 30.0, "dims": 16, "scaling": dict(factor=8.0, original=2, fast=1.0, slow=1.0)},
    {"base": 10000.0, "dims": 64, "scaling": dict(factor=40.0, original=4096, fast=32.0, slow=1.0)}])
def test_rotary_table_with_and_without_yarn(rot):
    s = rot.get("scaling")
    table = rotary_table(rot["base"], rot["dims"], 700, YarnScaling(**s) if s else None)
    f, mag = ref.yarn_frequencies(rot)
    a = np.arange(700)[:, None] * f
    np.testing.assert_allclose(table.numpy(), np.concatenate([np.cos(a), np.sin(a)], 1) * mag, atol=2e-7 * mag)


# ---- blocks, steps, plans ----------------------------------------------------------------------
def test_allocator_gives_every_block_once_and_takes_it_back():
    a = BlockAllocator(5, 8)
    x = a.allocate(3)
    y = a.allocate(2)
    assert sorted(x + y) == list(range(5))
    with pytest.raises(OutOfBlocks):
        a.allocate(1)
    a.free(x)
    assert sorted(a.allocate(3)) == sorted(x)
    with pytest.raises(ValueError):
        BlockAllocator(4, 24)


def test_step_builder_orders_portions_behind_tokens():
    alloc = BlockAllocator(20, 4)
    b = StepBuilder(alloc, "cpu", portion_min=4)
    a, c, d = Sequence("a", list(range(10, 22))), Sequence("c", [1, 2, 3]), Sequence("d", list(range(9)))
    c.n_cached = 2
    c.reserve(alloc, 2)
    d.n_cached = 3
    d.reserve(alloc, 3)
    s = b.build([(a, 6), (c, 1), (d, 5)], {0: [5, 0], 1: [0]})
    assert s.order == [1, 0, 2] and s.row0 == [1, 0, 7]
    assert s.tokens.tolist() == [3] + list(range(10, 16)) + list(range(3, 8))
    assert s.positions.tolist() == [2] + list(range(6)) + list(range(3, 8))
    p = s.params
    assert p.q_cu_seq_lens.tolist() == [0, 1, 7, 12] and p.kv_cu_seq_lens.tolist() == [0, 3, 9, 17]
    assert p.logit_rows.tolist() == [6, 1, 0] and (p.q_max_seq_len, p.kv_max_seq_len) == (6, 8)
    slots = [q.blocks[i // 4] * 4 + i % 4 for q, lo, hi in ((c, 2, 3), (a, 0, 6), (d, 3, 8)) for i in range(lo, hi)]
    assert p.new_cache_slots.tolist() == slots
    assert p.cu_block_lens.tolist() == [0, 1, 3, 5]
    assert p.block_tables.tolist() == [4 * x for q in (c, a, d) for x in q.blocks]
    assert [(x.row0, x.q_len, x.kv_len) for x in p.portions] == [(1, 6, 6), (7, 5, 8)]
    assert StepBuilder(alloc, "cpu").build([(a, 6), (c, 1)]).params.portions == []
    with pytest.raises(ValueError):
        b.build([(c, 2)])


@pytest.mark.parametrize("window", [0, 1, 7, 16, 200])
def test_portion_plan_covers_what_the_rows_see(window):
    rng = np.random.default_rng(window)
    B, portions, row = 8, [], 3
    for start, n in ((0, 300), (45, 128), (130, 17), (7, 129)):
        blocks = rng.permutation(200)[:(start + n + B - 1) // B].astype(np.int32) * B
        portions.append(Portion(row, n, start + n, blocks))
        row += n
    slots, tiles = LatentPlan.host(portions, window, B)
    seen_rows = []
    for row0, rows, base, n_ctx, first, pos0 in tiles.tolist():
        p = next(p for p in portions if p.row0 <= row0 < p.row0 + p.q_len)
        assert pos0 == p.kv_len - p.q_len + row0 - p.row0 and 1 <= rows <= 128 and row0 + rows <= p.row0 + p.q_len
        seen_rows += range(row0, row0 + rows)
        assert first + n_ctx == p.kv_len and base + n_ctx <= len(slots)
        lo = max(0, pos0 - window + 1) if window else 0
        assert first <= lo
        for q in range(first, p.kv_len):
            assert slots[base + q - first] == p.blocks[q // B] + q % B
    assert sorted(seen_rows) == list(range(3, row))


# ---- scheduling and generation with a stand-in model --------------------------------------------
class Counter:
    """Next token = (sum of the sequence so far, read back through its 'cache') mod vocab."""
    vocab, max_positions, portion_min = 50, 64, 4

    def __init__(self, n_blocks, B):
        self.cache, self.B, self.rows = torch.zeros(n_blocks * B, dtype=torch.int64), B, []

    def forward(self, tokens, positions, params, return_logits=False):
        self.cache[params.new_cache_slots.long()] = tokens.long()
        cu, bcu = params.kv_cu_seq_lens.tolist(), params.cu_block_lens.tolist()
        self.rows.append(tokens.numel())
        out = torch.zeros(len(cu) - 1, self.vocab)
        for s in range(len(cu) - 1):
            slots = [int(params.block_tables[bcu[s] + i // self.B]) + i % self.B for i in range(cu[s + 1] - cu[s])]
            out[s, int(self.cache[slots].sum()) % self.vocab] = 1.0
        return out


def _count(prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(sum(t) % 50)
    return t[len(prompt):]


@pytest.mark.parametrize("n_blocks,budget,seqs", [(40, 100, 8), (40, 7, 3), (9, 16, 4), (6, 5, 2)])
def test_engine_generates_under_every_budget(n_blocks, budget, seqs):
    model = Counter(n_blocks, 4)
    e = LLMEngine(model, n_blocks, 4, "cpu", EngineOptions(max_seqs=seqs, max_step_tokens=budget))
    prompts = [[3, 1], [9] * 11, [7], [4, 4, 4, 4, 4], list(range(13))]
    out = e.generate(prompts, SamplingParams(max_tokens=8))
    assert out == [_count(p, 8) for p in prompts]
    assert max(model.rows) <= budget and e.allocator.n_free == n_blocks


def test_engine_stops_and_refuses():
    e = LLMEngine(Counter(40, 4), 40, 4, "cpu")
    want = _count([3, 1], 8)
    assert e.generate([[3, 1]], SamplingParams(max_tokens=8, stop_ids=[want[3]])) == [want[:4]]
    assert len(e.generate([[1] * 60], SamplingParams(max_tokens=30))[0]) == 4     # 64 positions
    for bad in ([], [50], [-1], [1] * 65):
        with pytest.raises(ValueError):
            e.add_request(bad, SamplingParams())
    small = LLMEngine(Counter(2, 4), 2, 4, "cpu")
    with pytest.raises(ValueError, match="pool"):
        small.add_request([1] * 6, SamplingParams(max_tokens=4))


def test_scheduler_puts_decoding_first_and_cuts_prompts():
    alloc = BlockAllocator(50, 4)
    s = Scheduler(alloc, 3, 10)
    a, b, c, d = (Sequence(k, [1] * n) for k, n in (("a", 4), ("b", 30), ("c", 5), ("d", 2)))
    for q in (a, b, c, d):
        s.add(q)
    assert [(q.id, n) for q, n in s.schedule()] == [("a", 4), ("b", 6)]
    a.n_cached, b.n_cached = 4, 6
    a.tokens.append(2)
    assert [(q.id, n) for q, n in s.schedule()] == [("a", 1), ("b", 9)]
    a.n_cached, b.n_cached = 5, 15
    s.finish(a)
    assert [(q.id, n) for q, n in s.schedule()] == [("b", 10)]
    b.n_cached = 25
    assert [(q.id, n) for q, n in s.schedule()] == [("b", 5), ("c", 5)]


# ---- sampling ----------------------------------------------------------------------------------
def test_sampling_parameters():
    x = torch.tensor([0.0, 3.0, 2.0, 2.5, -1.0])
    assert Sampler(SamplingParams(), "cpu").sample(x) == 1
    assert {Sampler(SamplingParams(temperature=1.0, top_k=1, seed=i), "cpu").sample(x) for i in range(9)} == {1}
    picks = [Sampler(SamplingParams(temperature=1.0, top_k=2, seed=i), "cpu").sample(x) for i in range(60)]
    assert set(picks) == {1, 3}
    picks = [Sampler(SamplingParams(temperature=1.0, top_p=0.4, seed=i), "cpu").sample(x) for i in range(30)]
    assert set(picks) == {1}
    s = Sampler(SamplingParams(temperature=1.0, seed=3), "cpu")
    freq = np.bincount([s.sample(x) for _ in range(3000)], minlength=5) / 3000
    np.testing.assert_allclose(freq, torch.softmax(x, 0).numpy(), atol=0.04)
    a, b = (Sampler(SamplingParams(temperature=0.7, seed=5), "cpu") for _ in range(2))
    assert [a.sample(x) for _ in range(20)] == [b.sample(x) for _ in range(20)]
    with pytest.raises(ValueError):
        SamplingParams(top_p=0.0)


def test_state_slots_are_owned_by_live_sequences():
    """One slot per sequence from its first step to its end; a step names them in batch order; admission waits for one."""
    alloc = BlockAllocator(40, 4, n_states=2)
    a, b, c = (Sequence(n, list(range(9))) for n in "abc")
    step = StepBuilder(alloc, "cpu", portion_min=2).build([(a, 5), (b, 1)])
    assert step.order == [1, 0] and step.params.state_slots.tolist() == [b.state, a.state] and {a.state, b.state} == {0, 1}
    with pytest.raises(OutOfBlocks):
        c.reserve(alloc, 1)
    assert not alloc.can_admit(1)
    held = a.state
    c.release(alloc)
    a.release(alloc)
    assert a.state is None and alloc.n_free_states == 1
    c.reserve(alloc, 1)
    assert c.state == held
    step = StepBuilder(alloc, "cpu", portion_min=2).build([(b, 2), (c, 3)], {0: [1], 1: [0, 2]})
    assert step.params.state_slots.tolist() == [b.state, c.state] and step.params.logit_rows.tolist() == [1, 2, 4]
    s = Scheduler(BlockAllocator(40, 4, n_states=2), 8, 64)
    for n in range(3):
        s.add(Sequence(n, [1, 2, 3]))
    assert [e[0].id for e in s.schedule()] == [0, 1]
    s.finish(s.running[0])
    assert [e[0].id for e in s.schedule()][-1] == 2
    assert StepBuilder(BlockAllocator(4, 4), "cpu").build([(Sequence("x", [1]), 1)]).params.state_slots is None


@pytest.mark.parametrize("start,q,size,keep", [(0, 300, 70, 5), (0, 300, 70, 100), (130, 140, 64, 3), (130, 140, 0, 0), (500, 1, 16, 0), (40, 2, 64, 30)])
def test_window_plan_covers_what_the_rows_see(start, q, size, keep):
    from oracle import vebusun as ref
    from scalellm_amd.layers import Portion
    from scalellm_amd.mixer_layers import WindowPlan
    B, rng = 16, np.random.default_rng(0)
    ps, row = [], 0
    for extra in (0, 7):
        n = start + q + extra
        ps.append(Portion(row, q + extra, n, rng.permutation(200)[:(n + B - 1) // B].astype(np.int32) * B))
        row += q + extra
    slots, tiles = WindowPlan.host(ps, size, keep, B)
    seen = set()
    for row0, rows, base, n, kept, first, pos0 in tiles.tolist():
        p = next(p for p in ps if p.row0 <= row0 < p.row0 + p.q_len)
        at = {(j if j < kept else j + first - kept): int(slots[base + j]) for j in range(n)}
        for r in range(rows):
            assert pos0 + r == p.kv_len - p.q_len + row0 - p.row0 + r
            seen.add(row0 + r)
            for j in ref.visible(pos0 + r, {"size": size, "keep_first": keep}):
                assert at[j] == int(p.blocks[j // B]) + j % B
    assert seen == set(range(row)) and max(t[1] for t in tiles.tolist()) <= 128


def test_vebusun_configuration():
    from scalellm_amd.vebusun import VebusunConfig
    from .vebusun_common import CONFIGS
    c = VebusunConfig.parse(CONFIGS["odd"])
    assert c.runs == [0, 1, 2, 1, 2, 1, 2] and c.layers[1].ff is None and c.layers[1].mixer.left.window == 21
    assert VebusunConfig.parse(CONFIGS["tiny"]).runs == [0, 1]
    bad = dict(CONFIGS["tiny"], loop={"start": 1, "stop": 5, "times": 2})
    with pytest.raises(ValueError):
        VebusunConfig.parse(bad)
    bad = dict(CONFIGS["tiny"], layers=[dict(CONFIGS["tiny"]["layers"][0], type="other")])
    with pytest.raises(ValueError):
        VebusunConfig.parse(bad)
