"""The mechanisms of libslm_mixers one by one against the plain restatement (oracle/vebusun.py): recurrences, their norm and
gate, windowed attention in its three kernels; and the tanh norm, scaled adds and the SiLU GLU of the dense path."""
import numpy as np
import pytest
import torch

from .vebusun_common import lightning, mixer_weights, parallel, random_tensors, window
from oracle import vebusun as ref

pytestmark = pytest.mark.gpu
BOTH = [torch.float32, torch.bfloat16]
DEV = "cuda"


def _close(got, want, dtype, f32=2e-5, b16=4e-2):
    got = got.double().cpu().numpy() if isinstance(got, torch.Tensor) else got
    # (the largest difference over the root mean square: a value five times that, rounded to 16 bits, is off by 0.02 already)
    err = np.abs(got - want).max() / max(np.sqrt((want * want).mean()), 1e-30)
    assert err < (f32 if dtype == torch.float32 else b16), err


def _f64(w):
    return {k: v.double().numpy() for k, v in w.items()}


class _Batch:
    """Steps of one layer over sequences: entries [(sequence, rows)] -> positions and parameters."""

    def __init__(self, n_blocks=40, block_size=16, n_states=5):
        from scalellm_amd.engine import BlockAllocator, StepBuilder
        from scalellm_amd.registry import ModelLimits
        self.allocator = BlockAllocator(n_blocks, block_size, n_states)
        self.builder = StepBuilder(self.allocator, DEV, 2)
        self.limits = lambda dtype: ModelLimits(n_blocks, block_size, dtype, DEV, n_states)

    def run(self, mixer, cache, streams, entries):
        """streams: name -> hidden rows; entries: [(sequence, n)].  -> the mixer's output per entry."""
        step = self.builder.build(entries)
        h = torch.cat([streams[entries[i][0].id][entries[i][0].n_cached:entries[i][0].n_cached + entries[i][1]] for i in step.order])
        out = mixer(h, step.positions, cache, step.params)
        self.builder.commit(entries)
        return [out[step.row0[i]:step.row0[i] + n] for i, (_, n) in enumerate(entries)]


def _total(delta):
    return delta.t.sum(0) if hasattr(delta, "t") and not isinstance(delta, torch.Tensor) else delta.float()


def _hidden(n, width, dtype, seed):
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(n, width, generator=g).to(torch.bfloat16)
    pad = torch.zeros(n, (width + 63) // 64 * 64)
    pad[:, :width] = h.float()
    return h.double().numpy(), pad.to(device=DEV, dtype=dtype)


def _serve(layer, width, dtype, want_of, eps):
    """Streams of several lengths in uneven portions and single rows, slots used again; every row against want_of(h)."""
    from scalellm_amd.engine import Sequence
    b = _Batch()
    cache = layer.new_cache(b.limits(dtype))
    rng = np.random.default_rng(0)
    streams, want, got, live = {}, {}, {}, []
    for i, n in enumerate((70, 33, 150, 2, 1, 41)):
        h, streams[i] = _hidden(n, width, dtype, 20 + i)
        want[i], got[i] = want_of(h), []
    waiting = [Sequence(i, [0] * streams[i].size(0)) for i in streams]
    while live or waiting:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        entries = [(s, min(len(s.tokens) - s.n_cached, 1 if rng.random() < 0.4 else int(rng.integers(2, 50)))) for s in live]
        for (s, _), o in zip(entries, b.run(lambda *a: _total(layer.forward(*a)), cache, streams, entries)):
            got[s.id].append(o[:, :width])
        for s in [s for s in live if s.n_cached == len(s.tokens)]:
            live.remove(s)
            s.release(b.allocator)
    for i in want:
        _close(torch.cat(got[i]), want[i], dtype, 3e-5, 8e-2)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,taps,width", [(1, 1, 1, 1, 1, 16), (4, 2, 20, 13, 3, 77), (2, 2, 64, 64, 2, 64), (3, 1, 100, 65, 6, 50),
                                                               (2, 1, 192, 130, 4, 64), (2, 2, 256, 256, 4, 64), (70, 35, 32, 16, 4, 96)])
def test_channel_delta(heads, kv_heads, dim, vdim, taps, width, dtype):
    from scalellm_amd.mixer_layers import ChannelDelta, ChannelDeltaArgs
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}
    w = mixer_weights("channel_delta", m, width, random_tensors(1))
    layer = ChannelDelta(ChannelDeltaArgs(heads, kv_heads, dim, vdim, taps), width, 1e-5, w, dtype, DEV)
    _serve(layer, width, dtype, lambda h: ref.channel_delta(h, _f64(w), m, 1e-5), 1e-5)


class _Alone:
    """One half of a parallel mixer as a layer of its own."""

    def __init__(self, half, width, is_window):
        from scalellm_amd import latent_kernels as lk
        self.half, self.is_window, self.lk, self.width = half, is_window, lk, width

    def new_cache(self, limits):
        return self.half.new_cache(limits) if self.is_window else self.half.new_state(limits)

    def forward(self, h, positions, cache, params):
        proj = self.lk.linear(h, self.half.w_in)
        out = proj.new_full((h.size(0), self.half.out_width + 8), float("nan"))
        self.half.forward(proj, positions, cache, params, out[:, :self.half.out_width])
        return out[:, :self.half.out_width].float() @ self.half.w_o.float().t()


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("dim,vdim,decay", [(1, 1, (0.5,)), (11, 7, (0.3, 0.9, 0.99)), (64, 64, (1.0, 0.999)), (130, 200, (0.97, 0.0)),
                                            (256, 256, (0.9,)), (32, 48, tuple(0.5 + 0.007 * i for i in range(70)))])
def test_lightning_attention(dim, vdim, decay, dtype):
    from scalellm_amd.mixer_layers import LightningArgs, LightningAttention
    _, m = parallel(window(1, 1, 8, 8, 4, 5, 1), lightning(dim, vdim, decay))
    width = 80
    w = {k[6:]: v for k, v in mixer_weights("parallel", m, width, random_tensors(2)).items() if k.startswith("right.")}
    half = LightningAttention(LightningArgs(len(decay), dim, vdim, decay), width, 1e-5, w, dtype, DEV, 0.75)
    _serve(_Alone(half, width, False), width, dtype, lambda h: 0.75 * ref.lightning_attention(h, _f64(w), m["right"], 1e-5), 1e-5)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("m", [window(1, 1, 2, 1, 2, 1, 0), window(6, 3, 22, 18, 10, 21, 5, 5.0), window(4, 4, 64, 96, 64, 16, 16),
                               window(34, 2, 128, 64, 0, 40, 70, 8.0), window(3, 1, 96, 192, 50, 0, 0, 0.0), window(2, 2, 256, 256, 128, 33, 3),
                               window(2, 1, 200, 128, 200, 64, 1, 3.0), window(2, 1, 300, 260, 40, 30, 4)])
def test_window_attention(m, dtype):
    from scalellm_amd.latent_layers import rotary_table
    from scalellm_amd.mixer_layers import WindowAttention, WindowAttentionArgs
    width = 72
    _, both = parallel(m, lightning(4, 4, (0.5,)))
    w = {k[5:]: v for k, v in mixer_weights("parallel", both, width, random_tensors(3), sharp=1.5).items() if k.startswith("left.")}
    rot = m["rot"]
    args = WindowAttentionArgs(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], rot["base"], rot["dims"], m["softcap"],
                               m["mask"]["size"], m["mask"]["keep_first"])
    half = WindowAttention(args, width, 1e-5, w, rotary_table(rot["base"], rot["dims"], 256, device=DEV), dtype, DEV, 1.25)
    _serve(_Alone(half, width, True), width, dtype, lambda h: 1.25 * ref.sink_attention(h, _f64(w), m, 1e-5), 1e-5)


@pytest.mark.parametrize("softcap,sink", [(0.0, False), (6.0, True), (0.0, True)])
@pytest.mark.parametrize("size,keep", [(0, 0), (200, 0), (100, 40), (3, 2)])
@pytest.mark.parametrize("heads,kv_heads,D,V", [(8, 2, 128, 128), (40, 2, 64, 96)])
def test_attention_kernels_agree(heads, kv_heads, D, V, size, keep, softcap, sink):
    """Single rows by the any-size kernel, by MFMA with one and with many splits, and as portions, against the sums written
    out; unequal contexts, blocks in random order, one key per head that stands out just inside or outside the window."""
    from scalellm_amd import mixer_kernels as mk
    from scalellm_amd.layers import InputParameters, Portion
    from scalellm_amd.mixer_layers import WindowPlan
    g = torch.Generator().manual_seed(4)
    B, lens = 16, [1, 17, 700, 64, 333]
    nb = [(n + B - 1) // B for n in lens]
    perm = torch.randperm(sum(nb), generator=g).to(torch.int32) * B
    cu = np.concatenate([[0], np.cumsum(nb)])
    r = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16)  # noqa: E731
    kc, vc = r(sum(nb) * B, kv_heads, D), r(sum(nb) * B, kv_heads, V)
    q = r(len(lens), heads * D)
    slot = lambda s, j: int(perm[cu[s] + j // B]) + j % B  # noqa: E731
    for s, n in enumerate(lens):      # loud keys around the window's edge and the kept tokens' end
        for j in {n - size, n - size - 1, keep - 1, keep}:
            if 0 <= j < n:
                for a in range(kv_heads):
                    kc[slot(s, j), a] = q[s].view(heads, D)[a * (heads // kv_heads)] * 0.8
    sk = torch.randn(heads, generator=g) + 2 if sink else None
    scale, f = D ** -0.5, 0.5
    want = np.zeros((len(lens), heads, V))
    for s, n in enumerate(lens):
        js = ref.visible(n - 1, {"size": size, "keep_first": keep})
        at = [slot(s, j) for j in js]
        for h in range(heads):
            x = kc[at, h // (heads // kv_heads)].double().numpy() @ q[s].view(heads, D)[h].double().numpy() * scale
            x = softcap * np.tanh(x / softcap) if softcap else x
            p = np.exp(x - x.max())
            extra = np.exp(float(sk[h]) - x.max()) if sink else 0.0
            want[s, h] = f * (p @ vc[at, h // (heads // kv_heads)].double().numpy()) / (p.sum() + extra)
    dev = lambda t: t.to(DEV)  # noqa: E731
    i32 = lambda x: torch.tensor(np.asarray(x), dtype=torch.int32, device=DEV)  # noqa: E731
    q, kc, vc, table, sk = dev(q), dev(kc), dev(vc), dev(perm), None if sk is None else dev(sk)
    how = dict(heads=heads, window=size, keep_first=keep, scale=scale, softcap=softcap, out_scale=f)
    for kw in (dict(generic=True), dict(n_splits=1), dict(n_splits=3), dict(n_splits=7), dict()):
        out = torch.full((len(lens), heads * V), float("nan"), dtype=torch.bfloat16, device=DEV)
        mk.window_attention(q, kc, vc, out, sk, i32(lens) - 1, i32(range(len(lens) + 1)), table, i32(cu), block_size=B, max_kv_len=max(lens),
                            **how, **kw)
        _close(out.view(len(lens), heads, V), want, torch.bfloat16, b16=4e-2)
    ps = [Portion(s, 1, n, perm[cu[s]:cu[s + 1]].numpy()) for s, n in enumerate(lens)]
    prm = InputParameters(*[None] * 5, portions=ps)
    plan = WindowPlan.of(prm, size, keep, B, DEV)
    out = torch.full((len(lens), heads * V), float("nan"), dtype=torch.bfloat16, device=DEV)
    mk.window_prefill(q, kc, vc, out, sk, plan.slots, plan.tiles, **how)
    _close(out.view(len(lens), heads, V), want, torch.bfloat16, b16=4e-2)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("per_head", [True, False])
@pytest.mark.parametrize("heads,vdim", [(1, 1), (3, 13), (16, 128), (5, 200)])
def test_gated_norm(heads, vdim, per_head, dtype):
    from scalellm_amd import mixer_kernels as mk
    g = torch.Generator().manual_seed(5)
    rows, v_pad, n = 9, (vdim + 15) // 16 * 16, heads * vdim
    o = torch.randn(rows, heads, v_pad, generator=g) * 3
    gate = torch.randn(rows, n + 8, generator=g).to(dtype)
    w = torch.randn(vdim if per_head else n, generator=g)
    out = torch.full((rows, n + 24), float("nan"), dtype=dtype, device=DEV)
    mk.gated_norm(o.to(DEV), vdim, gate.to(DEV), w.to(DEV), out, eps=1e-3, per_head=per_head, scale=0.3)
    x = o[:, :, :vdim].double().numpy()
    x = x if per_head else x.reshape(rows, n)
    want = 0.3 * ref.rms_norm(x, w.double().numpy(), 1e-3).reshape(rows, n) * ref.sigmoid(gate[:, :n].double().numpy())
    _close(out[:, :n], want, dtype)
    assert float(out[:, n:].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width,rows", [(33, 5), (256, 3), (2048, 40)])
def test_tanh_norm_and_scaled_adds(width, rows, dtype):
    from scalellm_amd import latent_kernels as lk
    g = torch.Generator().manual_seed(6)
    r = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    w, b, alpha, mult, ld = r(width), r(width), 0.7, 0.3, (width + 63) // 64 * 64
    norm = lk.TanhNorm(alpha, w.to(DEV), b.to(DEV))
    plain = lambda x: ref.dynamic_tanh(x, alpha, w.double().numpy(), b.double().numpy())  # noqa: E731

    def check(x, resid, out):
        _close(resid, x, torch.float32, 1e-6)
        _close(out[:, :width], plain(x), dtype, 1e-5, 3e-2)
        assert ld == width or float(out[:, width:].abs().max()) == 0.0
    table, tokens = r(20, width).to(dtype), torch.arange(rows, dtype=torch.int32) % 20
    resid = torch.empty(rows, width, device=DEV)
    out = torch.empty(rows, ld, dtype=dtype, device=DEV)
    lk.residual_norm(resid, out, norm, 0.0, embed=(tokens.to(DEV), table.to(DEV), None, None), mult=4.5)
    x = table.double().numpy()[tokens.numpy()] * 4.5
    check(x, resid, out)
    delta = r(rows, ld).to(dtype)
    lk.residual_norm(resid, out, norm, 0.0, delta=delta.to(DEV), mult=mult)
    x = x + mult * delta[:, :width].double().numpy()
    check(x, resid, out)
    slabs = r(11, rows, ld)
    lk.residual_norm(resid, out, norm, 0.0, delta=lk.Slabs(slabs.to(DEV)), mult=mult)
    x = x + mult * slabs.double().sum(0)[:, :width].numpy()
    check(x, resid, out)
    pick = torch.tensor([rows - 1, 0], dtype=torch.int32, device=DEV)
    out = torch.empty(2, ld, dtype=dtype, device=DEV)
    lk.residual_norm(resid, out, norm, 0.0, row_index=pick)
    _close(out[:, :width], plain(x[[rows - 1, 0]]), dtype, 1e-5, 3e-2)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("rows", [1, 20, 70])
def test_silu_glu(rows, dtype):
    from scalellm_amd.latent_layers import ClampedGLU
    rnd, W, ff = random_tensors(7), 60, 90
    w = {"gate": rnd(ff, W, std=0.5), "up": rnd(ff, W, std=0.5), "down": rnd(W, ff, std=0.1)}
    h, x = _hidden(rows, W, dtype, 8)
    layer = ClampedGLU(W, ff, float("inf"), w, dtype, DEV, 1.0, 0.0)
    _close(_total(layer.forward(x))[:, :W], ref.feed_forward(h, _f64(w)), dtype, 1e-5, 3e-2)
