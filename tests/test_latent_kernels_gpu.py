"""The mechanisms of the dense / latent-attention library one by one against plain double-precision arithmetic."""
import numpy as np
import pytest
import torch

from oracle import dagupel as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def _lk():
    from scalellm_amd import latent_kernels
    return latent_kernels


def _rnd(seed, *shape, dtype=torch.float32, std=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * std).to(dtype).to(DEV)


def _f64(t):
    return t.detach().double().cpu().numpy()


def _close(got, want, dtype, f32=3e-6, b16=1e-2):
    got, want = _f64(got), np.asarray(want, dtype=np.float64)
    assert got.shape == want.shape and np.isfinite(got).all()
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-30)
    assert err < (f32 if dtype == torch.float32 else b16), err


# ---- residual stream and norm ------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 64), (5, 77), (3, 4096), (130, 100), (2, 7168)])
def test_residual_norm_modes(rows, width, dtype):
    lk, eps = _lk(), 1e-5
    pad = (width + 63) // 64 * 64
    w = _rnd(1, width)
    table, pos = _rnd(2, 32, pad, dtype=dtype), _rnd(3, 50, width, dtype=dtype)
    tokens = torch.randint(0, 32, (rows,), dtype=torch.int32, device=DEV)
    positions = torch.randint(0, 50, (rows,), dtype=torch.int32, device=DEV)
    resid = torch.full((rows, width), float("nan"), device=DEV)
    out = torch.full((rows, pad), 7.0, dtype=dtype, device=DEV)

    def check(x):
        np.testing.assert_allclose(_f64(resid), x, rtol=1e-6, atol=1e-6 * np.abs(x).max())
        _close(out[:, :width], ref.rms_norm(x, _f64(w), eps), dtype)
        assert not out[:, width:].any()
    x = _f64(table)[_f64(tokens).astype(int), :width]
    lk.residual_norm(resid, out, w, eps, embed=(tokens, table, None, None))
    check(x)
    x = x + _f64(pos)[_f64(positions).astype(int)]
    lk.residual_norm(resid, out, w, eps, embed=(tokens, table, positions, pos))
    check(x)
    delta = _rnd(4, rows, pad, dtype=dtype)
    lk.residual_norm(resid, out, w, eps, delta=delta)
    x = x + _f64(delta)[:, :width]
    check(x)
    slabs = _rnd(5, 3, rows, pad)
    lk.residual_norm(resid, out, w, eps, delta=lk.Slabs(slabs))
    x = x + _f64(slabs).sum(0)[:, :width]
    check(x)
    lk.residual_norm(resid, out, None, eps, delta=delta)      # the sum only
    x = x + _f64(delta)[:, :width]
    np.testing.assert_allclose(_f64(resid), x, rtol=1e-6, atol=2e-6 * np.abs(x).max())
    pick = torch.tensor([rows - 1, 0, rows // 2], dtype=torch.int32, device=DEV)
    out = torch.full((3, pad), 7.0, dtype=dtype, device=DEV)
    lk.residual_norm(resid, out, w, eps, row_index=pick)
    _close(out[:, :width], ref.rms_norm(x[[rows - 1, 0, rows // 2]], _f64(w), eps), dtype)


def test_eps_is_inside_the_root():
    lk = _lk()
    x = torch.full((1, 64), 1e-3, device=DEV)
    out = torch.empty(1, 64, device=DEV)
    lk.residual_norm(x, out, torch.ones(64, device=DEV), 1e-2)
    np.testing.assert_allclose(_f64(out), 1e-3 / np.sqrt(1e-6 + 1e-2), rtol=1e-6)


# ---- products ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(1, 16, 64), (3, 48, 320), (16, 80, 1024), (17, 112, 192), (33, 96, 2048), (64, 272, 128),
                                   (65, 64, 64), (200, 144, 256), (1, 4096, 4096),
                                   (30, 16416, 128), (20, 4096, 8192), (50, 16416, 64)])
def test_linear_epilogues(M, N, K, dtype):
    lk = _lk()
    x, w = _rnd(1, M, K, dtype=dtype), _rnd(2, N, K, dtype=dtype, std=K ** -0.5)
    want = _f64(x) @ _f64(w).T
    _close(lk.linear(x, w), want, dtype, f32=1e-5)
    _close(lk.linear_f32(x, w, 0.25), 0.25 * want, torch.float32, f32=1e-5)
    s = lk.linear_slabs(x, w)
    _close(s.t.sum(0), want, torch.float32, f32=1e-5)
    if N % 32 == 0:
        out = torch.empty(M, N // 2, dtype=dtype, device=DEV)
        lk.linear_glu(x, w, out, 0.6)
        _close(out, ref.clamped_glu(want[:, :N // 2], want[:, N // 2:], 0.6), dtype, f32=1e-5, b16=2e-2)


def test_split_k_slabs_cover_k_once():
    lk = _lk()
    x, w = _rnd(1, 4, 8192, dtype=torch.bfloat16), _rnd(2, 64, 8192, dtype=torch.bfloat16, std=0.01)
    s = lk.linear_slabs(x, w)
    assert s.t.size(0) > 1
    _close(s.t.sum(0), _f64(x) @ _f64(w).T, torch.float32, f32=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 20, 70])
def test_per_head_products_with_gate(rows, dtype):
    lk, H, K, N, head = _lk(), 3, 64, 32, 96
    x, w = _rnd(1, rows, H * head + 64, dtype=dtype), _rnd(2, H, N, K, dtype=dtype, std=0.1)
    gate = _rnd(3, rows, 16, dtype=dtype)
    out = torch.zeros(rows, H * 40, dtype=dtype, device=DEV)
    for g in (None, gate):
        lk.linear_heads(x, head, w, out, 40, gate=g)
        for h in range(H):
            want = _f64(x)[:, h * head:h * head + K] @ _f64(w)[h].T
            if g is not None:
                want = want * ref.sigmoid(_f64(gate)[:, h:h + 1])
            _close(out[:, h * 40:h * 40 + N], want, dtype)
        assert not out.view(rows, H, 40)[:, :, N:].any()


@pytest.mark.parametrize("dtype", DTYPES)
def test_clamped_glu_bends_where_it_should(dtype):
    lk, limit = _lk(), 1.25
    v = torch.tensor([-9.0, -1.5, -1.25, -1.0, -0.25, 0.0, 0.5, 1.25, 1.5, 9.0])
    g, u = torch.meshgrid(v, v, indexing="ij")
    g, u = torch.nn.functional.pad(g.reshape(4, 25), (0, 3)), torch.nn.functional.pad(u.reshape(4, 25), (0, 3))
    gu = torch.cat([g, u], dim=1).to(dtype).to(DEV)
    out = torch.empty(4, 28, dtype=dtype, device=DEV)
    lk.clamped_glu(gu, out, limit)
    _close(out, ref.clamped_glu(g.double().numpy(), u.double().numpy(), limit), dtype)


# ---- rotation, latent norm, cache --------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,q_dim,rot,rank", [(1, 32, 2, 5), (3, 64, 32, 80), (20, 96, 34, 100), (2, 32, 64, 500)])
def test_append_norms_rotates_and_writes_its_slots(heads, q_dim, rot, rank, dtype):
    from scalellm_amd.latent_layers import YarnScaling, round_up, rotary_table
    lk, eps, rows = _lk(), 1e-4, 7
    c_pad, r_pad = round_up(rank, 64), round_up(rot, 32)
    rcfg = {"base": 900.0, "dims": rot, "scaling": {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    cs = rotary_table(900.0, rot, 300, YarnScaling(3.0, 64, 8.0, 1.0), DEV)
    hd = q_dim + r_pad
    off_c = heads * hd
    off_r = off_c + c_pad
    proj = torch.zeros(rows, off_r + r_pad + 16, dtype=dtype, device=DEV)
    proj[:, :off_c].view(rows, heads, hd)[:, :, :q_dim + rot] = _rnd(1, rows, heads, q_dim + rot, dtype=dtype)
    proj[:, off_c:off_c + rank] = _rnd(2, rows, rank, dtype=dtype)
    proj[:, off_r:off_r + rot] = _rnd(3, rows, rot, dtype=dtype)
    before, w = _f64(proj), _rnd(4, rank)
    pos = torch.tensor([0, 1, 2, 50, 299, 64, 7], dtype=torch.int32, device=DEV)
    slots = torch.tensor([9, 3, 0, 31, 17, 4, 22], dtype=torch.int32, device=DEV)
    cache = torch.full((32, c_pad + r_pad), 5.0, dtype=dtype, device=DEV)
    q_abs = torch.full((4, heads, c_pad + r_pad), 5.0, dtype=dtype, device=DEV)
    lk.latent_append(proj, cache, q_abs, w, cs, pos, slots, heads=heads, q_dim=q_dim, q_rot=r_pad, rank=rank, c_pad=c_pad,
                     off_c=off_c, off_r=off_r, eps=eps)
    P = pos.tolist()
    rows_ = cache[slots.long()]
    _close(rows_[:, :rank], ref.rms_norm(before[:, off_c:off_c + rank], _f64(w), eps), dtype)
    _close(rows_[:, c_pad:c_pad + rot], ref.rotate(before[:, off_r:off_r + rot], P, rcfg), dtype)
    assert not rows_[:, rank:c_pad].any() and not rows_[:, c_pad + rot:].any()
    other = [i for i in range(32) if i not in slots.tolist()]
    assert (cache[other] == 5.0).all()
    q0 = before[:, :off_c].reshape(rows, heads, hd)
    q1 = proj[:, :off_c].view(rows, heads, hd)
    want = ref.rotate(q0[:, :, q_dim:q_dim + rot], P, rcfg)
    _close(q1[:, :, q_dim:q_dim + rot], want, dtype)
    assert np.array_equal(_f64(q1)[:, :, :q_dim], q0[:, :, :q_dim])
    _close(q_abs[:, :, c_pad:c_pad + rot], want[:4], dtype)
    assert not q_abs[:, :, c_pad + rot:].any() and (q_abs[:, :, :c_pad] == 5.0).all()


# ---- attention over the cache ------------------------------------------------------------------
class Paged:
    """Sequences of the given lengths on shuffled blocks, cache rows random (or given)."""

    def __init__(self, lens, block, c_pad, r_pad, dtype, seed=0):
        rng = np.random.default_rng(seed)
        self.lens, self.block = lens, block
        n = [(x + block - 1) // block for x in lens]
        ids = rng.permutation(sum(n) + 3)[:sum(n)]
        self.cu = np.concatenate([[0], np.cumsum(n)])
        self.table = (ids * block).astype(np.int32)
        self.cache = _rnd(seed, (sum(n) + 3) * block, c_pad + r_pad, dtype=dtype)

    def slot(self, s, p):
        return int(self.table[self.cu[s] + p // self.block]) + p % self.block

    def rows(self, s):
        return self.cache[[self.slot(s, p) for p in range(self.lens[s])]]

    def dev(self, a):
        return torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)


def _attn_ref(q, rows, p, window, scale, c_pad):
    lo = max(0, p - window + 1) if window > 0 else 0
    k = _f64(rows[lo:p + 1])
    out = []
    for h in range(q.shape[0]):
        s = k @ q[h] * scale
        e = np.exp(s - s.max())
        out.append(e / e.sum() @ k[:, :c_pad])
    return np.array(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("c_pad,r_pad", [(64, 32), (128, 64), (256, 32), (512, 64), (512, 32), (192, 96)])
@pytest.mark.parametrize("heads", [1, 16, 19, 40])
def test_latent_attention_sizes(c_pad, r_pad, heads, dtype):
    """Sequences of unequal lengths, rows anywhere in them, window borders, one and several splits."""
    lk = _lk()
    lens = [1, 31, 64, 65, 200, 333]
    pg = Paged(lens, 16, c_pad, r_pad, dtype, seed=heads)
    rows = [(0, 0), (1, 30), (2, 63), (3, 64), (3, 63), (4, 150), (5, 332), (5, 331), (5, 0)]
    pos = pg.dev([p for _, p in rows])
    q_cu = pg.dev(np.concatenate([[0], np.cumsum([sum(1 for s, _ in rows if s == k) for k in range(len(lens))])]))
    q = _rnd(7, len(rows), heads, c_pad + r_pad, dtype=dtype)
    scale = 2.0 * (c_pad + r_pad) ** -0.5
    for window in (0, 1, 33, 64, 200):
        want = np.stack([_attn_ref(_f64(q[i]), pg.rows(s), p, window, scale, c_pad) for i, (s, p) in enumerate(rows)])
        for kw in (dict(), dict(n_splits=1), dict(n_splits=5), dict(generic=True)):
            out = torch.full((len(rows), heads, c_pad), float("nan"), dtype=dtype, device=DEV)
            lk.latent_attention(q, pg.cache, out, pos, q_cu, pg.dev(pg.table), pg.dev(pg.cu), block_size=16, window=window,
                                scale=scale, max_kv_len=333, **kw)
            _close(out, want, dtype, f32=1e-5, b16=1.5e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_attention_sees_exactly_its_window(dtype):
    """One key that outweighs all others: present at distance window - 1, gone at distance window."""
    lk, c_pad, r_pad, H = _lk(), 64, 32, 2
    for block in (8, 64):
        for window in (1, 2, 16, 31, 64, 65, 128, 250):
            pg = Paged([400], block, c_pad, r_pad, dtype, seed=window)
            place = 97
            big = pg.slot(0, place)
            pg.cache[:, 64] = 0
            pg.cache[big, 64], pg.cache[big, :8] = 30.0, 9.0
            at = [p for p in (place, place + 1, place + window - 1, place + window, place + window + 1) if place <= p < 400]
            q = torch.zeros(len(at), H, c_pad + r_pad, dtype=dtype, device=DEV)
            q[:, :, 64] = 1.0
            for splits in (1, 4):
                out = torch.empty(len(at), H, c_pad, dtype=dtype, device=DEV)
                lk.latent_attention(q, pg.cache, out, pg.dev(at), pg.dev([0, len(at)]), pg.dev(pg.table), pg.dev(pg.cu), block_size=block,
                                    window=window, scale=1.0, max_kv_len=400, n_splits=splits)
                for i, p in enumerate(at):
                    seen = p - place < window
                    assert (float(out[i].float()[:, :8].min()) > 8.5) == seen, (block, window, p)


@pytest.mark.parametrize("block,lens", [(1, [2500, 1023, 1024, 1025]), (2, [5000, 2049])])
def test_latent_attention_of_more_blocks_than_are_staged_at_once(block, lens):
    lk, c_pad, r_pad, H, dt = _lk(), 64, 32, 3, torch.bfloat16
    pg = Paged(lens, block, c_pad, r_pad, dt)
    q = _rnd(1, len(lens), H, c_pad + r_pad, dtype=dt)
    pos = pg.dev([n - 1 for n in lens])
    for window in (0, 1500):
        want = np.stack([_attn_ref(_f64(q[i]), pg.rows(i), n - 1, window, 0.2, c_pad) for i, n in enumerate(lens)])
        for splits in (1, 2):
            out = torch.empty(len(lens), H, c_pad, dtype=dt, device=DEV)
            lk.latent_attention(q, pg.cache, out, pos, pg.dev(range(len(lens) + 1)), pg.dev(pg.table), pg.dev(pg.cu), block_size=block,
                                window=window, scale=0.2, max_kv_len=max(lens), n_splits=splits)
            _close(out, want, dt, b16=1.5e-2)


# ---- prompt portions ---------------------------------------------------------------------------
@pytest.mark.parametrize("q_dim,r_pad,v_pad", [(32, 32, 32), (32, 64, 64), (64, 64, 128), (128, 32, 64), (128, 64, 128), (192, 64, 64)])
@pytest.mark.parametrize("window", [0, 1, 40, 64, 129, 300])
def test_portion_attention(q_dim, r_pad, v_pad, window):
    """Portions at several offsets of unequal sequences, with the context gathered and cut to the window by the plan."""
    from scalellm_amd.latent_layers import LatentPlan
    from scalellm_amd.layers import Portion
    lk, H, c_pad, block = _lk(), 3, 64, 16
    dt = torch.bfloat16
    spans = [(0, 140), (77, 78 + 128), (200, 217), (129, 430)]    # [start, end) of every sequence's portion
    pg = Paged([e for _, e in spans], block, c_pad, r_pad, dt)
    row0 = np.concatenate([[0], np.cumsum([e - s for s, e in spans])])
    T = int(row0[-1]) + 5
    ld = H * (q_dim + r_pad) + 16
    proj = _rnd(1, T, ld, dtype=dt)
    w = _rnd(2, H * (q_dim + v_pad), c_pad, dtype=dt, std=c_pad ** -0.5)
    portions = [Portion(int(row0[i]) + 5, e - s, e, pg.table[pg.cu[i]:pg.cu[i + 1]]) for i, (s, e) in enumerate(spans)]
    plan = LatentPlan.build(portions, window, block, DEV)
    ctx = lk.latent_gather(pg.cache, plan.slots)
    kv = torch.mm(ctx[:, :c_pad], w.t())
    out = torch.full((T, H * v_pad), float("nan"), dtype=dt, device=DEV)
    scale = 1.5 * (q_dim + r_pad) ** -0.5
    lk.latent_prefill(proj, ctx, kv, out, plan.tiles, heads=H, q_dim=q_dim, c_pad=c_pad, v_pad=v_pad,
                      gate_off=H * (q_dim + r_pad), window=window, scale=scale)
    assert torch.isnan(out[:5].float()).all()     # rows in front of the portions are not touched
    kv64 = {}
    for i, (s, e) in enumerate(spans):
        rows = pg.rows(i)
        x = _f64(torch.mm(rows[:, :c_pad], w.t())).reshape(e, H, q_dim + v_pad)
        kv64[i] = x, _f64(rows[:, c_pad:])
    want = np.zeros((T - 5, H * v_pad))
    for i, (s, e) in enumerate(spans):
        x, kr = kv64[i]
        for p in range(s, e):
            r = int(row0[i]) + p - s
            pr = _f64(proj[r + 5])
            lo = max(0, p - window + 1) if window else 0
            for h in range(H):
                q = pr[h * (q_dim + r_pad):(h + 1) * (q_dim + r_pad)]
                sc = (x[lo:p + 1, h, :q_dim] @ q[:q_dim] + kr[lo:p + 1] @ q[q_dim:]) * scale
                ex = np.exp(sc - sc.max())
                want[r, h * v_pad:(h + 1) * v_pad] = ex / ex.sum() @ x[lo:p + 1, h, q_dim:] * ref.sigmoid(pr[H * (q_dim + r_pad) + h])
    _close(out[5:], want, dt, b16=1.5e-2)
