"""Mechanism ops against their equations in double precision: fp32-residual
norms, gated activations, interleaved rotation, the latent cache row and
attention over it.  Runs on the CPU ops and, marked gpu, on the HIP kernels."""
import pytest
import torch

import fetolix_oracle as oracle
from agentcontrolplane_amd import ops
from agentcontrolplane_amd.ops.reference import build_cos_sin
from op_helpers import BF16, F32, close, make_batch, rand

GPU = pytest.param("cuda", marks=pytest.mark.gpu)


@pytest.fixture(params=["cpu", GPU])
def device(request):
    if request.param == "cuda" and not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    return request.param


@pytest.fixture(params=[BF16, F32], ids=["bf16", "f32"])
def dtype(request):
    return request.param


# ------------------------------------------------------------------- norms


@pytest.mark.parametrize("n,w", [(1, 48), (5, 250), (3, 1027), (9, 4096)])
def test_layernorm(device, dtype, n, w):
    x = rand(n, w, dtype=F32, device=device) + 3.0
    wt = rand(w, dtype=dtype, device=device, seed=1)
    got = ops.layernorm(x, wt, 1e-3, dtype)
    assert got.dtype == dtype
    close(got, oracle.layer_norm(x.double().cpu(), wt.double().cpu(), 1e-3), dtype)


@pytest.mark.parametrize("n,w", [(1, 48), (7, 251), (4, 2048)])
@pytest.mark.parametrize("y_norm,x_norm", [(0, 0), (1, 0), (0, 1), (1, 1)])
def test_residual_norm(device, dtype, n, w, y_norm, x_norm):
    """x += y or rms(y) * wy; then layernorm(x) * wx, or x, into a strided view."""
    x = rand(n, w, dtype=F32, device=device)
    y = rand(n, w, dtype=dtype, device=device, seed=1, scale=0.01)
    wy = rand(w, dtype=dtype, device=device, seed=2) if y_norm else None
    wx = rand(w, dtype=dtype, device=device, seed=3) if x_norm else None
    eps = 1e-4  # the size of mean(y^2): eps inside the root shows
    xd, yd = x.double().cpu(), y.double().cpu()
    want = xd + (oracle.rms(yd, eps) * wy.double().cpu() if y_norm else yd)
    wide = torch.zeros(n, 2 * w, dtype=dtype, device=device)
    ops.residual_norm(x, y, eps, wy, wx, wide[:, w:])
    close(x, want, F32)
    out = oracle.layer_norm(want, wx.double().cpu(), eps) if x_norm else want
    close(wide[:, w:], out, dtype)
    assert not wide[:, :w].any()
    before = x.clone()
    ops.residual_norm(x, y, eps)  # no output: the residual only
    close(x, before.double().cpu() + yd, F32)


# ------------------------------------------------------- gated activations


def test_clamped_glu(device, dtype):
    """Values inside and outside the limits; gate is capped above only."""
    inter, limit = 24, 1.25
    wide = rand(33, 3 * inter, dtype=dtype, device=device, scale=2.0)
    out = torch.empty(33, 2 * inter, dtype=dtype, device=device)
    ops.clamped_glu(wide[:, inter:], limit, 1.702, 1.0, out[:, inter:])
    W = {"gate": torch.eye(2 * inter).double()[:inter],
         "up": torch.eye(2 * inter).double()[inter:], "down": torch.eye(inter).double()}
    want = oracle.clamped_glu(wide[:, inter:].double().cpu(), W, "", limit)
    close(out[:, inter:], want, dtype)
    ops.clamped_glu(wide[:, inter:], limit, 0.5, 0.0, out[:, inter:])  # other constants
    g = wide[:, inter : 2 * inter].double().cpu().clamp(max=limit)
    u = wide[:, 2 * inter :].double().cpu().clamp(-limit, limit)
    close(out[:, inter:], g * torch.sigmoid(0.5 * g) * u, dtype)


@pytest.mark.parametrize("n,w,dim", [(3, 40, 7), (19, 250, 5), (300, 64, 16), (2, 4096, 64)])
def test_side_gate(device, dtype, n, w, dim):
    """x + y, then the gated gelu of its projection; few and many tokens."""
    x, y = rand(n, w, dtype=F32, device=device), rand(n, w, dtype=dtype, device=device, seed=1)
    gate = rand(dim, w, dtype=dtype, device=device, seed=2, scale=w ** -0.5)
    table = rand(30, 3 * dim, dtype=dtype, device=device, seed=3)
    tok = torch.arange(n, device=device) * 3 % 30
    want_x = x.double().cpu() + y.double().cpu()
    x, got = ops.side_gate(x, y, gate, tok, table, dim)
    close(x, want_x, F32)
    want = oracle.gelu_tanh(want_x @ gate.double().cpu().T)
    close(got, want * table[tok][:, dim : 2 * dim].double().cpu(), dtype)


# -------------------------------------------------------------- per token


@pytest.mark.parametrize("kv_rank,rot_dim", [(24, 8), (100, 34), (512, 64)])
def test_latent_inputs(device, dtype, kv_rank, rot_dim):
    n, base, eps = 11, 3e4, 1e-2
    rank = ops.latent_rank(kv_rank)
    row = rank + 64
    wide = rand(n, kv_rank + rot_dim + 3, dtype=dtype, device=device, scale=0.1)
    kv = wide[:, 3:]
    w = rand(kv_rank, dtype=dtype, device=device, seed=1)
    pos = torch.tensor([0, 1, 2, 7, 300, 301, 999, 5, 64, 63, 65], device=device)
    slots = torch.randperm(32, generator=torch.Generator().manual_seed(1))[:n].to(device)
    cache = torch.full((8, 4, row), 7.0, dtype=dtype, device=device)
    cos_sin = build_cos_sin(1000, rot_dim, base, device, exact=True)
    args = (kv, w, eps, kv_rank, rot_dim, rank, pos, slots, cos_sin, cache)
    assert ops.latent_inputs(*args) is None
    # a low-rank query: 20 columns padded to 32, read out of a wider buffer
    buf = rand(n, 64, dtype=dtype, device=device, seed=2, scale=0.1)
    buf[:, 36:48] = 0
    qw = rand(32, dtype=dtype, device=device, seed=3)
    qw[20:] = 0
    cq = ops.latent_inputs(*args, buf[:, 16:48], qw, 20)
    close(cq[:, :20], oracle.rms(buf[:, 16:36].double().cpu(), eps) * qw[:20].double().cpu(), dtype)
    assert not cq[:, 20:].any()
    got = cache.view(32, row)[slots].cpu()
    kd = kv.double().cpu()
    close(got[:, :kv_rank], oracle.rms(kd[:, :kv_rank], eps) * w.double().cpu(), dtype)
    close(got[:, rank : rank + rot_dim],
          oracle.rotate_pairs(kd[:, kv_rank:], pos.cpu(), base), dtype)
    assert not got[:, kv_rank:rank].any() and not got[:, rank + rot_dim :].any()
    rest = torch.ones(32, dtype=torch.bool)
    rest[slots.cpu()] = False
    assert (cache.view(32, row).cpu()[rest] == 7.0).all()


@pytest.mark.parametrize("n", [1, 17, 70, 2100])
@pytest.mark.parametrize("O,K", [(32, 32), (96, 64), (512, 128), (128, 512)])
def test_head_linear(device, dtype, n, O, K):
    if n > 100 and (device == "cpu" or dtype == F32):
        n = 100
    H = 3
    x = rand(n, H, K + 32, dtype=dtype, device=device)[:, :, 32:]
    w = rand(H, O, K, dtype=dtype, device=device, seed=1, scale=K ** -0.5)
    gate = rand(n, H + 2, dtype=dtype, device=device, seed=2)[:, 1 : H + 1]
    out = torch.zeros(n, H, O + 32, dtype=dtype, device=device)
    want = torch.stack(
        [x[:, h].double().cpu() @ w[h].double().cpu().T for h in range(H)], 1
    )
    ops.head_linear(x, w, out[:, :, 32:])
    close(out[:, :, 32:], want, dtype)
    ops.head_linear(x, w, out[:, :, 32:], gate)
    close(out[:, :, 32:], want * torch.sigmoid(gate.double().cpu()).unsqueeze(-1), dtype)
    assert not out[:, :, :32].any()


# -------------------------------------------------------------- attention


def attend(q, rows, ctx, rank, scale, window):
    """q [L, H, row], rows [S, row] in double -> [L, H, rank]."""
    L, S = q.shape[0], rows.shape[0]
    ok = oracle.visible(S, window)[ctx : ctx + L]
    s = torch.einsum("lhd,sd->lhs", q, rows) * scale
    p = torch.softmax(s.masked_fill(~ok.unsqueeze(1), float("-inf")), -1)
    return torch.einsum("lhs,sr->lhr", p, rows[:, :rank])


ROT, BASE = 8, 2e3
SHAPES = [
    # heads, kv_rank, window, block, chunks
    (3, 24, None, 4, [(0, 5), (0, 1), (9, 2), (130, 1), (63, 1)]),
    (4, 64, 19, 16, [(0, 40), (200, 2), (17, 3), (18, 1), (19, 1), (500, 1), (1, 1)]),
    (16, 128, None, 16, [(0, 70), (300, 33), (64, 1), (1000, 1)]),
    (20, 200, 64, 16, [(0, 130), (63, 1), (64, 1), (65, 1), (700, 5)]),
    (33, 350, 100, 16, [(0, 9), (350, 1), (99, 1), (100, 1)]),
    (32, 512, None, 16, [(0, 150), (90, 1), (2000, 1), (777, 2)]),
    (128, 512, 300, 16, [(0, 3), (900, 1), (1200, 1)]),
    (2, 600, 50, 16, [(0, 60), (70, 1), (70, 2)]),
]


@pytest.mark.parametrize("H,kv_rank,window,block,chunks", SHAPES)
def test_latent_attention(device, dtype, H, kv_rank, window, block, chunks):
    rank = ops.latent_rank(kv_rank)
    row = rank + 64
    batch, chunks, tables, pages = make_batch(chunks, block, device)
    # pages outside a sequence hold NaN: reading one shows
    cache = torch.full((pages, block, row), float("nan"), dtype=dtype)
    kv = []
    for i, ((ctx, new), table) in enumerate(zip(chunks, tables)):
        r = rand(ctx + new, row, dtype=dtype, device="cpu", seed=10 + i)
        r[:, kv_rank:rank] = 0
        r[:, rank + ROT :] = 0
        kv.append(r.double())
        for p, page in enumerate(table):
            part = r[p * block : (p + 1) * block]
            cache[page, : len(part)] = part
    cache = cache.to(device)
    q = rand(batch.num_tokens, H, rank, dtype=dtype, device=device, seed=5)
    wide = rand(batch.num_tokens, H, 128, dtype=dtype, device=device, seed=6)
    wide[:, :, 64 + ROT :] = 0
    scale = 0.3 * kv_rank ** -0.5
    cos_sin = build_cos_sin(2100, ROT, BASE, device, exact=True)
    args = (cos_sin, ROT, cache, batch, scale, window)
    got = ops.latent_attention(q, wide[:, :, 64:], *args).cpu()
    part = batch.prefills[0].query_len  # rows from the second chunk on
    tail = ops.latent_attention(q[part:].clone(), wide[part:, :, 64:], *args, part, (0,)).cpu()
    rot = oracle.rotate_pairs(wide[:, :, 64 : 64 + ROT].double().cpu(), batch.positions.cpu(), BASE)
    full = torch.zeros(batch.num_tokens, H, row, dtype=torch.float64)
    full[:, :, :rank] = q.double().cpu()
    full[:, :, rank : rank + ROT] = rot.to(dtype)
    at = 0
    for (ctx, new), rows in zip(chunks, kv):
        want = attend(full[at : at + new], rows, ctx, rank, scale, window)
        close(got[at : at + new], want, dtype)
        if at:
            close(tail[at - part : at - part + new], want, dtype)
        at += new


@pytest.mark.parametrize("where", ["first", "far", "oldest_visible", "just_hidden", "self"])
@pytest.mark.parametrize("decode", [True, False])
def test_standout_key(device, dtype, where, decode):
    """One key scores far above the rest: attention must return its latent
    when it is visible, and never when it has just left the window."""
    H, rank, window, S, block = 4, 64, 40, 171, 16
    row = rank + 64
    i = S - 1
    hit = {"first": 0, "far": 77, "oldest_visible": i - window + 1,
           "just_hidden": i - window, "self": i}[where]
    win = None if where in ("first", "far") else window
    batch, chunks, tables, pages = make_batch([(i, 1)] if decode else [(i - 2, 3)], block, device)
    rows = rand(S, row, dtype=dtype, device="cpu", seed=3, scale=0.05)
    rows[:, rank:] = 0
    rows[hit, rank] = 8.0
    cache = torch.zeros(pages, block, row, dtype=dtype)
    for p, page in enumerate(tables[0]):
        cache[page, : len(rows[p * block : (p + 1) * block])] = rows[p * block : (p + 1) * block]
    q = torch.zeros(batch.num_tokens, H, rank, dtype=dtype)
    q_rot = torch.zeros(batch.num_tokens, H, 64, dtype=dtype)
    q_rot[:, :, 0] = 8.0
    still = torch.zeros(2, S, 1, device=device)
    still[0] = 1.0  # no rotation
    got = ops.latent_attention(
        q.to(device), q_rot.to(device), still, 2, cache.to(device), batch, 1.0, win
    )[-1]
    if where == "just_hidden":
        want = rows[i - window + 1 :, :rank].double().mean(0)
        assert (rows[hit, :rank].double() - want).abs().max() > 0.05
    else:
        want = rows[hit, :rank].double()
    close(got, want.expand(H, rank), dtype, scale=0.2)


EXPANDED = [
    # heads, dim, vdim, kv_rank, window, chunks
    (3, 64, 64, 64, None, [(0, 5), (0, 200), (100, 130)]),
    (8, 128, 128, 512, None, [(0, 300), (33, 1), (0, 129), (64, 65)]),
    (16, 128, 64, 128, 70, [(0, 333), (500, 40), (69, 2), (70, 2)]),
    (2, 256, 128, 256, 129, [(0, 257), (128, 128), (1000, 128)]),
    (5, 64, 256, 384, 64, [(0, 64), (64, 64), (63, 66)]),
    (1, 256, 256, 64, 1, [(0, 130), (77, 3)]),
]


@pytest.mark.gpu
@pytest.mark.parametrize("H,d,v,rank,window,chunks", EXPANDED)
@pytest.mark.parametrize("budget", [1 << 40, 1])
def test_expanded_prefill(H, d, v, rank, window, chunks, budget, monkeypatch):
    """Keys and values expanded from latents in one group or one per chunk;
    chunks left out and decode rows stay untouched."""
    from agentcontrolplane_amd.ops import hip

    monkeypatch.setattr(hip, "_EXPAND_BYTES", budget)
    device, dtype, row = "cuda", BF16, rank + 64
    batch, chunks, tables, pages = make_batch(chunks, 16, device)
    cache = torch.full((pages, 16, row), float("nan"), dtype=dtype)
    kv = []
    for i, ((ctx, new), table) in enumerate(zip(chunks, tables)):
        r = rand(ctx + new, row, dtype=dtype, device="cpu", seed=10 + i)
        r[:, rank + ROT :] = 0
        kv.append(r)
        for p, page in enumerate(table):
            part = r[p * 16 : (p + 1) * 16]
            cache[page, : len(part)] = part
    N = batch.num_tokens
    q = rand(N, H, d + 64, dtype=dtype, device=device, seed=5)
    q[:, :, d + ROT :] = 0
    w = rand(H * (d + v), rank, dtype=dtype, device=device, seed=6, scale=rank ** -0.5)
    gate = rand(N, H, dtype=dtype, device=device, seed=7)
    out = torch.full((N, H, v), 9.0, dtype=dtype, device=device)
    scale, skip = 0.5 * d ** -0.5, 1
    pick = tuple(i for i in range(len(batch.prefills)) if i != skip)
    ops.latent_expanded_prefill(
        q, w, gate, build_cos_sin(2100, ROT, BASE, device, exact=True), ROT,
        cache.to(device), batch, pick, rank, scale, window, out,
    )
    rot = oracle.rotate_pairs(q[:, :, d : d + ROT].double().cpu(), batch.positions.cpu(), BASE)
    wk = w[: H * d].double().cpu().view(H, d, rank)
    wv = w[H * d :].double().cpu().view(H, v, rank)
    at = 0
    for i, ((ctx, new), rows) in enumerate(zip(chunks, kv)):
        got = out[at : at + new].cpu()
        if i not in pick:
            assert (got == 9.0).all()
        else:
            c = rows[:, :rank].double()
            k = torch.einsum("sr,hdr->shd", c, wk).to(dtype).double()
            val = torch.einsum("sr,hvr->shv", c, wv).to(dtype).double()
            s = torch.einsum("lhd,shd->lhs", q[at : at + new, :, :d].double().cpu(), k)
            s += torch.einsum("lhd,sd->lhs", rot[at : at + new].to(dtype).double(),
                              rows[:, rank : rank + ROT].double())
            ok = oracle.visible(ctx + new, window)[ctx:]
            p = torch.softmax((s * scale).masked_fill(~ok.unsqueeze(1), float("-inf")), -1)
            want = torch.einsum("lhs,shv->lhv", p, val)
            want = want * torch.sigmoid(gate[at : at + new].double().cpu()).unsqueeze(-1)
            close(got, want, dtype)
        at += new
