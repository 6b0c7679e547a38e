"""Noganex's mechanisms against their equations in double precision: norms over all heads
ahead of the rotation, chunks, scores mixed over the heads, the delta rule with one decay
per head and a silu gate, sigmoid routing with a correction, and the residual update that
gates and norms a sublayer's result.  Runs on the CPU ops and, marked gpu, on the HIP
kernels."""
import math

import pytest
import torch

import noganex_oracle as oracle
from agentcontrolplane_amd import ops
from agentcontrolplane_amd.engine.config import YarnScaling, gelu_glu, silu_glu
from agentcontrolplane_amd.models.layout import pair_halves, pad_to
from agentcontrolplane_amd.models.rotary import frequencies, rotation_table
from op_helpers import BF16, F32, close, make_batch, rand
from test_tezinex_ops import DeltaCase, paged

GPU = pytest.param("cuda", marks=pytest.mark.gpu)


@pytest.fixture(params=["cpu", GPU])
def device(request):
    if request.param == "cuda" and not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    return request.param


@pytest.fixture(params=[BF16, F32], ids=["bf16", "f32"])
def dtype(request):
    return request.param


# ---------------------------------------------------------- attention inputs


@pytest.mark.parametrize("base,dims,factor,original,fast,slow", [
    (1e4, 48, 6.0, 300, 16.0, 1.0), (3e5, 2, 2.0, 40, 1.0, 1.0), (80.0, 20, 4.0, 90, 50.0, 0.01),
])
def test_yarn(base, dims, factor, original, fast, slow):
    want, mult = oracle.yarn({"base": base, "dims": dims, "scaling": {
        "factor": factor, "original": original, "fast": fast, "slow": slow}})
    got, m = frequencies(base, dims, YarnScaling(factor, original, fast, slow))
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64), rtol=1e-12)
    assert abs(m - mult) < 1e-12


@pytest.mark.parametrize("H,G,dim,vdim,rot", [
    (6, 2, 12, 20, 8), (1, 1, 2, 1, 2), (5, 5, 70, 64, 70), (32, 8, 128, 128, 128),
    (8, 1, 256, 130, 64), (3, 1, 300, 8, 32), (48, 48, 128, 64, 20),
])
def test_norm_over_all_heads(device, dtype, H, G, dim, vdim, rot):
    """Row norms, rotation and cache write of rows at scattered positions and slots."""
    d, e, N, block = ops.latent_head(dim), ops.latent_head(vdim), 9, 4
    scaling, eps = YarnScaling(3.0, 64, 8.0, 1.0), 0.2
    pos = torch.tensor([0, 1, 2, 77, 5, 300, 8, 9, 131])
    table = rotation_table(301, 1e3, rot, scaling, device)
    x = {n: rand(N, heads * size, dtype=dtype, device="cpu", seed=i) * (i + 1)
         for i, (n, heads, size) in enumerate((("q", H, dim), ("k", G, dim), ("v", G, vdim)))}
    w = {n: 1 + 0.3 * rand(t.shape[1], dtype=dtype, device="cpu", seed=7) for n, t in x.items()}
    freqs, mult = oracle.yarn({"base": 1e3, "dims": rot, "scaling": {
        "factor": 3.0, "original": 64, "fast": 8.0, "slow": 1.0}})

    parts = [pad_to(pair_halves(x[n].view(N, h, dim), rot), N, h, d).flatten(1)
             for n, h in (("q", H), ("k", G))]
    parts.append(pad_to(x["v"].view(N, G, vdim), N, G, e).flatten(1))
    wide = torch.cat(parts + [torch.full((N, 16), 5.0, dtype=dtype)], 1).to(device)
    norms = [pad_to(pair_halves(w[n].view(h, dim), rot), h, d).flatten().contiguous().to(device)
             for n, h in (("q", H), ("k", G))]
    kc = torch.full((8, block, G, d), float("nan"), dtype=dtype, device=device)
    vc = torch.full((8, block, G, e), float("nan"), dtype=dtype, device=device)
    batch, _, _, _ = make_batch([(0, N)], block, device)
    batch.positions = pos.to(device)
    slots = torch.tensor([31, 0, 8, 7, 15, 16, 30, 1, 2])
    batch.slot_mapping = slots.to(device)
    q = ops.attention_inputs(
        wide[:, : wide.shape[1] - 16], H, dim, vdim, kc, vc, batch, eps, q_norm=norms[0],
        k_norm=norms[1], cos_sin=table,
    )
    for n, h, got in (("q", H, q), ("k", G, kc.view(-1, G, d)[slots.to(device)])):
        t = (oracle.rms(x[n].double(), eps) * w[n].double()).view(N, h, dim)
        for i, p in enumerate(pos.tolist()):
            turned = oracle.rotate(t[i : i + 1].expand(p + 1, -1, -1), freqs, mult)[-1]
            close(got[i, :, :dim], pair_halves(turned, rot), dtype)
        assert not got[..., dim:].any()
    assert torch.equal(vc.view(-1, G, e)[slots.to(device)][..., :vdim].cpu(),
                       x["v"].view(N, G, vdim))


# ------------------------------------------------- chunks, scores mixed over heads


def attend(q, k, v, ctx, scale, chunk, talk):
    """q [L, H, d], k [S, G, d], v [S, G, e] in double -> [L, H, e]."""
    L, H, S = q.shape[0], q.shape[1], k.shape[0]
    group = H // k.shape[1]
    s = torch.stack([q[:, n] @ k[:, n // group].T * scale for n in range(H)])
    if talk is not None:
        s = oracle.mixed_scores(s, talk)
    ok = oracle.visible(S, chunk or S)[ctx : ctx + L]
    a = oracle.softmax(s.masked_fill(~ok, -math.inf))
    return torch.stack([a[n] @ v[:, n // group] for n in range(H)], 1)


TALK = [
    # heads, kv heads, dim, vdim, chunk, talk, block, chunks
    (3, 3, 12, 20, 7, True, 4, [(0, 5), (0, 1), (9, 2), (130, 1), (63, 1), (62, 1), (0, 30)]),
    (4, 2, 64, 64, 19, True, 16, [(0, 40), (200, 2), (17, 3), (18, 1), (19, 1), (500, 1)]),
    (32, 8, 128, 128, 200, True, 16, [(0, 150), (300, 133), (64, 1), (1000, 1), (199, 1), (200, 1)]),
    (16, 8, 128, 128, 1000, True, 16, [(0, 9), (950, 130), (999, 1), (1000, 1), (1001, 1), (101, 30)]),
    (8, 1, 96, 128, 64, True, 16, [(0, 260), (1200, 1), (63, 1), (64, 1), (70, 2)]),
    (10, 2, 128, 64, None, True, 16, [(0, 100), (32, 1), (800, 1), (600, 43)]),
    (9, 3, 64, 100, 330, True, 8, [(0, 60), (700, 1), (329, 2), (400, 1)]),
    (6, 6, 64, 64, 50, True, 16, [(0, 60), (70, 1), (200, 2), (49, 1), (48, 4)]),
    (1, 1, 1, 1, 1, True, 1, [(0, 5), (3, 1), (8, 2)]),
    (12, 1, 64, 64, 90, True, 64, [(0, 130), (1, 1), (64, 1), (65, 64)]),
    (40, 8, 64, 64, 100, True, 16, [(0, 130), (91, 1), (300, 9)]),
    (2, 2, 256, 256, 33, True, 16, [(0, 40), (40, 1), (33, 2)]),
    (4, 2, 300, 30, 20, True, 16, [(0, 50), (70, 1), (39, 2)]),
    (18, 9, 64, 64, 40, True, 16, [(0, 50), (70, 1), (39, 2)]),
    # chunks alone
    (4, 2, 64, 64, 19, False, 16, [(0, 40), (200, 2), (17, 3), (18, 1), (19, 1), (500, 1)]),
    (8, 8, 128, 64, 130, False, 16, [(0, 260), (1200, 1), (259, 1), (260, 1), (777, 2)]),
    (6, 2, 20, 300, 64, False, 16, [(0, 70), (63, 1), (64, 1), (100, 40)]),
    (16, 4, 256, 128, 1, False, 64, [(0, 130), (1, 1), (64, 1), (65, 64)]),
]


def attention_case(H, G, d, e, block, chunks, dtype, device):
    """Unwritten pages are NaN: reading them shows."""
    D, E = ops.latent_head(d), ops.latent_head(e)
    batch, chunks, tables, pages = make_batch(chunks, block, device)
    kc = torch.full((pages, block, G, D), float("nan"), dtype=dtype)
    vc = torch.full((pages, block, G, E), float("nan"), dtype=dtype)
    kv = []
    for i, ((ctx, new), table) in enumerate(zip(chunks, tables)):
        k = rand(ctx + new, G, D, dtype=dtype, device="cpu", seed=10 + i)
        v = rand(ctx + new, G, E, dtype=dtype, device="cpu", seed=40 + i)
        k[..., d:], v[..., e:] = 0, 0
        paged(k, table, kc, block)
        paged(v, table, vc, block)
        kv.append((k.double(), v.double()))
    N = batch.num_tokens
    wide = rand(N, H * D + 64, dtype=dtype, device=device, seed=5)  # a row-strided query
    q = wide.as_strided((N, H, D), (H * D + 64, D, 1))
    q[..., d:] = 0
    return batch, chunks, q, kc.to(device), vc.to(device), kv


@pytest.mark.parametrize("H,G,d,e,chunk,talk,block,chunks", TALK)
def test_mixed_scores_in_chunks(device, dtype, H, G, d, e, chunk, talk, block, chunks):
    batch, chunks, q, kc, vc, kv = attention_case(H, G, d, e, block, chunks, dtype, device)
    N, E = q.shape[0], vc.shape[3]
    mix = rand(H, H, dtype=BF16, device="cpu", seed=6, scale=H ** -0.5).float() if talk else None
    scale = 1.5 * d ** -0.5
    out = torch.full((N, H * E + 32), 7.0, dtype=dtype, device=device)
    ops.grouped_attention(
        q, kc, vc, batch, scale, None, None, 0, None, out.as_strided((N, H, E), (H * E + 32, E, 1)),
        chunk=chunk, talk=None if mix is None else mix.to(device),
    )
    assert (out[:, H * E :] == 7.0).all()
    got, at = out[:, : H * E].view(N, H, E), 0
    for (ctx, new), (k, v) in zip(chunks, kv):
        want = attend(q[at : at + new].double().cpu(), k, v, ctx, scale, chunk,
                      None if mix is None else mix.double())
        close(got[at : at + new], want, dtype)
        at += new


def test_prompt_tiles_are_ordered_by_their_keys():
    batch, chunks, _, _ = make_batch([(0, 70), (25, 30), (7, 1), (100, 9)], 16, "cpu")
    meta = batch.prefill_meta(8, chunk=30)
    tiles = list(zip(meta.tile_seq.tolist(), meta.tile_q0.tolist()))
    plain = batch.prefill_meta(8)
    assert sorted(tiles) == sorted(zip(plain.tile_seq.tolist(), plain.tile_q0.tolist()))

    def keys(s, q0):
        ctx, new = chunks[s]
        return ctx + min(q0 + 8, new) - (ctx + q0) // 30 * 30

    assert [keys(*t) for t in tiles] == sorted(keys(*t) for t in tiles)


@pytest.mark.parametrize("H,G", [(9, 3), (8, 2), (32, 8)])
@pytest.mark.parametrize("portion", [1, 3, 100], ids=["decode", "portion", "prompt"])
def test_every_head_hears_the_right_one(device, dtype, portion, H, G):
    """Talk weights that permute the heads: a head attends by another one's scores, to its
    own values.  Each head's scores stand out at a key of its own."""
    d, S, block, chunk = 64, 230, 16, 1000
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    k = rand(S, G, d, dtype=dtype, device="cpu", seed=3, scale=0.02)
    v = rand(S, G, d, dtype=dtype, device="cpu", seed=4)
    key = [(37 * h + 5) % (S - portion) for h in range(H)]
    q = torch.zeros(portion, H, d, dtype=dtype)
    for h in range(H):
        q[:, h, h % d] = 1.0
        k[key[h], h // (H // G), h % d] = 40.0
    order = torch.randperm(H, generator=torch.Generator().manual_seed(1))
    talk = torch.eye(H)[order]
    kc, vc = (torch.zeros(pages, block, G, d, dtype=dtype) for _ in range(2))
    paged(k, tables[0], kc, block)
    paged(v, tables[0], vc, block)
    out = torch.empty(portion, H, d, dtype=dtype, device=device)
    ops.grouped_attention(q.to(device), kc.to(device), vc.to(device), batch, 1.0, None, None, 0,
                          None, out, chunk=chunk, talk=talk.to(device))
    for h in range(H):
        alone = v[key[int(order[h])], h // (H // G)]
        close(out[:, h], alone.expand(portion, d), dtype)


@pytest.mark.parametrize("talk", [True, False])
@pytest.mark.parametrize("portion", [1, 2, 140], ids=["decode", "portion", "prompt"])
@pytest.mark.parametrize("hit,seen", [
    ("self", True), ("chunk_in", True), ("chunk_out", False), ("page", True), ("first", False),
])
def test_standout_key(device, dtype, portion, hit, seen, talk):
    """One key scores far above the rest: its value comes back if it lies in the query's
    chunk, and never from the chunk before."""
    H, G, d, chunk, block, S = 4, 2, 64, 75, 16, 181
    i = S - 1
    j = {"self": i, "chunk_in": 150, "chunk_out": 149, "page": 160, "first": 0}[hit]
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    k = rand(S, G, d, dtype=dtype, device="cpu", seed=3, scale=0.02)
    v = rand(S, G, d, dtype=dtype, device="cpu", seed=4)
    k[j, :, 0] = 60.0
    kc, vc = (torch.zeros(pages, block, G, d, dtype=dtype) for _ in range(2))
    paged(k, tables[0], kc, block)
    paged(v, tables[0], vc, block)
    q = torch.zeros(portion, H, d, dtype=dtype)
    q[:, :, 0] = 1.0
    mix = torch.full((H, H), 0.25) if talk else None
    out = torch.empty(portion, H, d, dtype=dtype, device=device)
    ops.grouped_attention(q.to(device), kc.to(device), vc.to(device), batch, 1.0, None, None, 0,
                          None, out, chunk=chunk, talk=None if mix is None else mix.to(device))
    got = out[-1].double().cpu()
    near = (got - v[j].double().repeat_interleave(H // G, 0)).abs().max() < 0.02
    assert near == seen
    want = attend(q[-1:].double(), k.double(), v.double(), i, 1.0, chunk,
                  None if mix is None else mix.double())
    close(got, want[0], dtype)


def test_large_scores_keep_their_differences(device):
    """Scores near 2000 that differ by one: the mix and the softmax are 32-bit, so that
    the weights are right where 16 bits would tell nothing apart."""
    H, G, d, S = 4, 2, 64, 96
    for portion in (1, 40):
        batch, _, tables, pages = make_batch([(S - portion, portion)], 16, device)
        k = torch.zeros(S, G, d, dtype=BF16)
        k[:, :, 0] = 1.0
        k[:, :, 1] = (torch.arange(S) % 7).view(-1, 1).to(BF16)
        v = rand(S, G, d, dtype=BF16, device="cpu", seed=4)
        kc, vc = (torch.zeros(pages, 16, G, d, dtype=BF16) for _ in range(2))
        paged(k, tables[0], kc, 16)
        paged(v, tables[0], vc, 16)
        q = torch.zeros(portion, H, d, dtype=BF16)
        q[:, :, 0], q[:, :, 1] = 2048.0, 1.0
        talk = torch.eye(H) + torch.diag(torch.full((H - 1,), 0.5), 1)
        out = torch.empty(portion, H, d, dtype=BF16, device=device)
        ops.grouped_attention(q.to(device), kc.to(device), vc.to(device), batch, 1.0, None, None,
                              0, None, out, chunk=1000, talk=talk.to(device))
        want = attend(q.double(), k.double(), v.double(), S - portion, 1.0, 1000, talk.double())
        close(out, want, BF16)


# ------------------------------------------------------------------ delta rule


class HeadDeltaCase(DeltaCase):
    """One decay per head, a silu gate."""

    options = {"gate_silu": True}

    def __init__(self, H, *args, **kw):
        super().__init__(H, *args, **kw)
        n = self.z.shape[0]
        self.z = rand(n, H, dtype=self.dtype, device="cpu", seed=91, scale=2.0)
        self.dt_bias = rand(H, dtype=F32, device="cpu", seed=92) - 2

    def want(self, s):
        H, G, D, V, taps = self.shape
        T = self.lens[s]
        r = slice(self.start[s], self.start[s] + T)
        y = oracle.short_conv(self.qkv[r].double(), self.conv.double())
        q, k, v = y.split([G * D, G * D, H * V], 1)
        q = oracle.unit(q.view(T, G, D)) * D ** -0.5
        k, v = oracle.unit(k.view(T, G, D)), v.view(T, H, V)
        g = oracle.decay(self.z[r].double() + self.dt_bias.double(), self.A_log.double())
        beta = torch.sigmoid(self.b[r].double())
        o = torch.stack([
            oracle.delta_rule(q[:, n // (H // G)], k[:, n // (H // G)], v[:, n], g[:, n], beta[:, n])
            for n in range(H)
        ], 1)
        o = oracle.rms(o, self.eps) * self.norm.double()
        return o.view(T, H * V) * oracle.silu(self.gate[r].double())


DELTA = [
    # heads, key heads, dim, vdim, taps
    (4, 2, 12, 18, 3), (6, 3, 64, 64, 4), (2, 2, 128, 128, 4), (3, 1, 20, 7, 1),
    (2, 1, 256, 64, 2), (1, 1, 300, 40, 4), (2, 2, 16, 260, 5), (1, 1, 1, 1, 2),
    (1, 1, 600, 8, 4), (32, 16, 128, 128, 4), (8, 2, 32, 128, 4),
]


@pytest.mark.parametrize("H,G,D,V,taps", DELTA)
def test_head_delta_in_portions(device, dtype, H, G, D, V, taps):
    """Sequences of other lengths side by side, whole, in portions that are shorter
    and longer than the convolution and the kernels' token tiles, and token by token."""
    lens = [45, 1, 2, 35]
    case = HeadDeltaCase(H, G, D, V, taps, lens, dtype, device)
    plan = [[(0, 17), (3, 35)], [(1, 1), (0, 1)], [(0, 2), (2, 2)], [(0, 1)], [(0, 16)],
            [(0, 3)], [(0, 1)], [(0, 1)], [(0, 3)]]
    got = {s: [] for s in range(len(lens))}
    for portions in plan:
        for (s, _), rows in zip(portions, case.step(portions)):
            got[s].append(rows)
    for s in got:
        close(torch.cat(got[s]), case.want(s), dtype)


def test_many_sequences_fill_the_wide_scan(device, dtype):
    """Enough columns for two of them a lane."""
    case = HeadDeltaCase(16, 8, 128, 128, 4, [33] * 9, dtype, device)
    got = case.step([(s, 20) for s in range(9)])
    more = case.step([(s, 13) for s in range(9)])
    for s in range(9):
        close(torch.cat([got[s], more[s]]), case.want(s), dtype)


def test_head_delta_slot_is_used_again(device):
    case = HeadDeltaCase(2, 1, 16, 16, 4, [20, 15, 24], F32, device, slots=[3, 0, 3])
    first = case.step([(0, 20), (1, 6)])
    third = case.step([(2, 2)]) + case.step([(2, 21)]) + case.step([(2, 1)])
    second = case.step([(1, 9)])
    close(first[0], case.want(0), F32)
    close(torch.cat([first[1], second[0]]), case.want(1), F32)
    close(torch.cat(third), case.want(2), F32)


def test_head_delta_remembers_far_keys(device, dtype):
    """With a slow decay a value written once is read hundreds of tokens later by the
    same key; with a fast one it is gone."""
    T, D, V = 300, 32, 8
    case = HeadDeltaCase(2, 1, D, V, 4, [T + 1], dtype, device)
    case.A_log = torch.tensor([-12.0, 3.0])
    case.conv.zero_()[:, -1] = 1.0
    q, k, v = case.qkv[:, :D], case.qkv[:, D : 2 * D], case.qkv[:, 2 * D :]
    k[:, 0], q[:] = -30.0, -30.0       # silu(-30) = 0: other tokens leave channel 0 alone
    q[T, 0] = k[5, 0] = 9.0
    k[5, 1:] = -30.0
    v[5], case.b[5], case.gate[T] = 3.0, 20.0, 2.0
    got = torch.cat(case.step([(0, 200)]) + case.step([(0, T - 200)]) + case.step([(0, 1)]))
    want = case.want(0)
    close(got, want, dtype)
    assert want[T, :V].abs().min() > 50 * want[T, V:].abs().max()


def test_head_delta_extreme_decays(device):
    """Decays of exactly one and zero: no overflow, no loss."""
    case = HeadDeltaCase(2, 2, 16, 16, 4, [40], F32, device)
    case.z[::3], case.z[1::3] = 300.0, -300.0
    got = torch.cat(case.step([(0, 33)]) + case.step([(0, 1)]) + case.step([(0, 6)]))
    assert got.isfinite().all()
    close(got, case.want(0), F32)


# --------------------------------------------------- residual, gated units, routing


@pytest.mark.parametrize("n,w,top", [(1, 48, 1), (7, 251, 3), (4, 2048, 8), (600, 64, 0), (3, 4096, 4)])
def test_gated_normed_residual(device, dtype, n, w, top):
    """x + norm(sigmoid(gate) (y + experts)) and its copy in the model's dtype."""
    x, y = rand(n, w, dtype=F32, device=device), rand(n, w, dtype=dtype, device=device, seed=1)
    gate = rand(n, w + 16, dtype=dtype, device=device, seed=2, scale=2.0)[:, :w]
    weight = rand(w, dtype=dtype, device=device, seed=3)
    experts, add = None, y.double().cpu()
    if top:
        rows = rand(n, top, w, dtype=dtype, device=device, seed=4)
        weights = torch.rand(n, top, generator=torch.Generator().manual_seed(5)).to(device)
        experts = rows, weights
        add = add + (rows.double() * weights.double().unsqueeze(-1)).sum(1).cpu()
    add = add * torch.sigmoid(gate.double().cpu())
    want = x.double().cpu() + oracle.rms(add, 0.02) * weight.double().cpu()
    wide = torch.zeros(n, w + 12, dtype=dtype, device=device)
    ops.residual_norm(x, y, 0.02, weight, out=wide[:, :w], experts=experts, gate=gate)
    close(x, want, F32)
    close(wide[:, :w], want, dtype)
    assert not wide[:, w:].any()
    ops.residual_norm(x, y, 0.02, experts=experts, gate=gate)  # without the norm
    close(x, want + add, F32)


def test_dense_unit_with_biases(device, dtype):
    spec = gelu_glu(48, bias=True)
    assert spec.bias and spec.params(10) == 3 * 480 + 2 * 48 + 10
    x = rand(5, 96, dtype=dtype, device=device, scale=4.0)
    out = torch.empty(5, 48, dtype=dtype, device=device)
    ops.clamped_glu(x, spec.limit, spec.alpha, spec.offset, out, spec.cubic)
    g, u = x.double().cpu().chunk(2, -1)
    close(out, oracle.gelu_tanh(g) * u, dtype)


@pytest.mark.parametrize("n,E,K,top,scale", [
    (1, 8, 64, 2, 1.0), (37, 5, 192, 5, 2.5), (16, 1, 64, 1, 0.3), (130, 70, 128, 8, 1.5),
    (9, 200, 320, 3, 2.0), (33, 64, 2048, 6, 1.0), (5000, 32, 64, 4, 0.7),
])
def test_sigmoid_routing(device, dtype, n, E, K, top, scale):
    h = rand(n, K + 16, dtype=dtype, device=device)[:, :K]
    w = rand(E, K, dtype=dtype, device=device, seed=1, scale=2 * K ** -0.5)
    c = rand(E, dtype=F32, device=device, seed=2, scale=0.3)
    ids, weights = ops.moe_route(h, w, c, top, sigmoid=True, scale=scale)
    s = torch.sigmoid(h.double().cpu() @ w.double().cpu().T)
    key = s + c.double().cpu()
    assert all(len(set(r)) == top for r in ids.tolist())
    chosen = key.gather(1, ids.cpu().long()).sort(-1, descending=True).values
    # a close call may go either way, by rounding alone
    assert (chosen - torch.topk(key, top, -1).values).abs().max() < 1e-5
    mine = s.gather(1, ids.cpu().long())
    close(weights, mine / (mine.sum(-1, keepdim=True) + 1e-20) * scale, F32)


def test_correction_moves_the_choice_alone(device, dtype):
    """Equal scores: the corrections choose, and the weights stay equal.  Scores that
    vanish make no NaN."""
    w = torch.zeros(6, 64, dtype=dtype, device=device)
    c = torch.tensor([0.1, -0.3, 0.5, 0.0, 0.7, -9.0], device=device)
    ones = torch.ones(3, 64, dtype=dtype, device=device)
    ids, weights = ops.moe_route(ones, w, c, 3, sigmoid=True, scale=1.5)
    assert ids.tolist() == [[4, 2, 0]] * 3 and (weights - 0.5).abs().max() < 1e-6
    ids, weights = ops.moe_route(ones, w - 4, c, 3, sigmoid=True)  # logits of -256
    assert ids.tolist() == [[4, 2, 0]] * 3 and not weights.isnan().any()


@pytest.mark.parametrize("n,E,top", [(5, 4, 2), (300, 3, 1)])
def test_silu_experts(device, dtype, n, E, top):
    K, I, W = 128, 128, 96
    ids = torch.stack([torch.randperm(E, generator=torch.Generator().manual_seed(i))[:top]
                       for i in range(n)]).int()
    h = rand(n, K, dtype=dtype, device=device)
    gate_up = rand(E, 2 * I, K, dtype=dtype, device=device, seed=1, scale=2 * K ** -0.5)
    down = rand(E, W, I, dtype=dtype, device=device, seed=2, scale=I ** -0.5)
    got = ops.moe_experts(h, gate_up, down, ids.to(device), silu_glu(I)).cpu()
    for e in range(E):
        x = {"gate": gate_up[e, :I].double().cpu(), "up": gate_up[e, I:].double().cpu(),
             "down": down[e].double().cpu()}
        t, c = (ids == e).nonzero(as_tuple=True)
        if len(t):
            close(got[t, c], oracle.silu_glu(h.double().cpu()[t], x, ""), dtype)
