"""Lobuvik's mechanisms against their equations in double precision: rotations slowed
for long contexts, distance buckets, what happens to q, k and v ahead of attention,
sigmoid attention with distance biases, sinks in latent attention, head gates, the gelu
unit, routing and experts, and the residual update that collects them.  Runs on the CPU
ops and, marked gpu, on the HIP kernels."""
import math

import pytest
import torch

import lobuvik_oracle as oracle
from agentcontrolplane_amd import ops
from agentcontrolplane_amd.engine.config import (
    ClampedGluSpec, DistanceBias, WavelengthScaling, YarnScaling, gelu_glu,
)
from agentcontrolplane_amd.models.grouped_attention import distance_buckets
from agentcontrolplane_amd.models.layout import pair_halves, unpair_halves
from agentcontrolplane_amd.models.rotary import frequencies, rotation_table
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


# ------------------------------------------------------------------ positions


@pytest.mark.parametrize("base,dims,factor,original,fast,slow", [
    (1e4, 64, 8.0, 512, 32.0, 1.0), (5e5, 10, 2.5, 100, 4.0, 0.5), (1e4, 2, 3.0, 50, 1.0, 1.0),
    (100.0, 16, 4.0, 64, 40.0, 0.01),  # both ends of the ramp beyond the dimensions
])
def test_yarn(base, dims, factor, original, fast, slow):
    rot = {"base": base, "dims": dims, "scaling": {
        "factor": factor, "original": original, "fast": fast, "slow": slow}}
    want, mult = oracle.yarn(oracle.frequencies(rot), rot)
    got, m = frequencies(base, dims, YarnScaling(factor, original, fast, slow))
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64), rtol=1e-12) and m == mult
    table = rotation_table(70000, base, dims, YarnScaling(factor, original, fast, slow), "cpu")
    a = 69999 * torch.tensor(want, dtype=torch.float64)
    assert (table[0, -1] - m * a.cos()).abs().max() < 1e-6  # far positions keep precision
    assert (table[1, -1] - m * a.sin()).abs().max() < 1e-6


@pytest.mark.parametrize("base,dims,factor,low,high,original", [
    (1e4, 64, 8.0, 1.0, 4.0, 512), (3e5, 12, 2.0, 0.5, 6.0, 77), (50.0, 4, 32.0, 1.0, 1.5, 8192),
])
def test_wavelength_scaling(base, dims, factor, low, high, original):
    s = {"factor": factor, "low": low, "high": high, "original": original}
    f = oracle.frequencies({"base": base, "dims": dims})
    got, m = frequencies(base, dims, WavelengthScaling(factor, low, high, original))
    assert m == 1.0
    assert torch.allclose(got, torch.tensor(oracle.smoothed(f, s), dtype=torch.float64), rtol=1e-12)


def test_pairing_halves():
    t = torch.arange(11).view(1, 11)
    assert pair_halves(t, 6).tolist() == [[0, 3, 1, 4, 2, 5, 6, 7, 8, 9, 10]]
    assert torch.equal(unpair_halves(pair_halves(t, 6), 6), t)
    r = torch.arange(8).view(4, 2)
    assert torch.equal(unpair_halves(pair_halves(r, 4, 0), 4, 0), r)


@pytest.mark.parametrize("B,D", [(32, 128), (32, 200), (64, 512), (8, 30), (2, 9), (12, 6.5),
                                 (16, 128), (10, 1000)])
def test_distance_buckets(B, D):
    """Also reaches whose buckets begin exactly at a distance."""
    got = distance_buckets(DistanceBias(B, D)).tolist()
    assert got == [oracle.bucket(n, B, D) for n in range(len(got))]
    assert got[-1] == B - 1 and B - 1 not in got[:-1]
    assert oracle.bucket(10 ** 6, B, D) == B - 1
    if (B, D) == (32, 128):  # 16 * 2^(k/16 * 3): every 16/3 buckets the distance doubles
        assert [got[n] for n in (15, 16, 31, 32, 63, 64)] == [15, 16, 21, 21, 26, 26]
    if (B, D) == (16, 128):  # 8 * 2^(k/2): whole distances at even k
        assert [got[n] for n in (7, 8, 15, 16, 31, 32, 63, 64)] == [7, 8, 9, 10, 11, 12, 13, 14]


# ------------------------------------------------------------ attention inputs

INPUTS = [
    # heads, kv heads, dim, vdim, taps, norms, rotated dims, temperature, head factor
    (6, 2, 64, 48, 4, True, 0, (0.7, 7), False),
    (6, 3, 12, 20, 3, True, 8, None, True),
    (8, 1, 128, 128, 2, False, 128, (0.3, 1), True),
    (3, 3, 70, 256, 6, True, 2, (2.0, 100), False),
    (2, 1, 260, 64, 4, True, 60, None, True),
    (5, 5, 64, 130, 0, False, 32, None, True),
    (1, 1, 4, 1, 1, True, 0, None, False),
    (2, 2, 30, 300, 0, True, 0, (1.0, 3), False),
]


#: portions of every sequence, the step it begins in, its state slot: the last sequence
#: takes over the third one's slot after its end
SHORT = ([[7, 1, 1, 2, 12], [2, 3, 1, 3], [1, 20, 2, 17], [1, 1]], [0, 1, 0, 4], [2, 0, 1, 1])
#: enough rows for the kernel's longer turns, sequences that begin within one
LONG = ([[3, 2042, 2, 1], [2, 3, 1, 5], [1, 9, 2000, 90], [2, 50]], [0, 0, 0, 4], [0, 3, 1, 1])


@pytest.mark.parametrize("H,G,dim,vdim,taps,norms,rot,temp,mult", INPUTS)
def test_attention_inputs(device, dtype, H, G, dim, vdim, taps, norms, rot, temp, mult):
    """Sequences run in steps of unequal portions, down to one token, beside each other;
    state slots are handed on uncleared.  Queries and cached rows are those of the whole
    sequences."""
    run_attention_inputs(device, dtype, H, G, dim, vdim, taps, norms, rot, temp, mult, SHORT)


@pytest.mark.parametrize("H,G,dim,vdim,taps,norms,rot,temp,mult", [
    (2, 1, 60, 64, 4, True, 0, (0.7, 700), False), (1, 1, 64, 20, 3, True, 64, None, True),
    (3, 1, 64, 128, 0, False, 10, None, True),
])
def test_attention_inputs_of_long_prompts(device, dtype, H, G, dim, vdim, taps, norms, rot, temp,
                                          mult):
    run_attention_inputs(device, dtype, H, G, dim, vdim, taps, norms, rot, temp, mult, LONG)


def run_attention_inputs(device, dtype, H, G, dim, vdim, taps, norms, rot, temp, mult, steps):
    from agentcontrolplane_amd.engine.batch import FlatBatch, SeqMeta

    sizes, start, slot = steps
    d, e, block, eps = ops.latent_head(dim), ops.latent_head(vdim), 4, 1e-2
    C, lens = (H + G) * d + G * e, [sum(z) for z in sizes]
    live = torch.zeros(C, dtype=torch.bool)  # the rest is padding
    for n in range(H + G):
        live[n * d : n * d + dim] = True
    for n in range(G):
        at = (H + G) * d + n * e
        live[at : at + vdim] = True
    u = [rand(n, C, dtype=dtype, device="cpu", seed=i) * live for i, n in enumerate(lens)]
    conv = rand(taps, C, dtype=dtype, device="cpu", seed=9) if taps else None
    qn = kn = None
    if norms:
        qn, kn = (1 + 0.3 * rand(d, dtype=dtype, device="cpu", seed=s) for s in (10, 11))
    factor = 1 + rand(H, dtype=F32, device="cpu", seed=12) if mult else None
    table = rotation_table(2200, 300.0, rot, None, "cpu") if rot else None

    def whole(x):  # the mechanisms on a whole sequence, pairs (2i, 2i + 1) put back in halves
        T, x = len(x), x.double()
        if taps:
            x = oracle.short_conv(x, conv.double().T)
        q, k, v = x.split([H * d, G * d, G * e], 1)
        q, k, v = (t.reshape(T, n, s) for t, n, s in ((q, H, d), (k, G, d), (v, G, e)))
        if norms:
            q = oracle.rms(q[..., :dim], eps) * qn.double()[:dim]
            k = oracle.rms(k[..., :dim], eps) * kn.double()[:dim]
            v = oracle.rms(v[..., :vdim], eps)
        if rot:
            f = oracle.frequencies({"base": 300.0, "dims": rot})
            q, k = (pair_halves(oracle.rotate(unpair_halves(t, rot), f), rot) for t in (q, k))
        if mult:
            q = q * factor.double().view(1, H, 1)
        if temp:
            q = q * oracle.query_temperature(T, *temp).view(T, 1, 1)
        return [torch.nn.functional.pad(t, (0, s - t.shape[-1])) for t, s in
                ((q, d), (k, d), (v, e))]

    want = [whole(x) for x in u]
    pages, tables = 0, []
    for n in lens:
        tables.append(list(range(pages, pages + -(-n // block))))
        pages += len(tables[-1])
    kc = torch.full((pages, block, G, d), float("nan"), dtype=dtype, device=device)
    vc = torch.full((pages, block, G, e), float("nan"), dtype=dtype, device=device)
    ring = torch.full((4, max(taps, 1), C), float("nan"), dtype=dtype, device=device)
    at, dev = [0] * 4, lambda t: None if t is None else t.to(device)  # noqa: E731
    for step in range(max(s + len(z) for s, z in zip(start, sizes))):
        parts = [(i, sizes[i][step - start[i]]) for i in range(4)
                 if start[i] <= step < start[i] + len(sizes[i])]
        parts.sort(key=lambda p: p[1] == 1 and at[p[0]] > 0)  # decode rows come last
        prefills = [SeqMeta(i, n, at[i] + n, at[i], tables[i], True, slot[i])
                    for i, n in parts if n > 1 or at[i] == 0]
        dec = [i for i, n in parts if n == 1 and at[i] > 0]
        places = [(i, at[i] + k) for i, n in parts for k in range(n)]

        def t(x, kind=torch.long):
            return torch.tensor(x, dtype=kind, device=device)

        batch = FlatBatch(
            token_ids=t([0] * len(places)), positions=t([p for _, p in places]),
            slot_mapping=t([tables[i][p // block] * block + p % block for i, p in places]),
            prefills=prefills, num_prefill_tokens=sum(m.query_len for m in prefills),
            decode_seq_ids=dec, decode_block_tables=t([tables[i][:1] for i in dec]) if dec else None,
            decode_seq_lens=t([at[i] + 1 for i in dec]) if dec else None, logit_rows=t([0]),
            sample_seq_ids=[],
            decode_state_slots=t([slot[i] for i in dec], torch.int32) if dec else None,
        )
        wide = torch.full((len(places), C + 24), 7.0, dtype=dtype, device=device)
        wide[:, :C] = torch.stack([u[i][p] for i, p in places]).to(device)
        q = ops.attention_inputs(
            wide[:, :C], H, dim, vdim, kc, vc, batch, eps, conv=dev(conv),
            ring=ring if taps else None, q_norm=dev(qn), k_norm=dev(kn), v_norm=norms,
            cos_sin=dev(table), head_mult=dev(factor), q_temp=temp,
        )
        close(q, torch.stack([want[i][0][p] for i, p in places]), dtype)
        for i, n in parts:
            at[i] += n
    assert at == lens
    for i, n in enumerate(lens):
        rows = torch.tensor([tables[i][p // block] * block + p % block for p in range(n)])
        close(kc.cpu().view(-1, G, d)[rows], want[i][1], dtype)
        close(vc.cpu().view(-1, G, e)[rows], want[i][2], dtype)


# ----------------------------------------------------------- grouped attention


def paged(rows, table, cache, block):
    for p, page in enumerate(table):
        part = rows[p * block : (p + 1) * block]
        cache[page, : len(part)] = part


def attend(q, k, v, ctx, scale, cap, window, bias, sigmoid, gate):
    """q [L, H, d], k [S, G, d], v [S, G, e] in double -> [L, H, e]."""
    L, H, S = q.shape[0], q.shape[1], k.shape[0]
    ok = oracle.visible(S, window)[ctx : ctx + L]
    far = (torch.arange(S).view(-1, 1) - torch.arange(S))[ctx : ctx + L].clamp(min=0)
    out = []
    for n in range(H):
        j = n // (H // k.shape[1])
        s = q[:, n] @ k[:, j].T * scale
        if cap:
            s = oracle.cap(s, cap)
        if bias is not None:
            s = s + bias[n][far.clamp(max=bias.shape[1] - 1)]
        a = oracle.sigmoid_weights(s, ok) if sigmoid else oracle.sink_softmax(
            s.masked_fill(~ok, -math.inf))
        out.append(a @ v[:, j])
    out = torch.stack(out, 1)
    return out if gate is None else out * torch.sigmoid(gate).unsqueeze(-1)


FORMS = [
    # heads, kv heads, dim, vdim, window, cap, biased distances, sigmoid, gate, block, chunks
    (6, 2, 64, 32, None, None, 60, True, False, 16, [(0, 40), (200, 2), (17, 3), (300, 1), (59, 1)]),
    (6, 3, 12, 20, None, None, 1, True, True, 4, [(0, 5), (0, 1), (9, 2), (130, 1), (63, 1)]),
    (8, 1, 128, 128, 100, None, 300, True, True, 16, [(0, 9), (350, 1), (99, 1), (101, 130)]),
    (8, 8, 128, 64, None, None, 3, True, False, 16, [(0, 260), (1200, 1), (777, 2), (2, 1)]),
    (9, 1, 256, 250, 50, None, 40, True, True, 8, [(0, 60), (70, 1), (70, 2), (400, 1)]),
    (2, 2, 300, 40, None, None, 90, True, True, 16, [(0, 60), (70, 1), (200, 2)]),
    (1, 1, 1, 1, None, None, 2, True, False, 1, [(0, 5), (3, 1), (8, 2)]),
    (16, 4, 64, 128, None, None, 129, True, True, 64, [(0, 130), (1, 1), (64, 1), (65, 64)]),
    (12, 4, 64, 64, 43, 20.0, 0, False, True, 16, [(0, 100), (42, 1), (43, 1), (44, 1), (600, 3)]),
    (4, 4, 96, 70, None, None, 33, False, True, 16, [(0, 70), (500, 1), (31, 2)]),
    (4, 2, 64, 64, 70, 3.0, 50, False, True, 16, [(0, 170), (500, 1), (70, 1), (31, 2)]),
    (4, 2, 64, 64, None, 2.0, 30, True, False, 16, [(0, 50), (500, 1), (31, 2)]),
]


@pytest.mark.parametrize("H,G,d,e,window,cap,near,sigmoid,gated,block,chunks", FORMS)
def test_attention_forms(device, dtype, H, G, d, e, window, cap, near, sigmoid, gated, block,
                         chunks):
    D, E = ops.latent_head(d), ops.latent_head(e)
    batch, chunks, tables, pages = make_batch(chunks, block, device)
    # what a sequence has not written is NaN: reading it shows
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
    gate = rand(N, H + 16, dtype=dtype, device=device, seed=6, scale=2.0)[:, :H] if gated else None
    bias = rand(H, near, dtype=F32, device=device, seed=7, scale=1.5) - 2 if near else None
    scale = 1.5 * d ** -0.5
    out = torch.full((N, H * E + 32), 7.0, dtype=dtype, device=device)
    ops.grouped_attention(
        q, kc.to(device), vc.to(device), batch, scale, cap, window, 0, None,
        out.as_strided((N, H, E), (H * E + 32, E, 1)), bias=bias, sigmoid=sigmoid, gate=gate,
    )
    assert (out[:, H * E :] == 7.0).all()
    got, at = out[:, : H * E].view(N, H, E), 0
    for (ctx, new), (k, v) in zip(chunks, kv):
        want = attend(q[at : at + new].double().cpu(), k, v, ctx, scale, cap, window,
                      None if bias is None else bias.double().cpu(), sigmoid,
                      None if gate is None else gate[at : at + new].double().cpu())
        close(got[at : at + new], want, dtype)
        at += new


@pytest.mark.parametrize("portion", [1, 3, 140], ids=["decode", "portion", "prompt"])
@pytest.mark.parametrize("back", [0, 1, 15, 16, 63, 64, 99, 100, 170])
def test_standout_distance(device, dtype, portion, back):
    """All keys score far below zero but one, or one distance: with sigmoid weights, just
    its value comes back, whole, on either side of page edges and of the last distance
    with a bias of its own."""
    H, G, S, block, near = 4, 2, 171, 16, 101
    i, j = S - 1, S - 1 - back
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    v = rand(S, G, 64, dtype=dtype, device="cpu", seed=4)
    for by_key in (False, True):
        k = torch.zeros(S, G, 64, dtype=dtype)
        bias = torch.full((H, near), -30.0)
        if by_key:
            k[j, :, 0] = 60.0
        elif back < near - 1:
            bias[:, back] = 30.0
        else:
            continue
        kc, vc = (torch.zeros(pages, block, G, 64, dtype=dtype) for _ in range(2))
        paged(k, tables[0], kc, block)
        paged(v, tables[0], vc, block)
        q = torch.zeros(portion, H, 64, dtype=dtype)
        q[:, :, 0] = 1.0
        out = torch.empty(portion, H, 64, dtype=dtype, device=device)
        ops.grouped_attention(q.to(device), kc.to(device), vc.to(device), batch, 1.0, None, None,
                              0, None, out, bias=bias.to(device), sigmoid=True)
        close(out[-1], v[j].double().repeat_interleave(H // G, 0), dtype)


@pytest.mark.parametrize("portion", [1, 2, 70])
def test_sigmoid_weights_add_up(device, dtype, portion):
    """n equal keys weigh n times one: nothing is normalized, no key counts twice, also
    where a row's keys are split over workgroups."""
    H, S, block = 2, 900, 16
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    kc = torch.zeros(pages, block, 1, 64, dtype=dtype, device=device)
    vc = torch.ones(pages, block, 1, 64, dtype=dtype, device=device)
    q = torch.zeros(portion, H, 64, dtype=dtype, device=device)
    out = torch.empty(portion, H, 64, dtype=dtype, device=device)
    bias = torch.tensor([[-3.0], [0.5]], device=device)
    ops.grouped_attention(q, kc, vc, batch, 1.0, None, None, 0, None, out, bias=bias, sigmoid=True)
    want = torch.sigmoid(bias.double().cpu()) * torch.arange(S - portion + 1, S + 1).double()
    close(out, want.T.unsqueeze(-1).expand(-1, -1, 64), dtype)


# ------------------------------------------------------ sinks, latent attention


def still(positions, device):
    """A rotation table that does not rotate."""
    t = torch.zeros(2, positions, 32, device=device)
    t[0] = 1.0
    return t


SINKS = [
    # heads, latent, window, chunks
    (3, 24, None, [(0, 5), (0, 20), (100, 3), (130, 1), (0, 1)]),
    (6, 64, 40, [(0, 100), (39, 1), (40, 1), (700, 1), (300, 2)]),
    (20, 500, 33, [(0, 40), (500, 1), (32, 1)]),
    (40, 130, 1, [(0, 9), (17, 1)]),
    (2, 600, 20, [(0, 30), (90, 1)]),
]


@pytest.mark.parametrize("H,kv_rank,window,chunks", SINKS)
def test_latent_sink(device, dtype, H, kv_rank, window, chunks):
    """The sink joins the denominator once, whatever the row tile, split or portion."""
    rank = ops.latent_rank(kv_rank)
    row, block = rank + 64, 16
    batch, chunks, tables, pages = make_batch(chunks, block, device)
    cache = torch.full((pages, block, row), float("nan"), dtype=dtype)
    kv = []
    for i, ((ctx, new), table) in enumerate(zip(chunks, tables)):
        r = rand(ctx + new, row, dtype=dtype, device="cpu", seed=10 + i)
        r[:, kv_rank:rank] = 0
        paged(r, table, cache, block)
        kv.append(r.double())
    q = rand(batch.num_tokens, H, rank, dtype=dtype, device=device, seed=5)
    q_rot = rand(batch.num_tokens, H, 64, dtype=dtype, device=device, seed=6)
    sink = 3.0 * rand(H, dtype=F32, device=device, seed=7) + 2.0
    scale = 0.3 * kv_rank ** -0.5
    got = ops.latent_attention(q, q_rot, still(1000, device), 64, cache.to(device), batch, scale,
                               window, sink=sink).cpu()
    full, at = torch.cat([q, q_rot], -1).double().cpu(), 0
    for (ctx, new), rows in zip(chunks, kv):
        s = torch.einsum("lhr,sr->hls", full[at : at + new], rows) * scale
        s = s.masked_fill(~oracle.visible(ctx + new, window)[ctx:], -math.inf)
        for h in range(H):
            want = oracle.sink_softmax(s[h], sink[h].double().cpu()) @ rows[:, :rank]
            close(got[at : at + new, h], want, dtype)
        at += new


@pytest.mark.gpu
@pytest.mark.parametrize("H,d,v,rank,window,chunks", [
    (3, 64, 64, 64, None, [(0, 5), (0, 200), (100, 130)]),
    (8, 128, 64, 512, 70, [(0, 333), (500, 40), (69, 2), (70, 2)]),
    (2, 256, 256, 128, 1, [(0, 130), (77, 3)]),
])
def test_expanded_latent_sink(H, d, v, rank, window, chunks):
    device, dtype, row = "cuda", BF16, rank + 64
    batch, chunks, tables, pages = make_batch(chunks, 16, device)
    cache = torch.full((pages, 16, row), float("nan"), dtype=dtype)
    kv = []
    for i, ((ctx, new), table) in enumerate(zip(chunks, tables)):
        r = rand(ctx + new, row, dtype=dtype, device="cpu", seed=10 + i)
        paged(r, table, cache, 16)
        kv.append(r.double())
    N = batch.num_tokens
    q = rand(N, H, d + 64, dtype=dtype, device=device, seed=5)
    w = rand(H * (d + v), rank, dtype=dtype, device=device, seed=6, scale=rank ** -0.5)
    sink = 3.0 * rand(H, dtype=F32, device=device, seed=7) + 2.0
    out = torch.empty(N, H, v, dtype=dtype, device=device)
    scale = 0.5 * d ** -0.5
    ops.latent_expanded_prefill(
        q, w, None, still(1000, device), 64, cache.to(device), batch,
        tuple(range(len(batch.prefills))), rank, scale, window, out, sink,
    )
    wk, wv = w.double().cpu().split([H * d, H * v])
    at = 0
    for (ctx, new), rows in zip(chunks, kv):
        k = (rows[:, :rank] @ wk.T).to(dtype).double().view(-1, H, d)
        val = (rows[:, :rank] @ wv.T).to(dtype).double().view(-1, H, v)
        qd = q[at : at + new].double().cpu()
        for h in range(H):
            s = (qd[:, h, :d] @ k[:, h].T + qd[:, h, d:] @ rows[:, rank:].T) * scale
            s = s.masked_fill(~oracle.visible(ctx + new, window)[ctx:], -math.inf)
            close(out[at : at + new, h], oracle.sink_softmax(s, sink[h].double().cpu()) @ val[:, h],
                  dtype)
        at += new


# --------------------------------------------------------- norms, gated units


@pytest.mark.parametrize("n,w,top", [(1, 48, 1), (7, 251, 3), (4, 2048, 8), (600, 64, 4)])
def test_residual_with_expert_rows_and_two_norms(device, dtype, n, w, top):
    x, y = rand(n, w, dtype=F32, device=device), rand(n, w, dtype=dtype, device=device, seed=1)
    rows = rand(n, top, w, dtype=dtype, device=device, seed=2)
    weights = torch.rand(n, top, generator=torch.Generator().manual_seed(3)).to(device)
    w1, w2 = (rand(w, dtype=dtype, device=device, seed=s) for s in (4, 5))
    want = x.double().cpu() + y.double().cpu() + (
        rows.double() * weights.double().unsqueeze(-1)).sum(1).cpu()
    out = torch.empty(n, w, dtype=dtype, device=device)
    wide = torch.zeros(n, w + 12, dtype=dtype, device=device)
    ops.residual_norm(x, y, 1e-2, None, w1, out, x_norm2=w2, out2=wide[:, :w],
                      experts=(rows, weights))
    close(x, want, F32)
    close(out, oracle.layer_norm(want, w1.double().cpu(), 1e-2), dtype)
    close(wide[:, :w], oracle.layer_norm(want, w2.double().cpu(), 1e-2), dtype)
    assert not wide[:, w:].any()
    ops.residual_norm(x, y, 1e-2, experts=(rows, weights))  # the residual only
    close(x, 2 * want - rand(n, w, dtype=F32, device="cpu").double(), F32)


def test_gelu_glu(device, dtype):
    spec = gelu_glu(48)
    x = rand(5, 96, dtype=dtype, device=device, scale=4.0)
    x[0, :4] = torch.tensor([0.0, 30.0, -30.0, -1e4])
    out = torch.empty(5, 48, dtype=dtype, device=device)
    ops.clamped_glu(x, spec.limit, spec.alpha, spec.offset, out, spec.cubic)
    g, u = x.double().cpu().chunk(2, -1)
    close(out, oracle.gelu_tanh(g) * u, dtype)


def test_scaled_embedding(device, dtype):
    tok = torch.tensor([4, 0, 9], device=device)
    table = rand(10, 37, dtype=dtype, device=device)
    x = torch.empty(3, 37, device=device)
    ops.embed_positions(tok, tok, table, None, x, scale=0.3)
    close(x, 0.3 * table.double().cpu()[tok.cpu()], F32)


# -------------------------------------------------------------------- experts


@pytest.mark.parametrize("n,E,K,top", [
    (1, 8, 64, 2), (37, 5, 192, 5), (16, 1, 64, 1), (130, 70, 128, 8), (9, 200, 320, 3),
    (33, 64, 2048, 6), (5000, 32, 64, 4),
])
def test_route(device, dtype, n, E, K, top):
    h = rand(n, K + 16, dtype=dtype, device=device)[:, :K]
    w = rand(E, K, dtype=dtype, device=device, seed=1, scale=K ** -0.5)
    b = rand(E, dtype=F32, device=device, seed=2, scale=0.5)
    ids, weights = ops.moe_route(h, w, b, top)
    z = h.double().cpu() @ w.double().cpu().T + b.double().cpu()
    assert ids.shape == weights.shape == (n, top) and weights.dtype == F32
    chosen = z.gather(1, ids.cpu().long())
    assert all(len(set(r)) == top for r in ids.tolist())
    best = torch.topk(z, top, -1).values
    # a close call may go either way, by rounding alone
    assert (chosen.sort(-1, descending=True).values - best).abs().max() < 1e-5
    close(weights, torch.softmax(chosen, -1), F32)
    assert torch.equal(ops.moe_route(h, w, None, top)[0].sort(-1).values.cpu(),
                       ops.moe_route(h, w, torch.full_like(b, 3.0), top)[0].sort(-1).values.cpu())


def test_route_ties_and_order(device, dtype):
    """Equal logits: the lower expert first; the weights fall."""
    w = torch.zeros(6, 64, dtype=dtype, device=device)
    b = torch.tensor([1.0, 3.0, 3.0, 0.0, 3.0, 2.0], device=device)
    ids, weights = ops.moe_route(torch.ones(3, 64, dtype=dtype, device=device), w, b, 4)
    if device == "cuda":
        assert ids.tolist() == [[1, 2, 4, 5]] * 3
    assert (weights[:, :-1] >= weights[:, 1:]).all()


EXPERTS = [
    # tokens, experts, top, K, inner, W: few and many rows per expert, padded inner sizes
    (1, 4, 2, 64, 64, 40), (3, 6, 3, 192, 64, 160), (50, 8, 4, 128, 128, 96),
    (70, 3, 2, 64, 192, 31), (300, 4, 2, 128, 128, 130), (700, 2, 1, 256, 256, 258),
    (260, 3, 3, 128, 384, 512), (40, 40, 1, 64, 64, 64), (1030, 5, 2, 512, 128, 72),
]


@pytest.mark.parametrize("skew", [False, True])
@pytest.mark.parametrize("n,E,top,K,I,W", EXPERTS)
def test_experts(device, dtype, n, E, top, K, I, W, skew):
    """Every entry gets its own expert's unit of its own row; with skew nearly all tokens
    go to one expert and some experts get none."""
    g = torch.Generator().manual_seed(n)
    p = torch.ones(n, E)
    if skew:
        p[:, 0], p[: n - 1, top + 1 :] = 1e4, 1e-12
    ids = torch.multinomial(p, top, generator=g).int()
    h = rand(n, K + 64, dtype=dtype, device=device)[:, :K]
    gate_up = rand(E, 2 * I, K, dtype=dtype, device=device, seed=1, scale=2 * K ** -0.5)
    down = rand(E, W, I, dtype=dtype, device=device, seed=2, scale=I ** -0.5)
    got = ops.moe_experts(h, gate_up, down, ids.to(device), ClampedGluSpec(I, 1.25)).cpu()
    assert got.shape == (n, top, W) and got.dtype == dtype
    hd = h.double().cpu()
    for e in range(E):
        x = {"gate": gate_up[e, :I].double().cpu(), "up": gate_up[e, I:].double().cpu(),
             "down": down[e].double().cpu()}
        t, c = (ids == e).nonzero(as_tuple=True)
        if len(t):
            close(got[t, c], oracle.clamped_glu(hd[t], x, "", 1.25), dtype)
