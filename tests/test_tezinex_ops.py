"""Mechanism ops against their equations in double precision: RMS norms with an
offset and the depth average, sinusoidal positions, capped logits, grouped attention
with windows, kept tokens, caps and sinks, and the gated delta rule with its state
slots.  Runs on the CPU ops and, marked gpu, on the HIP kernels."""
import math

import pytest
import torch

import tezinex_oracle as oracle
from agentcontrolplane_amd import ops
from agentcontrolplane_amd.engine.batch import FlatBatch, SeqMeta
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


# ------------------------------------------------------- norms, depth average


@pytest.mark.parametrize("n,w", [(1, 48), (7, 251), (4, 2048)])
@pytest.mark.parametrize("y_norm,x_norm", [(0, 0), (1, 0), (0, 1), (1, 1)])
def test_rms_residual_norm(device, dtype, n, w, y_norm, x_norm):
    """x += m rms(y) (1 + wy); then rms(x) (1 + wx), into a strided view."""
    x = rand(n, w, dtype=F32, device=device) + 2.0  # a mean that must stay in
    y = rand(n, w, dtype=dtype, device=device, seed=1, scale=0.01)
    wy = rand(w, dtype=dtype, device=device, seed=2, scale=0.4) if y_norm else None
    wx = rand(w, dtype=dtype, device=device, seed=3, scale=0.4) if x_norm else None
    eps, m = 1e-4, 0.37  # eps the size of mean(y^2): inside the root shows
    xd, yd = x.double().cpu(), y.double().cpu()
    if y_norm:
        yd = oracle.norm(yd, wy.double().cpu(), eps)
    xd = xd + m * yd
    wide = torch.zeros(n, w + 8, dtype=dtype, device=device)
    ops.residual_norm(x, y, eps, wy, wx, wide[:, 8:], center=False, offset=1.0, mult=m)
    close(x, xd, F32)
    close(wide[:, 8:], oracle.norm(xd, wx.double().cpu(), eps) if x_norm else xd, dtype)
    assert not wide[:, :8].any()


@pytest.mark.parametrize("layers", [1, 2, 4, 5, 11])
@pytest.mark.parametrize("n,w", [(3, 64), (2, 129)])
def test_depth_average(device, dtype, layers, n, w):
    """Every layer's result is filed before the averaging; weights of all layers
    differ, so that a state taken twice, left out or averaged too early shows."""
    coef = torch.zeros(layers, layers + 1)
    for i in range(layers):
        coef[i, : i + 2] = rand(i + 2, dtype=F32, device="cpu", seed=50 + i)
    depth = ops.Depth.new(coef.to(device), n, w)
    x = rand(n, w, dtype=F32, device=device)
    depth.states[0] = x
    wx = rand(w, dtype=dtype, device=device, seed=1)
    xd = x.double().cpu()
    states = [xd]
    for i in range(layers):
        y = rand(n, w, dtype=dtype, device=device, seed=10 + i)
        out = torch.empty(n, w, dtype=dtype, device=device)
        ops.residual_norm(x, y, 1e-5, None, wx, out, center=False, offset=1.0, mult=0.5,
                          depth=depth, layer=i)
        states.append(xd + 0.5 * y.double().cpu())
        xd = oracle.depth_average(states, coef[i, : i + 2].double())
        close(depth.states[i + 1], states[-1], F32)
        close(x, xd, F32)
        close(out, oracle.norm(xd, wx.double().cpu(), 1e-5), dtype)


@pytest.mark.parametrize("w", [6, 33, 256, 1028])
def test_embed_positions(device, dtype, w):
    """Far positions: angles must not lose precision."""
    pos = torch.tensor([0, 1, 2, 4095, 777])
    tok = torch.tensor([4, 0, 9, 9, 1])
    table = rand(10, w, dtype=dtype, device=device)
    cos_sin = build_cos_sin(4096, w, 10000.0, device, exact=True)
    x, copy = (torch.empty(5, w, device=device) for _ in range(2))
    ops.embed_positions(tok.to(device), pos.to(device), table, cos_sin, x, copy)
    want = table.double().cpu()[tok] + oracle.positions(4096, w)[pos]
    assert (x.double().cpu() - want).abs().max() < 1e-6 * max(1, want.abs().max())
    assert torch.equal(x, copy)
    ops.embed_positions(tok.to(device), pos.to(device), table, None, x)
    assert torch.equal(x, table[tok.to(device)].float())


def test_softcap(device, dtype):
    x = torch.cat([rand(5, 77, dtype=F32, device=device, scale=20.0),
                   torch.tensor([[0.0, 1e-3, 500.0, -500.0] + [1.0] * 73], device=device)])
    x = x.to(dtype)
    got = ops.softcap(x, 7.0)
    assert got.dtype == F32
    assert (got.double().cpu() - oracle.cap(x.double().cpu(), 7.0)).abs().max() < 5e-6
    assert torch.equal(ops.softcap(x, None), x.float())


def test_silu_glu(device, dtype):
    """The clamped GLU without its clamp is silu(gate) * up."""
    from agentcontrolplane_amd.engine.config import silu_glu

    spec = silu_glu(48)
    x = rand(5, 96, dtype=dtype, device=device, scale=4.0)
    out = torch.empty(5, 48, dtype=dtype, device=device)
    ops.clamped_glu(x, spec.limit, spec.alpha, spec.offset, out)
    g, u = x.double().cpu().chunk(2, -1)
    close(out, oracle.silu(g) * u, dtype)


# --------------------------------------------------------- grouped attention


def paged(rows, table, cache, block):
    for p, page in enumerate(table):
        part = rows[p * block : (p + 1) * block]
        cache[page, : len(part)] = part


def attend(q, k, v, ctx, scale, cap, window, keep, sink):
    """q [L, H, d], k [S, G, d], v [S, G, e] in double -> [L, H, e]."""
    L, H, S = q.shape[0], q.shape[1], k.shape[0]
    ok = oracle.visible(S, window or S + 1, keep)[ctx : ctx + L]
    out = []
    for n in range(H):
        j = n // (H // k.shape[1])
        s = q[:, n] @ k[:, j].T * scale
        if cap:
            s = oracle.cap(s, cap)
        s = s.masked_fill(~ok, -math.inf)
        a = torch.softmax(s, -1) if sink is None else oracle.sink_softmax(s, sink[n])
        out.append(a @ v[:, j])
    return torch.stack(out, 1)


ATTN = [
    # heads, kv heads, dim, vdim, window, keep, cap, sink, block, chunks
    (3, 3, 12, 20, None, 0, None, False, 4, [(0, 5), (0, 1), (9, 2), (130, 1), (63, 1)]),
    (4, 2, 64, 64, 19, 3, 5.0, True, 16, [(0, 40), (200, 2), (17, 3), (18, 1), (19, 1), (500, 1)]),
    (6, 2, 96, 128, 64, 70, 2.0, True, 16, [(0, 150), (300, 33), (64, 1), (1000, 1), (134, 1)]),
    (8, 1, 128, 128, 100, 1, 30.0, True, 16, [(0, 9), (350, 1), (99, 1), (100, 1), (101, 130)]),
    (8, 8, 128, 64, 130, 65, None, True, 16, [(0, 260), (1200, 1), (777, 2), (194, 1)]),
    (10, 2, 64, 200, 33, 0, 4.0, False, 16, [(0, 100), (32, 1), (33, 1), (600, 3)]),
    (9, 1, 256, 250, 50, 5, 9.0, True, 8, [(0, 60), (70, 1), (70, 2), (400, 1)]),
    (2, 2, 300, 40, 50, 7, 3.0, True, 16, [(0, 60), (70, 1), (200, 2)]),
    (1, 1, 1, 1, 1, 0, 1.0, True, 1, [(0, 5), (3, 1), (8, 2)]),
    (16, 4, 64, 128, 2, 1, 8.0, True, 64, [(0, 130), (1, 1), (64, 1), (65, 64)]),
]


@pytest.mark.parametrize("H,G,d,e,window,keep,cap,sink,block,chunks", ATTN)
def test_grouped_attention(device, dtype, H, G, d, e, window, keep, cap, sink, block, chunks):
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
    sk = rand(H, dtype=F32, device=device, seed=7, scale=2.0) + 1 if sink else None
    scale = 2.0 * d ** -0.5
    out = torch.empty(N, H, E, dtype=dtype, device=device)
    ops.grouped_attention(q, kc.to(device), vc.to(device), batch, scale, cap, window, keep, sk, out)
    at = 0
    for (ctx, new), (k, v) in zip(chunks, kv):
        want = attend(q[at : at + new].double().cpu(), k, v, ctx, scale, cap, window, keep,
                      None if sk is None else sk.double().cpu())
        close(out[at : at + new], want, dtype)
        at += new


@pytest.mark.parametrize("portion", [1, 3, 140], ids=["decode", "portion", "prompt"])
@pytest.mark.parametrize("hit,seen", [
    ("self", True), ("window_in", True), ("window_out", False), ("kept", True),
    ("first", True), ("not_kept", False), ("page", True),
])
def test_standout_key(device, dtype, portion, hit, seen):
    """One key scores far above the rest: its value must come back where the query
    sees it, and never where it has just left the window or the kept tokens."""
    H, G, d, e, window, keep, S, block = 4, 2, 64, 64, 40, 6, 171, 16
    i = S - 1
    j = {"self": i, "window_in": i - window + 1, "window_out": i - window, "kept": keep - 1,
         "first": 0, "not_kept": keep, "page": 143}[hit]
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    k = rand(S, G, d, dtype=dtype, device="cpu", seed=3, scale=0.02)
    v = rand(S, G, e, dtype=dtype, device="cpu", seed=4)
    k[j, :, 0] = 30.0
    kc, vc = (torch.zeros(pages, block, G, n, dtype=dtype) for n in (d, e))
    paged(k, tables[0], kc, block)
    paged(v, tables[0], vc, block)
    q = torch.zeros(portion, H, d, dtype=dtype)
    q[:, :, 0] = 1.0
    out = torch.empty(portion, H, e, dtype=dtype, device=device)
    ops.grouped_attention(q.to(device), kc.to(device), vc.to(device), batch, 1.0, 25.0, window,
                          keep, torch.zeros(H, device=device), out)
    got = out[-1].double().cpu()
    alone = v[j].double().repeat_interleave(H // G, 0)
    near = (got - alone).abs().max() < 0.02
    assert near == seen, (got - alone).abs().max()
    want = attend(q[-1:].double(), k.double(), v.double(), i, 1.0, 25.0, window, keep,
                  torch.zeros(H, dtype=torch.float64))
    close(got, want[0], dtype)


@pytest.mark.parametrize("portion", [1, 2, 70])
def test_sink_takes_its_share(device, dtype, portion):
    """Equal scores s over n visible keys: what remains of a constant value is
    n e^s / (n e^s + e^sink); the sink is neither scaled nor capped, and counts once,
    also where a row's keys are split or lie in both key ranges."""
    H, S, block, window, keep = 2, 300, 16, 200, 4
    batch, _, tables, pages = make_batch([(S - portion, portion)], block, device)
    kc = torch.zeros(pages, block, 1, 64, dtype=dtype, device=device)
    vc = torch.ones(pages, block, 1, 64, dtype=dtype, device=device)
    kc[..., 0] = 1.0
    q = torch.zeros(portion, H, 64, dtype=dtype, device=device)
    q[..., 0] = 2.0
    sink = torch.tensor([9.0, -2.0], device=device)
    out = torch.empty(portion, H, 64, dtype=dtype, device=device)
    ops.grouped_attention(q, kc, vc, batch, 0.5, 2.0, window, keep, sink, out)
    e = math.exp(2.0 * math.tanh(0.5))
    for h in range(H):
        n = (window + keep) * e
        want = n / (n + math.exp(sink[h].item()))
        assert abs(out[-1, h].double().mean().item() - want) < (5e-3 if dtype == BF16 else 1e-5)


def test_cache_keys_values(device, dtype):
    N, G, d, e, block = 7, 3, 64, 128, 8
    wide = rand(N, G * (d + e) + 64, dtype=dtype, device=device)
    k = wide.as_strided((N, G, d), (wide.shape[1], d, 1))
    v = wide.as_strided((N, G, e), (wide.shape[1], e, 1), G * d)
    kc = torch.zeros(4, block, G, d, dtype=dtype, device=device)
    vc = torch.zeros(4, block, G, e, dtype=dtype, device=device)
    slots = torch.tensor([31, 0, 8, 7, 15, 16, 30], device=device)
    ops.cache_keys_values(k, v, slots, kc, vc)
    assert torch.equal(kc.view(-1, G, d)[slots], k) and torch.equal(vc.view(-1, G, e)[slots], v)
    rest = [i for i in range(32) if i not in slots.tolist()]
    assert not kc.view(-1, G, d)[rest].any() and not vc.view(-1, G, e)[rest].any()


# ------------------------------------------------------------------ delta rule


class DeltaCase:
    """Inputs of several sequences and a step function over portions of them."""

    options = {}  # of the op

    def __init__(self, H, G, D, V, taps, lens, dtype, device, seed=0, slots=None):
        self.shape = H, G, D, V, taps
        self.dtype, self.device, self.lens = dtype, device, lens
        self.C = 2 * G * D + H * V
        r = lambda *s, k, scale=1.0, dt=dtype: rand(  # noqa: E731
            *s, dtype=dt, device="cpu", seed=seed * 100 + k, scale=scale)
        n = sum(lens)
        self.start = [sum(lens[:i]) for i in range(len(lens))]
        self.qkv, self.b = r(n, self.C, k=1), r(n, H, k=2)
        self.z, self.gate = r(n, H * D, k=3, scale=2.0), r(n, H * V, k=4)
        self.conv = r(self.C, taps, k=5, scale=0.6)
        self.A_log = torch.linspace(-4, 1.5, H)      # slow and fast heads
        self.dt_bias, self.norm = r(H * D, k=6, dt=F32) - 2, 1 + r(V, k=7, dt=F32) * 0.3
        self.eps, self.unit_eps = 1e-3, 1e-6
        # what no sequence has written is NaN: a first token that reads it shows
        num = (max(slots) if slots else len(lens)) + 2
        self.state = torch.full((num, H, D, V), float("nan"), device=device)
        self.ring = torch.full((num, taps, self.C), float("nan"), dtype=dtype, device=device)
        self.slots = slots or list(range(len(lens), 0, -1))
        self.at = [0] * len(lens)

    def step(self, portions):
        """[(sequence, tokens)] -> their rows, in order; single tokens after the
        first run as decode rows."""
        chunks = [(s, n) for s, n in portions if n > 1 or self.at[s] == 0]
        single = [(s, n) for s, n in portions if (s, n) not in chunks]
        rows, prefills, lens = [], [], []
        for s, n in chunks + single:
            lo = self.start[s] + self.at[s]
            rows += range(lo, lo + n)
            if (s, n) in chunks:
                prefills.append(SeqMeta(s, n, self.at[s] + n, self.at[s], [0], True, self.slots[s]))
            else:
                lens.append(self.at[s] + 1)
            self.at[s] += n
        t = lambda x, dt: torch.tensor(x, dtype=dt, device=self.device)  # noqa: E731
        batch = FlatBatch(
            token_ids=t([0] * len(rows), torch.long), positions=t([0], torch.long),
            slot_mapping=t([0], torch.long), prefills=prefills,
            num_prefill_tokens=sum(m.query_len for m in prefills),
            decode_seq_ids=[s for s, _ in single],
            decode_block_tables=None,
            decode_seq_lens=t(lens, torch.long) if lens else None,
            logit_rows=t([0], torch.long), sample_seq_ids=[],
            decode_state_slots=t([self.slots[s] for s, _ in single], torch.int32) if lens else None,
        )
        H, G, D, V, taps = self.shape
        dev = lambda x: x[rows].to(self.device)  # noqa: E731
        # sections of one wide projection, as the model passes them
        pad = -(-self.C // 16) * 16
        wide = torch.zeros(len(rows), pad + 16 * -(-H // 16), dtype=self.dtype, device=self.device)
        wide[:, : self.C], wide[:, pad : pad + H] = dev(self.qkv), dev(self.b)
        out = ops.gated_delta(
            wide[:, : self.C], self.conv.to(self.device), wide[:, pad : pad + H], dev(self.z),
            self.A_log.to(self.device), self.dt_bias.to(self.device), dev(self.gate),
            self.norm.to(self.device), self.eps, self.unit_eps, G, self.state, self.ring, batch,
            **self.options,
        ).cpu()
        at, got = 0, {}
        for s, n in chunks + single:
            got[s] = out[at : at + n]
            at += n
        return [got[s] for s, _ in portions]

    def want(self, s):
        """The whole sequence by the oracle, and its final state."""
        H, G, D, V, taps = self.shape
        T = self.lens[s]
        r = slice(self.start[s], self.start[s] + T)
        y = oracle.short_conv(self.qkv[r].double(), self.conv.double())
        q, k, v = y.split([G * D, G * D, H * V], 1)
        q = oracle.unit(q.view(T, G, D)) * D ** -0.5
        k, v = oracle.unit(k.view(T, G, D)), v.view(T, H, V)
        g = oracle.decay((self.z[r].double() + self.dt_bias.double()).view(T, H, D),
                         self.A_log.double())
        beta = torch.sigmoid(self.b[r].double())
        o = torch.stack([
            oracle.delta_rule(q[:, n // (H // G)], k[:, n // (H // G)], v[:, n], g[:, n], beta[:, n])
            for n in range(H)
        ], 1)
        o = oracle.rms(o, self.eps) * self.norm.double()
        return o.view(T, H * V) * torch.sigmoid(self.gate[r].double())


DELTA = [
    # heads, key heads, dim, vdim, taps
    (4, 2, 12, 18, 3),
    (6, 3, 32, 32, 4),
    (2, 2, 128, 128, 4),
    (3, 1, 20, 7, 1),
    (4, 4, 64, 96, 4),
    (2, 1, 256, 64, 2),
    (1, 1, 300, 40, 4),
    (2, 2, 16, 260, 5),
    (1, 1, 1, 1, 2),
    (1, 1, 600, 8, 4),
    (1, 1, 260, 512, 4),
    (3, 3, 33, 12, 4),
]


@pytest.mark.parametrize("H,G,D,V,taps", DELTA)
def test_delta_rule_in_portions(device, dtype, H, G, D, V, taps):
    """Sequences of other lengths side by side, whole, in portions that are shorter
    and longer than the convolution and the kernels' token tiles, and token by token."""
    lens = [45, 1, 2, 35]
    case = DeltaCase(H, G, D, V, taps, lens, dtype, device)
    plan = [[(0, 17), (3, 35)], [(1, 1), (0, 1)], [(0, 2), (2, 2)], [(0, 1)], [(0, 16)],
            [(0, 3)], [(0, 1)], [(0, 1)], [(0, 3)]]
    got = {s: [] for s in range(len(lens))}
    for portions in plan:
        for (s, _), rows in zip(portions, case.step(portions)):
            got[s].append(rows)
    for s in got:
        close(torch.cat(got[s]), case.want(s), dtype)


def test_delta_single_tokens(device, dtype):
    """Token by token from the first one, several sequences at once."""
    case = DeltaCase(4, 2, 24, 20, 4, [30, 21, 9], dtype, device)
    got = {0: [], 1: [], 2: []}
    for t in range(30):
        portions = [(s, 1) for s in got if t < case.lens[s]]
        for (s, _), rows in zip(portions, case.step(portions)):
            got[s].append(rows)
    for s in got:
        close(torch.cat(got[s]), case.want(s), dtype)


def test_delta_slot_is_used_again(device):
    """A slot's next sequence starts from zero, whatever the last one left, and the
    slots of waiting sequences keep theirs."""
    case = DeltaCase(2, 1, 16, 16, 4, [20, 15, 24], F32, device, slots=[3, 0, 3])
    first = case.step([(0, 20), (1, 6)])
    third = case.step([(2, 2)]) + case.step([(2, 21)]) + case.step([(2, 1)])
    second = case.step([(1, 9)])
    close(first[0], case.want(0), F32)
    close(torch.cat([first[1], second[0]]), case.want(1), F32)
    close(torch.cat(third), case.want(2), F32)


def test_delta_remembers_far_keys(device, dtype):
    """With slow decays a value written once is read hundreds of tokens later by the
    same key; with fast decays it is gone."""
    T, D, V = 300, 32, 8
    case = DeltaCase(2, 1, D, V, 4, [T + 1], dtype, device)
    case.A_log = torch.tensor([-12.0, 3.0])
    case.conv.zero_()[:, -1] = 1.0
    q, k, v = case.qkv[:, :D], case.qkv[:, D : 2 * D], case.qkv[:, 2 * D :]
    k[:, 0], q[:] = -30.0, -30.0       # silu(-30) = 0: other tokens leave channel 0 alone
    q[T, 0] = k[5, 0] = 9.0
    k[5, 1:] = -30.0
    v[5], case.b[5] = 3.0, 20.0
    got = torch.cat(case.step([(0, 200)]) + case.step([(0, T - 200)]) + case.step([(0, 1)]))
    want = case.want(0)
    close(got, want, dtype)
    assert want[T, :V].abs().min() > 50 * want[T, V:].abs().max()


def test_delta_extreme_decays(device):
    """Decays of exactly one and zero: no overflow, no loss."""
    case = DeltaCase(2, 2, 16, 16, 4, [40], F32, device)
    case.z[:, ::3], case.z[:, 1::3] = 300.0, -300.0
    got = torch.cat(case.step([(0, 33)]) + case.step([(0, 1)]) + case.step([(0, 6)]))
    assert got.isfinite().all()
    close(got, case.want(0), F32)
