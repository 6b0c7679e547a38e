"""Tezinex end to end against the plain oracle: checkpoints in the design's own config
and tensor names, loaded and run by the engine's scheduler, block manager, state slots
and forward.  CPU ops unmarked, HIP kernels marked gpu."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import tezinex_oracle as oracle
from agentcontrolplane_amd.engine.config import PRESETS, EngineConfig
from agentcontrolplane_amd.engine.engine import InferenceEngine
from agentcontrolplane_amd.engine.request import InferenceRequest, SamplingParams
from agentcontrolplane_amd.engine.state import OutOfStateSlotsError, StateSlots
from agentcontrolplane_amd.engine.trace import TraceReplay
from agentcontrolplane_amd.models.configs import read_architecture, read_model_config
from agentcontrolplane_amd.models.weights import save_checkpoint
from model_helpers import CUTS, assert_close, feed, make_engine, tokens

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)


def dense(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def attn(heads, kv, dim, vdim, size, keep, scale=0.4, cap=4.0, ff=None, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
             "softcap": cap, "mask": {"size": size, "keep_first": keep}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": dense(ff)}


def delta(heads, kv, dim, vdim, conv, ff=None):
    return {"type": "channel_delta", "mlp": dense(ff),
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def config(vocab, width, layers, eps=1e-5, m=0.6, cap=20.0):
    return {"architecture": "Tezinex", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "residual_mult": m, "logit_softcap": cap, "layers": layers}


#: name -> (config, inner sizes of the decay and gate projections)
CONFIGS = {
    # odd sizes, no two layers alike, keys borrowed with another window and twice,
    # feed-forwards on some layers of either kind
    "odd": (config(311, 42, [
        attn(6, 3, 10, 14, 7, 2, ff=50),
        delta(4, 2, 6, 9, 3, ff=33),
        delta(3, 3, 20, 4, 4),
        attn(2, 1, 12, 6, 23, 0, scale=0.9, cap=1.5),
        attn(4, 1, 12, 6, 40, 5, cap=9.0, ff=61, kv_from=3),
        delta(2, 1, 5, 30, 2),
        attn(3, 3, 10, 14, 11, 1, kv_from=0),
    ], eps=0.05), (5, 7)),
    # head sizes the matrix-core kernels take unpadded
    "wide": (config(400, 96, [
        delta(4, 4, 128, 64, 4, ff=128),
        attn(8, 2, 64, 128, 64, 16, scale=0.2, ff=96),
        delta(4, 2, 64, 64, 4),
        attn(4, 2, 64, 128, 100, 3, scale=0.2, kv_from=1, ff=96),
        attn(16, 1, 128, 64, 33, 1, scale=0.2),
    ], m=1.3), (32, 16)),
    # beyond the matrix-core kernels' sizes
    "large": (config(290, 64, [
        attn(2, 1, 260, 20, 40, 4, scale=0.1, ff=64),
        delta(1, 1, 270, 24, 5),
        delta(2, 2, 24, 260, 4, ff=16),
    ], eps=1e-3), (24, 40)),
    # nothing repeated: one head, one dimension, one tap, a window of one token
    "ones": (config(270, 16, [
        attn(1, 1, 4, 1, 1, 0, ff=3),
        delta(1, 1, 1, 1, 1, ff=1),
        attn(1, 1, 4, 1, 1, 2, kv_from=0),
    ], eps=0.5, m=1.0), (1, 1)),
}


def make_weights(cfg, ranks, seed=0):
    """bf16 tensors with scores, gates and decays that vary."""
    g = torch.Generator().manual_seed(seed)
    w, V = cfg["width"], cfg["vocab"]

    def t(*shape, gain=1.0):
        return (torch.randn(*shape, generator=g) * gain * shape[-1] ** -0.5).bfloat16()

    def vec(n, mean=0.0, spread=0.3):
        return (mean + spread * torch.randn(n, generator=g)).bfloat16()

    W = {"embed": t(V, w, gain=3.0), "final.norm": vec(w)}
    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}.mix."
        H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        W[f"l{i}.norm1"], W[f"l{i}.norm1b"] = vec(w), vec(w)
        W[f"l{i}.dwa"] = vec(i + 2, spread=0.2)
        W[f"l{i}.dwa"][-1] += 0.8
        W[p + "q"], W[p + "o"] = t(G * D, w), t(w, H * E)
        if spec["type"] == "attention":
            W[p + "q"], W[p + "q.b"] = t(H * D, w, gain=1.5), vec(H * D)
            W[p + "sink"] = vec(H, spread=1.0)
            if "kv_from" not in m:
                for n, size in (("k", D), ("v", E)):
                    W[p + n], W[p + n + ".b"] = t(G * size, w, gain=1.5), vec(G * size)
        else:
            ra, rg = ranks
            W[p + "k"], W[p + "v"] = t(G * D, w), t(H * E, w)
            for n in "qkv":
                W[p + n + ".conv"] = t(W[p + n].shape[0], m["conv"], gain=1.5)
            W[p + "b"], W[p + "A_log"], W[p + "norm"] = t(H, w, gain=2.0), vec(H, -1, 1), vec(E, 1)
            W[p + "a1"], W[p + "a2"] = t(ra, w), t(H * D, ra, gain=2.0)
            W[p + "g1"], W[p + "g2"] = t(rg, w), t(H * E, rg, gain=2.0)
            W[p + "dt_bias"] = vec(H * D, -2, 1)
        if spec["mlp"]:
            ff = spec["mlp"]["ff"]
            W[f"l{i}.norm2"], W[f"l{i}.norm2b"] = vec(w), vec(w)
            W[f"l{i}.mlp.gate"], W[f"l{i}.mlp.up"] = t(ff, w), t(ff, w)
            W[f"l{i}.mlp.down"] = t(w, ff)
    return W


def write_checkpoint(path, cfg, W):
    save_file(W, str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return str(path)


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
    """name -> (folder, config, float64 weights)"""
    out = {}
    for n, (name, (cfg, ranks)) in enumerate(CONFIGS.items()):
        W = make_weights(cfg, ranks, seed=n)
        path = write_checkpoint(tmp_path_factory.mktemp(name), cfg, W)
        out[name] = (path, cfg, {k: v.double() for k, v in W.items()})
    return out


@pytest.fixture(params=["cpu", GPU])
def device(request):
    if request.param == "cuda" and not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    return request.param


# ------------------------------------------------------------------ config


def test_config_reader(checkpoints):
    path, d, W = checkpoints["odd"]
    cfg = read_model_config(path)
    assert read_architecture(path) == cfg.architecture == "Tezinex"
    assert (cfg.vocab_size, cfg.hidden_size, cfg.rms_eps) == (311, 42, 0.05)
    assert (cfg.residual_mult, cfg.logit_softcap) == (0.6, 20.0)
    a, b, c = (cfg.layers[i].mixer for i in (0, 1, 4))
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.softcap, a.kv_from) == (
        6, 3, 10, 14, 7, 2, 4.0, None)
    assert (b.heads, b.kv_heads, b.dim, b.vdim, b.conv, b.decay_rank, b.gate_rank) == (
        4, 2, 6, 9, 3, 5, 7)
    assert (c.kv_from, c.window, c.keep_first) == (3, 40, 5)
    assert cfg.layers[2].mlp is None and cfg.layers[1].mlp.width == 33
    assert cfg.params_bytes(1) == sum(v.numel() for v in W.values())


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="attention_9"),
    lambda d: d["layers"][0]["mlp"].update(kind="experts"),
    lambda d: d["layers"][4]["mixer"].update(kv_from=1),   # a delta layer
    lambda d: d["layers"][4]["mixer"].update(kv_from=5),   # a later layer
    lambda d: d["layers"][6]["mixer"].update(kv_from=4),   # a borrower
    lambda d: d["layers"][4]["mixer"].update(dim=13),
    lambda d: d["layers"][1]["mixer"].update(kv_heads=3),
    lambda d: d.update(architecture="Other"),
])
def test_config_reader_refuses(checkpoints, tmp_path, change):
    path, cfg, W = checkpoints["odd"]
    d = json.loads(json.dumps(cfg))
    change(d)
    write_checkpoint(tmp_path, d, {k: v.bfloat16() for k, v in W.items()})
    with pytest.raises(ValueError):
        read_model_config(str(tmp_path))


@pytest.mark.parametrize("name", ["l1.mix.a2", "l0.mix.k.b", "l3.dwa"])
def test_loader_refuses_wrong_shape(checkpoints, tmp_path, name):
    _, cfg, W = checkpoints["odd"]
    W = {k: v.bfloat16() for k, v in W.items()}
    W[name] = W[name][:-1].contiguous()
    with pytest.raises(ValueError, match=name):
        make_engine(write_checkpoint(tmp_path, cfg, W), "cpu")


def test_checkpoint_round_trip(checkpoints, tmp_path):
    """Export undoes the padded, fused layout exactly."""
    for name, (path, cfg, W) in checkpoints.items():
        m = make_engine(path, "cpu").model
        out = m.named_tensors()
        assert out.keys() == W.keys()
        for k in W:
            assert torch.equal(out[k].double(), W[k]), (name, k)
    save_checkpoint(m, str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    again = make_engine(str(tmp_path), "cpu").model.named_tensors()
    assert all(torch.equal(again[k], out[k]) for k in out)


# ------------------------------------------------------------------ forward


@pytest.mark.parametrize("name", CONFIGS)
def test_stream_after_every_layer(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    eng = make_engine(path, device)
    ids = tokens(37, cfg)
    want, got = [], []
    oracle.forward(cfg, W, ids, want)
    plain = eng.model.forward
    eng.model.forward = lambda batch: plain(batch, got)
    feed(TraceReplay(eng), "a", ids, [len(ids)])
    assert len(got) == len(want) == len(cfg["layers"])
    for g, w in zip(got, want):
        assert (g.double().cpu() - w).abs().max() < 5e-5 * w.abs().max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("name", CONFIGS)
def test_portions(checkpoints, device, name, cuts, dtype):
    """However the prompt is cut, decoded tail included, the logits are the whole
    sequence's: windows of 1 to 100, kept tokens and pages of 16 pass by."""
    if name == "ones" and dtype == "bfloat16":
        pytest.skip("a width of 16 leaves bf16 no room")
    path, cfg, W = checkpoints[name]
    ids = tokens(150, cfg)
    replay = TraceReplay(make_engine(path, device, dtype))
    got = feed(replay, "a", ids, CUTS[cuts](len(ids)))
    assert_close(got, oracle.forward(cfg, W, ids), dtype)
    eng = replay.engine
    assert eng.bm.free_blocks == eng.bm.num_blocks and eng.states.free == eng.states.num_slots


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_mixed_batches_and_reused_storage(checkpoints, device, name, dtype):
    """Portions of some requests beside single tokens of others, requests that pause,
    end and come back, with pages and state slots too few for all of them at once."""
    path, cfg, W = checkpoints[name]
    lens = {"a": 130, "b": 3, "c": 77, "d": 1, "e": 64, "f": 90, "g": 2, "h": 40}
    ids = {r: tokens(n, cfg, seed=ord(r)) for r, n in lens.items()}
    want = {r: oracle.forward(cfg, W, ids[r]) for r in ids}
    replay = TraceReplay(make_engine(path, device, dtype, num_kv_blocks=19, max_batch_size=3))
    eng = replay.engine
    assert eng.states.num_slots == 3
    for t in eng.model.states + eng.model.caches:
        t.fill_(float("nan"))  # what was never written must not be read
    g = torch.Generator().manual_seed(7)
    sizes = [1, 1, 2, 30, 5, 17, 1, 64]
    at, queue, live, seen = {r: 0 for r in ids}, list(lens), [], set()
    for _ in range(400):
        def held(rs):
            return sum(-(-lens[r] // 16) for r in rs)
        while queue and len(live) < 3 and held(live + queue[:1]) <= 19:
            live.append(queue.pop(0))
        if not live:
            break
        picked = [r for r in live if torch.rand(1, generator=g) < 0.7] or live[:1]
        entries, end = [], []
        for r in picked:
            n = sizes[int(torch.randint(0, len(sizes), (1,), generator=g))]
            part = ids[r][at[r] : at[r] + n]
            entries.append({"id": r, "tokens": part, "want": list(range(len(part)))})
            if at[r] + len(part) == lens[r]:
                end.append(r)
        got = replay.step(entries, end)
        row = 0
        for e in entries:
            n, r = len(e["tokens"]), e["id"]
            assert_close(got[row : row + n], want[r][at[r] : at[r] + n], dtype)
            row += n
            at[r] += n
        for r in end:
            live.remove(r)
            seen.add(r)
    assert seen == set(ids)
    assert eng.bm.free_blocks == 19 and eng.states.free == 3


def test_first_tokens(checkpoints, device):
    for name, (path, cfg, W) in checkpoints.items():
        replay = TraceReplay(make_engine(path, device))
        for n in (1, 2, 3):
            ids = tokens(n, cfg, seed=n)
            got = feed(replay, f"{name}{n}", ids, [1] * n)
            assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("decode", [False, True])
def test_window_edges_through_the_model(tmp_path, device, decode):
    """One attention layer, a window of 9 that keeps 2: changing a token moves the
    logits of the 8 tokens after it, of every later one if it is kept, of no other."""
    cfg = config(280, 32, [attn(2, 1, 8, 8, 9, 2, ff=24)])
    path = write_checkpoint(tmp_path, cfg, make_weights(cfg, (4, 4), seed=5))
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(60, cfg)
    cuts = [14] + [1] * 46 if decode else [60]
    base = feed(replay, "a", ids, cuts)
    for j in (0, 1, 2, 15, 16, 40):  # the kept tokens, a page's last and first
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-5
        reach = 60 if j < 2 else j + 9
        assert moved[j : min(reach, j + 9)].all() and not moved[:j].any(), j
        assert moved[j + 9 : reach].float().mean() > 0.9 if j < 2 else not moved[reach:].any(), j


@pytest.mark.parametrize("decode", [False, True])
def test_borrowed_keys_have_their_own_window(tmp_path, device, decode):
    """The borrower sees further back than the layer whose keys it uses: a far token
    reaches the logits through it, over keys the owner's own window has left."""
    cfg = config(280, 32, [attn(2, 1, 8, 8, 3, 0), attn(2, 1, 8, 8, 30, 0, kv_from=0)])
    W = make_weights(cfg, (4, 4), seed=6)
    path = write_checkpoint(tmp_path, cfg, W)
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(70, cfg)
    cuts = [14] + [1] * 56 if decode else [70]
    base = feed(replay, "a", ids, cuts)
    other = list(ids)
    other[20] = (other[20] + 1) % 280
    moved = (feed(replay, "b", other, cuts) - base).abs().amax(-1) > 1e-5
    # the keys are made of what enters layer 0: a token reaches exactly its window
    assert moved[20:50].all() and not moved[50:].any() and not moved[:20].any()
    assert_close(base, oracle.forward(cfg, {k: v.double() for k, v in W.items()}, ids))


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    ids = tokens(400, cfg, seed=3)
    got = feed(TraceReplay(make_engine(path, device)), "a", ids, [5] + [1] * 395)
    assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replay_matches_eager(checkpoints, dtype):
    """Decode-only steps replay a captured graph; every replay, with other work in
    between, matches the eager step.  Padding rows leave the real states alone."""
    path, cfg, _ = checkpoints["wide"]
    runs = []
    for eager in (False, True):
        eng = make_engine(path, "cuda", dtype, enforce_eager=eager)
        replay, rows = TraceReplay(eng), []
        ids = {r: tokens(90, cfg, seed=ord(r)) for r in "abc"}
        replay.step([{"id": r, "tokens": ids[r][: 20 + 9 * k], "want": []}
                     for k, r in enumerate("abc")], [])
        for s in range(30):
            who = "abc" if s % 4 else "ab"  # other batch sizes in the same bucket
            rows.append(replay.step(
                [{"id": r, "tokens": [ids[r][60 + s]], "want": [0]} for r in who], []))
            torch.cuda.synchronize()
        assert bool(eng._m.get("graph_steps")) != eager
        runs.append(torch.cat(rows))
    assert (runs[0] - runs[1]).abs().max() <= 1e-3 * runs[1].abs().max()


# -------------------------------------------------------------- state slots


def test_state_slots():
    s = StateSlots(2)
    a, b = s.acquire(7), s.acquire(8)
    assert {a, b} == {0, 1} and s.free == 0
    with pytest.raises(OutOfStateSlotsError):
        s.acquire(9)
    with pytest.raises(KeyError):
        s.acquire(7)
    s.transfer(9, 7)
    assert s.slot(9) == a and not s.has(7)
    s.release(9)
    s.release(9)  # once is enough
    assert s.free == 1 and s.acquire(10) == a


def test_slots_are_a_hard_limit(checkpoints):
    path, cfg, _ = checkpoints["odd"]
    replay = TraceReplay(make_engine(path, "cpu", num_state_slots=1))
    replay.step([{"id": "a", "tokens": [1, 2], "want": []}], [])
    with pytest.raises(OutOfStateSlotsError):
        replay.step([{"id": "b", "tokens": [1], "want": []}], [])


# --------------------------------------------------------------- generation


def greedy(cfg, W, prompt, n, live):
    ids, out = list(prompt), []
    for _ in range(n):
        tok = int(oracle.forward(cfg, W, ids)[-1, :live].argmax())
        if tok == 259:  # end of turn
            break
        ids.append(tok)
        out.append(tok)
    return out


@pytest.mark.parametrize("pool,slots", [(96, 8), (9, 8), (96, 2)])
def test_greedy_generation_through_the_engine(checkpoints, device, pool, slots):
    """engine.submit: chunked prefill, continuous batching, the sampler, reuse of pages
    and states across turns; a small pool preempts, few slots make requests wait."""
    path, cfg, W = checkpoints["odd"]
    eng = make_engine(path, device, start=True, num_kv_blocks=pool, num_state_slots=slots,
                      max_prefill_tokens=24)
    try:
        prompts = [tokens(n, cfg, seed=n) for n in (5, 41, 60, 17)]
        turns = [[], []]
        for group in (0, 1):
            reqs = [
                eng.submit(InferenceRequest(list(p), SamplingParams(max_tokens=14, temperature=0.0)))
                for p in prompts
            ]
            for p, r in zip(prompts, reqs):
                out = r.wait(120)
                assert out == greedy(cfg, W, p, 14, 261)
                turns[group].append(list(p) + out)
            # the next turns: what was said, and some more; one prompt once more
            prompts = [t + tokens(5, cfg, seed=99) for t in turns[0][1:]] + [prompts[2]]
        if pool == 9:
            assert eng.metrics()["preemptions"] >= 1
        elif slots == 8:
            assert eng.metrics()["continuation_hits"] >= 2
        held = len(eng.scheduler.retired)
        assert eng.states.free == slots - held
    finally:
        eng.stop()


def test_a_turn_goes_on_from_the_retired_state(checkpoints):
    """The state is taken over with the pages only when the new prompt begins with
    every token it covers."""
    path, cfg, W = checkpoints["wide"]
    eng = make_engine(path, "cpu")
    sched = eng.scheduler

    def turn(prompt, n):
        req = InferenceRequest(list(prompt), SamplingParams(max_tokens=n, temperature=0.0))
        sched.add_request(req)
        while not req._event.is_set():
            eng.step()
        return req.output_ids

    def hits():
        return sched.continuation_hits

    first = tokens(37, cfg, seed=1)
    out = turn(first, 6)
    assert len(sched.retired) == 1
    # the same beginning, but not all of what the state has seen
    fork = first[:30] + tokens(9, cfg, seed=2)
    assert turn(fork, 3) == greedy(cfg, W, fork, 3, 261) and hits() == 0
    more = first + out + tokens(11, cfg, seed=3)
    again = turn(more, 5)
    assert again == greedy(cfg, W, more, 5, 261) and hits() == 1
    assert sched.continuation_tokens_saved == len(first) + len(out) - 1
    # taken over means gone: the first turn's state cannot be used twice
    assert turn(more, 5) == again and hits() == 1


def test_presets_and_random_init(device):
    cfg = EngineConfig(model="tiny-tezinex", device=device, num_kv_blocks=64, max_batch_size=8)
    eng = InferenceEngine(cfg)
    try:
        res = eng.chat([{"role": "user", "content": "hello"}],
                       sampling=SamplingParams(max_tokens=6, temperature=0.8))
        assert res.completion_tokens <= 6 and res.finish_reason in ("stop", "length")
    finally:
        eng.stop()
    assert PRESETS["tezinex-8b"].params_bytes() > 10e9
    owners = [x.mixer.kv_from for x in PRESETS["tezinex-8b"].layers if hasattr(x.mixer, "kv_from")]
    assert owners == [None, 3, None, 11, None, 19, None, 27]


# ---------------------------------------------------------- tensor parallel

SHARDED = config(300, 32, [
    delta(4, 2, 8, 6, 4, ff=26),
    attn(4, 2, 8, 6, 11, 2, ff=40),
    delta(2, 2, 6, 10, 3),
    attn(2, 2, 8, 6, 20, 0, kv_from=1),
], eps=1e-2)


def _tp_worker(rank, path, prompt, q):
    try:
        os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT="29547")
        import torch.distributed as dist

        from agentcontrolplane_amd.parallel.tp import run_tp_worker

        torch.set_num_threads(2)
        dist.init_process_group("gloo", rank=rank, world_size=2)
        eng = make_engine(path, "cpu", start=rank == 0, tensor_parallel=2, max_prefill_tokens=16)
        if rank:
            run_tp_worker(eng)
            q.put((rank, [x.mixer.heads for x in eng.model.layers]))
        else:
            outs = [eng.generate(p, SamplingParams(max_tokens=12, temperature=0.0),
                                 timeout=120).output_ids for p in (prompt, prompt[3:])]
            eng.stop()
            q.put((rank, outs))
    except Exception as e:  # pragma: no cover
        import traceback

        q.put((rank, f"{e}\n{traceback.format_exc()}"))


def test_tensor_parallel_generation(tmp_path):
    """Two ranks, each with its heads and feed-forward columns: one model."""
    import torch.multiprocessing as mp

    W = make_weights(SHARDED, (4, 6), seed=4)
    path = write_checkpoint(tmp_path, SHARDED, W)
    prompt = tokens(21, SHARDED)
    W = {k: v.double() for k, v in W.items()}
    want = [greedy(SHARDED, W, p, 12, 261) for p in (prompt, prompt[3:])]
    ctx = mp.get_context("spawn")
    q = ctx.Queue()
    procs = [ctx.Process(target=_tp_worker, args=(r, path, prompt, q)) for r in (0, 1)]
    for p in procs:
        p.start()
    got = dict(q.get(timeout=180) for _ in procs)
    for p in procs:
        p.join(timeout=30)
    assert got[0] == want and got[1] == [2, 2, 1, 1], got


# -------------------------------------------------- command line, trace runner


def test_serve_takes_the_checkpoint_configuration(checkpoints):
    from argparse import Namespace

    from agentcontrolplane_amd.__main__ import _engine_config

    args = Namespace(model=None, checkpoint=checkpoints["wide"][0], dtype="float32", kv_blocks=64)
    cfg = _engine_config(args, "cpu").model_config()
    assert cfg.architecture == "Tezinex" and cfg.dtype == "float32" and cfg.vocab_size == 400


def test_trace_run_program(checkpoints, device, tmp_path):
    path, cfg, W = checkpoints["odd"]
    a, b = tokens(20, cfg, 1), tokens(9, cfg, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:13], "want": [12, 0]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]},
                                {"id": "a", "tokens": a[13:], "want": [6, 2]}], "end": ["a"]},
        {"step": 7, "entries": [{"id": "a", "tokens": b, "want": [8]}], "end": ["a", "b"]},
    ]
    r = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype",
         "float32", "--out", str(tmp_path / "out"), "--max-tokens", "128", "--device", device],
        input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
        timeout=240,
    )
    assert r.returncode == 0, r.stderr[-2000:]
    done = [x for x in r.stdout.splitlines() if x.startswith("done")]
    assert done == ["done 0", "done 1", "done 2", "done 7"]
    la, lb = oracle.forward(cfg, W, a), oracle.forward(cfg, W, b)
    for step, want in ((0, la[[12, 0]]), (2, torch.stack([lb[8], la[19], la[15]])), (7, lb[[8]])):
        got = np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(-1, 311)
        assert_close(torch.from_numpy(got), want)
    assert not (tmp_path / "out" / "1.f32").exists()
