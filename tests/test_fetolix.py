"""Fetolix end to end against the plain oracle: checkpoints in the design's own
config and tensor names, loaded and run by the engine's scheduler, block manager
and forward.  CPU ops unmarked, HIP kernels marked gpu."""
import dataclasses
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import fetolix_oracle as oracle
from agentcontrolplane_amd.engine.config import PRESETS, EngineConfig
from agentcontrolplane_amd.engine.engine import InferenceEngine
from agentcontrolplane_amd.engine.kv import OutOfBlocksError
from agentcontrolplane_amd.engine.request import InferenceRequest, SamplingParams
from agentcontrolplane_amd.engine.trace import TraceReplay
from agentcontrolplane_amd.models import create_model
from agentcontrolplane_amd.models.configs import read_architecture, read_model_config
from agentcontrolplane_amd.models.weights import save_checkpoint
from model_helpers import CUTS, assert_close, feed, make_engine, tokens

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)


def layer(kind, *, heads, dim, rot, vdim, rank, base, scale=0.4, q_rank=None, window=None,
          ff=None, limit=1.0):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
             "rot": {"base": base, "dims": rot}, "scale": scale}
    if kind == "latent_attention":
        mixer |= {"q_rank": q_rank, "mask": {"size": window}}
    return {"type": kind, "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def win(**kw):
    return layer("latent_attention", **kw)


def full(**kw):
    return layer("latent_attention_2", **kw)


CONFIGS = {
    # odd sizes, no two layers alike, a layer without feed-forward, layers
    # before and after the loop
    "odd": {
        "architecture": "Fetolix", "vocab": 311, "width": 42, "norm": {"eps": 0.05},
        "layers": [
            win(heads=3, dim=10, rot=6, vdim=14, rank=20, base=1e4, q_rank=18, window=7, ff=50),
            full(heads=5, dim=8, rot=12, vdim=6, rank=36, base=500.0, scale=0.9),
            win(heads=1, dim=20, rot=2, vdim=9, rank=11, base=37.0, q_rank=40, window=23,
                ff=33, limit=0.4),
            full(heads=2, dim=6, rot=4, vdim=16, rank=70, base=1e6, ff=61, limit=9.0),
        ],
        "loop": {"start": 1, "stop": 3, "times": 3}, "token_side": {"dim": 5},
    },
    # sizes the matrix-core kernels take unpadded, two head groups
    "wide": {
        "architecture": "Fetolix", "vocab": 400, "width": 96, "norm": {"eps": 1e-6},
        "layers": [
            full(heads=20, dim=64, rot=64, vdim=64, rank=128, base=1e4, scale=0.2, ff=128),
            win(heads=20, dim=128, rot=32, vdim=64, rank=64, base=2e5, q_rank=64, window=64,
                scale=0.2, ff=96),
        ],
        "loop": {"start": 0, "stop": 2, "times": 2}, "token_side": {"dim": 16},
    },
    # beyond the matrix-core kernels' sizes
    "large": {
        "architecture": "Fetolix", "vocab": 290, "width": 64, "norm": {"eps": 1e-3},
        "layers": [
            full(heads=2, dim=130, rot=80, vdim=20, rank=40, base=1e4, scale=0.1, ff=64),
            win(heads=3, dim=24, rot=16, vdim=260, rank=530, base=1e5, q_rank=24, window=40,
                scale=0.2, ff=16),
        ],
        "loop": {"start": 0, "stop": 1, "times": 2}, "token_side": {"dim": 3},
    },
    # nothing repeated: a loop of one pass, a window of one token, one head
    "ones": {
        "architecture": "Fetolix", "vocab": 270, "width": 16, "norm": {"eps": 0.5},
        "layers": [
            full(heads=1, dim=1, rot=2, vdim=1, rank=1, base=10.0, ff=1, limit=0.1),
            win(heads=1, dim=4, rot=2, vdim=4, rank=4, base=10.0, q_rank=1, window=1, ff=3),
        ],
        "loop": {"start": 1, "stop": 2, "times": 1}, "token_side": {"dim": 1},
    },
}


def make_weights(cfg, seed=0):
    """bf16 tensors with scores and gates that vary (not all near zero)."""
    g = torch.Generator().manual_seed(seed)
    w, V, side = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"]

    def t(*shape, gain=1.0):
        return (torch.randn(*shape, generator=g) * gain * shape[-1] ** -0.5).bfloat16()

    def norm(n):
        return (1 + 0.3 * torch.randn(n, generator=g)).bfloat16()

    W = {"embed": t(V, w, gain=3.0), "final.norm": norm(w), "loop.in": t(w, 2 * w),
         "side.embed": t(V, len(cfg["layers"]) * side, gain=2.0)}
    for i, spec in enumerate(cfg["layers"]):
        m, p = spec["mixer"], f"l{i}."
        H, qk = m["heads"], m["heads"] * (m["dim"] + m["rot_dim"])
        W[p + "norm1"] = norm(w)
        if "q_rank" in m:
            W[p + "mix.dq"], W[p + "mix.dq.norm"] = t(m["q_rank"], w), norm(m["q_rank"])
            W[p + "mix.uq"] = t(qk, m["q_rank"])
        else:
            W[p + "mix.q"] = t(qk, w)
        W[p + "mix.dkv"] = t(m["kv_rank"] + m["rot_dim"], w)
        W[p + "mix.dkv.norm"] = norm(m["kv_rank"])
        W[p + "mix.uk"] = t(H * m["dim"], m["kv_rank"])
        W[p + "mix.uv"] = t(H * m["vdim"], m["kv_rank"])
        W[p + "mix.g"] = t(H, w, gain=2.0)
        W[p + "mix.o"] = t(w, H * m["vdim"], gain=0.6)
        if spec["mlp"]:
            ff = spec["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"] = t(ff, w), t(ff, w)
            W[p + "mlp.down"] = t(w, ff, gain=0.6)
        W[p + "side.gate"], W[p + "side.proj"] = t(side, w), t(w, side)
        W[p + "side.norm"] = norm(w)
    return W


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
    """name -> (folder, config, float64 weights)"""
    out = {}
    for n, (name, cfg) in enumerate(CONFIGS.items()):
        path = tmp_path_factory.mktemp(name)
        W = make_weights(cfg, seed=n)
        save_file(W, str(path / "model.safetensors"))
        (path / "config.json").write_text(json.dumps(cfg))
        out[name] = (str(path), cfg, {k: v.double() for k, v in W.items()})
    return out


@pytest.fixture(params=["cpu", GPU])
def device(request):
    if request.param == "cuda" and not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    return request.param


# ------------------------------------------------------------------ config


def test_config_reader(checkpoints):
    path, d, _ = checkpoints["odd"]
    cfg = read_model_config(path)
    assert read_architecture(path) == cfg.architecture == "Fetolix"
    assert (cfg.vocab_size, cfg.hidden_size, cfg.rms_eps) == (311, 42, 0.05)
    assert [i for i, _ in cfg.layer_runs] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [e for _, e in cfg.layer_runs] == [False, True, False, True, False, True, False, False]
    m = cfg.layers[0].mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.q_rank, m.window) == (
        3, 10, 6, 14, 20, 18, 7)
    full_m = cfg.layers[1].mixer
    assert full_m.window is None and full_m.q_rank is None and cfg.layers[1].mlp is None
    assert cfg.layers[2].mlp.limit == 0.4 and full_m.scale == 0.9 and full_m.rope_base == 500.0
    n = sum(v.numel() for v in make_weights(d).values())
    assert cfg.params_bytes(1) == n


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="attention_9"),
    lambda d: d["layers"][0]["mlp"].update(kind="experts"),
    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=4),
    lambda d: d.update(architecture="Other"),
])
def test_config_reader_refuses(tmp_path, change):
    d = json.loads(json.dumps(CONFIGS["odd"]))
    change(d)
    (tmp_path / "config.json").write_text(json.dumps(d))
    with pytest.raises(ValueError):
        read_model_config(str(tmp_path))


def test_loader_refuses_wrong_shape(checkpoints, tmp_path):
    _, cfg, _ = checkpoints["odd"]
    W = make_weights(cfg)
    W["l0.mix.uk"] = W["l0.mix.uk"][:-1].contiguous()
    save_file(W, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match="l0.mix.uk"):
        make_engine(str(tmp_path), "cpu")


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


def test_model_without_loop_or_side(tmp_path):
    """Both are parameters of the model class, not of this one design."""
    base = dataclasses.replace(PRESETS["tiny-fetolix"], loop=None, token_side_dim=0)
    m = create_model(base, EngineConfig(model="tiny-fetolix", device="cpu"), "cpu")
    m.random_init(0)
    assert not any("side" in k or "loop" in k for k in m.named_tensors())
    assert [i for i, _ in base.layer_runs] == [0, 1, 2, 3]


# ------------------------------------------------------------------ forward


@pytest.mark.parametrize("name", CONFIGS)
def test_residual_after_every_layer_run(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    eng = make_engine(path, device)
    ids = tokens(37, cfg)
    want = []
    oracle.forward(cfg, W, ids, want)
    got = []
    plain = eng.model.forward
    eng.model.forward = lambda batch: plain(batch, got)
    feed(TraceReplay(eng), "a", ids, [len(ids)])
    assert len(got) == len(want) == len(oracle.layer_order(cfg))
    for g, w in zip(got, want):
        assert (g.double().cpu() - w).abs().max() < 5e-5 * w.abs().max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("name", CONFIGS)
def test_portions(checkpoints, device, name, cuts, dtype):
    """However the prompt is cut, decoded tail included, the logits are the
    whole sequence's: windows of 1, 7, 23 and 64 and pages of 16 pass by."""
    if name == "ones" and dtype == "bfloat16":
        pytest.skip("a width of 16 leaves bf16 no room")
    path, cfg, W = checkpoints[name]
    ids = tokens(150, cfg)
    replay = TraceReplay(make_engine(path, device, dtype))
    got = feed(replay, "a", ids, CUTS[cuts](len(ids)))
    assert_close(got, oracle.forward(cfg, W, ids), dtype)
    assert replay.engine.bm.free_blocks == replay.engine.bm.num_blocks


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_mixed_batches_and_reused_pages(checkpoints, device, name, dtype):
    """Portions of some requests beside single tokens of others, requests that
    pause, end and come back, in a pool too small for all of them at once."""
    path, cfg, W = checkpoints[name]
    lens = {"a": 130, "b": 3, "c": 77, "d": 1, "e": 64, "f": 90}
    ids = {r: tokens(n, cfg, seed=ord(r)) for r, n in lens.items()}
    want = {r: oracle.forward(cfg, W, ids[r]) for r in ids}
    # 4 live at most; 19 pages hold a + c + e, not everything that ever ran
    replay = TraceReplay(make_engine(path, device, dtype, num_kv_blocks=19, max_batch_size=4))
    g = torch.Generator().manual_seed(7)
    sizes = [1, 1, 2, 30, 5, 17, 1, 64]
    at, queue, live, seen = {r: 0 for r in ids}, list("abcdef"), [], set()
    for _ in range(400):
        def held(rs):
            return sum(-(-lens[r] // 16) for r in rs)
        while queue and len(live) < 4 and held(live + queue[:1]) <= 19:
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
    assert replay.engine.bm.free_blocks == 19


def test_pool_is_a_hard_limit(checkpoints):
    path, cfg, _ = checkpoints["odd"]
    replay = TraceReplay(make_engine(path, "cpu", num_kv_blocks=4, max_batch_size=1))
    feed(replay, "a", tokens(60, cfg), [60], end=False)
    with pytest.raises((OutOfBlocksError, RuntimeError), match="blocks"):
        replay.step([{"id": "a", "tokens": [1] * 5, "want": []}], [])
    with pytest.raises(RuntimeError, match="live"):
        replay.step([{"id": "b", "tokens": [1], "want": []}], [])


def test_first_tokens(checkpoints, device):
    for name, (path, cfg, W) in checkpoints.items():
        replay = TraceReplay(make_engine(path, device))
        for n in (1, 2, 3):
            ids = tokens(n, cfg, seed=n)
            got = feed(replay, f"{name}{n}", ids, [1] * n)
            assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("decode", [False, True])
def test_window_edge_through_the_model(tmp_path, device, decode):
    """One layer, a window of 9: changing a token moves the logits of the 8
    tokens after it and of no later one."""
    cfg = {
        "architecture": "Fetolix", "vocab": 280, "width": 32, "norm": {"eps": 1e-5},
        "layers": [win(heads=2, dim=8, rot=4, vdim=8, rank=16, base=100.0, q_rank=12,
                       window=9, ff=24)],
        "loop": {"start": 0, "stop": 1, "times": 1}, "token_side": {"dim": 4},
    }
    save_file(make_weights(cfg, seed=5), str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    replay = TraceReplay(make_engine(str(tmp_path), device))
    ids = tokens(60, cfg)
    cuts = [14] + [1] * 46 if decode else [60]
    base = feed(replay, "a", ids, cuts)
    for j in (0, 15, 16, 40):  # a page's last and first token among them
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-4
        assert moved[j : j + 9].all(), j
        assert not moved[:j].any() and not moved[j + 9 :].any(), j


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    ids = tokens(400, cfg, seed=3)
    got = feed(TraceReplay(make_engine(path, device)), "a", ids, [5] + [1] * 395)
    assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replay_matches_eager(checkpoints, dtype):
    """Decode-only steps replay a captured graph; every replay, with other work
    in between, matches the eager step."""
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


@pytest.mark.parametrize("pool", [96, 9])
def test_greedy_generation_through_the_engine(checkpoints, device, pool):
    """engine.submit: chunked prefill, continuous batching, the sampler, page
    reuse across turns; the small pool preempts."""
    path, cfg, W = checkpoints["odd"]
    eng = make_engine(path, device, start=True, num_kv_blocks=pool, max_prefill_tokens=24)
    try:
        prompts = [tokens(n, cfg, seed=n) for n in (5, 41, 60, 17)]
        prompts.append(prompts[2] + tokens(4, cfg, seed=99))  # extends a finished turn
        for group in (prompts[:4], prompts[4:]):
            reqs = [
                eng.submit(InferenceRequest(list(p), SamplingParams(max_tokens=24, temperature=0.0)))
                for p in group
            ]
            for p, r in zip(group, reqs):
                assert r.wait(120) == greedy(cfg, W, p, 24, 261)
        if pool == 96:
            assert eng.metrics()["continuation_hits"] >= 1
        else:
            assert eng.metrics()["preemptions"] >= 1
    finally:
        eng.stop()


def test_presets_and_random_init(device):
    cfg = EngineConfig(model="tiny-fetolix", device=device, num_kv_blocks=64)
    eng = InferenceEngine(cfg)
    try:
        res = eng.chat([{"role": "user", "content": "hello"}],
                       sampling=SamplingParams(max_tokens=6, temperature=0.8))
        assert res.completion_tokens <= 6 and res.finish_reason in ("stop", "length")
    finally:
        eng.stop()
    assert PRESETS["fetolix-8b"].params_bytes() > 10e9


def test_small_vocabulary_runs_on_token_ids(tmp_path):
    """Too few ids for bytes and specials: requests are token ids."""
    cfg = json.loads(json.dumps(CONFIGS["ones"]))
    cfg["vocab"] = 50
    save_file(make_weights(cfg), str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    eng = make_engine(str(tmp_path), "cpu", start=True)
    try:
        r = eng.generate([1, 2, 3], SamplingParams(max_tokens=4, temperature=0.0))
        assert len(r.output_ids) == 4 and eng._live == 50
    finally:
        eng.stop()


# ---------------------------------------------------------- tensor parallel

SHARDED = {
    "architecture": "Fetolix", "vocab": 300, "width": 32, "norm": {"eps": 1e-2},
    "layers": [
        win(heads=2, dim=8, rot=4, vdim=6, rank=16, base=1e3, q_rank=12, window=11, ff=26),
        full(heads=4, dim=6, rot=4, vdim=8, rank=20, base=1e4, ff=40),
    ],
    "loop": {"start": 1, "stop": 2, "times": 2}, "token_side": {"dim": 4},
}


def _tp_worker(rank, path, prompt, q):
    try:
        os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT="29541")
        import torch.distributed as dist

        from agentcontrolplane_amd.parallel.tp import run_tp_worker

        torch.set_num_threads(2)
        dist.init_process_group("gloo", rank=rank, world_size=2)
        eng = make_engine(path, "cpu", start=rank == 0, tensor_parallel=2, max_prefill_tokens=16)
        if rank:
            run_tp_worker(eng)
            q.put((rank, eng.model.layers[0].mixer.heads))
        else:
            req = eng.generate(prompt, SamplingParams(max_tokens=12, temperature=0.0), timeout=120)
            eng.stop()
            q.put((rank, req.output_ids))
    except Exception as e:  # pragma: no cover
        import traceback

        q.put((rank, f"{e}\n{traceback.format_exc()}"))


def test_tensor_parallel_generation(tmp_path):
    """Two ranks, each with its heads and feed-forward columns: one model."""
    import torch.multiprocessing as mp

    W = make_weights(SHARDED, seed=4)
    save_file(W, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(SHARDED))
    prompt = tokens(21, SHARDED)
    want = greedy(SHARDED, {k: v.double() for k, v in W.items()}, prompt, 12, 261)
    ctx = mp.get_context("spawn")
    q = ctx.Queue()
    procs = [ctx.Process(target=_tp_worker, args=(r, str(tmp_path), prompt, q)) for r in (0, 1)]
    for p in procs:
        p.start()
    got = dict(q.get(timeout=180) for _ in procs)
    for p in procs:
        p.join(timeout=30)
    assert got[0] == want and got[1] == 1, got


# -------------------------------------------------------------- command line


def test_serve_takes_the_checkpoint_configuration(checkpoints, tmp_path):
    from argparse import Namespace

    from agentcontrolplane_amd.__main__ import _engine_config

    path, _, _ = checkpoints["wide"]
    args = Namespace(model=None, checkpoint=path, dtype="float32", kv_blocks=64)
    cfg = _engine_config(args, "cpu").model_config()
    assert cfg.architecture == "Fetolix" and cfg.dtype == "float32" and cfg.vocab_size == 400
    # checkpoints that name no registered design keep the preset route
    (tmp_path / "config.json").write_text('{"architectures": ["LlamaForCausalLM"]}')
    args = Namespace(model=None, checkpoint=str(tmp_path), dtype=None, kv_blocks=None)
    assert _engine_config(args, "cuda").model == "llama3-8b"
    assert _engine_config(args, "cpu").model == "tiny"


# -------------------------------------------------------------- trace runner


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
