"""Lobuvik end to end against the plain oracle: checkpoints in the design's own config
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

import lobuvik_oracle as oracle
from agentcontrolplane_amd.engine.config import (
    PRESETS, ClampedGluSpec, EngineConfig, ExpertsSpec, GroupedAttentionSpec,
    LatentAttentionSpec, WavelengthScaling, YarnScaling,
)
from agentcontrolplane_amd.engine.engine import InferenceEngine
from agentcontrolplane_amd.engine.request import InferenceRequest, SamplingParams
from agentcontrolplane_amd.engine.trace import TraceReplay
from agentcontrolplane_amd.models.configs import read_architecture, read_model_config
from agentcontrolplane_amd.models.weights import save_checkpoint
from model_helpers import CUTS, assert_close, feed, make_engine, tokens

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.param("cuda", marks=pytest.mark.gpu)


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit=1.5, shared=None, shared_limit=1.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit},
            "router": {"experts": experts, "top": top},
            "shared": {"ff": shared, "limit": shared_limit} if shared else None}


def biased(heads, kv, dim, vdim, conv, reach, mlp=None, scale=0.4, coef=0.6, every=9):
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale,
        "bias_max": reach, "q_temp": {"coef": coef, "every": every}}}


def latent(heads, dim, rot, vdim, rank, size, mlp=None, base=500.0, factor=4.0, original=64,
           fast=8.0, slow=0.5):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
        "scale": 1.3 * (dim + rot) ** -0.5, "mask": {"size": size},
        "rot": {"base": base, "dims": rot, "scaling": {
            "factor": factor, "original": original, "fast": fast, "slow": slow}}}}


def rotated(heads, kv, dim, vdim, dims, size, mlp=None, cap=6.0, scale=0.3, base=300.0,
            factor=5.0, low=0.7, high=3.0, original=90):
    return {"type": "attention_2", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
        "softcap": cap, "mask": {"size": size}, "rot": {"base": base, "dims": dims, "scaling": {
            "factor": factor, "low": low, "high": high, "original": original}}}}


def config(vocab, width, layers, eps=1e-5, scale=0.7):
    return {"architecture": "Lobuvik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


#: name -> (config, rows of the distance tables by layer)
CONFIGS = {
    # odd sizes, no two layers alike, layers without a feed-forward or a shared expert
    "odd": (config(311, 42, [
        rotated(6, 2, 10, 14, 6, 7, dense(33)),
        biased(4, 2, 12, 6, 3, 40, moe(5, 2, 9, 1.2, 21)),
        latent(3, 10, 6, 14, 20, 23, moe(7, 3, 11, 0.8)),
        biased(3, 3, 9, 20, 5, 30),
        latent(5, 8, 4, 6, 9, 5),
        rotated(4, 1, 8, 8, 8, 40, moe(3, 3, 17, 2.0, 5, 3.0)),
    ], eps=0.03), {1: 10, 3: 4}),
    # head, latent and inner sizes the matrix-core kernels take unpadded
    "wide": (config(400, 128, [
        biased(8, 2, 64, 128, 4, 100, moe(4, 2, 128, 1.5, 96)),
        latent(4, 64, 64, 64, 128, 50, dense(96)),
        rotated(16, 4, 64, 64, 32, 33, moe(8, 3, 64, 1.25, 128)),
        biased(2, 1, 128, 64, 2, 64, dense(64)),
    ], scale=1.3), {0: 32, 3: 16}),
    # beyond the matrix-core kernels' sizes
    "large": (config(290, 64, [
        biased(2, 1, 260, 20, 4, 20, dense(64), scale=0.1),
        latent(2, 30, 70, 20, 530, 30, moe(3, 1, 20, 1.0, 16)),
        rotated(2, 2, 24, 270, 24, 20, moe(2, 2, 30)),
    ], eps=1e-3), {0: 8}),
    # nothing repeated: one head, one dimension, one tap, one expert, a window of one token
    "ones": (config(270, 16, [
        biased(1, 1, 1, 1, 1, 2, moe(1, 1, 1, 1.0, 1), every=1),
        latent(1, 1, 2, 1, 1, 1, moe(2, 1, 3)),
        rotated(1, 1, 2, 1, 2, 1, dense(1)),
    ], eps=0.5, scale=1.0), {0: 2}),
}


def make_weights(cfg, buckets, seed=0):
    """bf16 tensors with scores, biases, gates and routes that vary."""
    g = torch.Generator().manual_seed(seed)
    w, V = cfg["width"], cfg["vocab"]

    def t(*shape, gain=1.0):
        return (torch.randn(*shape, generator=g) * gain * shape[-1] ** -0.5).bfloat16()

    def vec(*shape, mean=0.0, spread=0.3):
        return (mean + spread * torch.randn(*shape, generator=g)).bfloat16()

    W = {"embed": t(V, w, gain=3.0), "final.norm": vec(w, mean=1), "head": t(V, w)}
    for i, spec in enumerate(cfg["layers"]):
        m, p, H = spec["mixer"], f"l{i}.mix.", spec["mixer"]["heads"]
        W[f"l{i}.norm1"] = vec(w, mean=1)
        W[p + "o"] = t(w, H * m["vdim"])
        if spec["type"] == "latent_attention":
            W[p + "q"] = t(H * (m["dim"] + m["rot_dim"]), w, gain=1.5)
            W[p + "dkv"] = t(m["kv_rank"] + m["rot_dim"], w, gain=1.5)
            W[p + "dkv.norm"] = vec(m["kv_rank"], mean=1)
            W[p + "uk"] = t(H * m["dim"], m["kv_rank"])
            W[p + "uv"] = t(H * m["vdim"], m["kv_rank"], gain=2.0)
            W[p + "sink"] = vec(H, spread=1.0)
        else:
            G = m["kv_heads"]
            for n, size in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"])):
                W[p + n] = t(size, w, gain=1.5)
            if spec["type"] == "attention":
                for n in "qkv":
                    W[p + n + ".b"] = vec(len(W[p + n]))
                    W[p + n + ".conv"] = t(len(W[p + n]), m["conv"], gain=1.5)
                W[p + "q.norm"], W[p + "k.norm"] = (vec(m["dim"], mean=1) for _ in range(2))
                W[p + "rel"] = vec(buckets[i], H, spread=1.0)
                W[p + "pb"], W[p + "o.b"] = vec(H, mean=-2, spread=1.0), vec(w)
            else:
                W[p + "temp"], W[p + "g"] = vec(H, mean=1), t(H, w, gain=2.0)
        mlp = spec["mlp"]
        if not mlp:
            continue
        W[f"l{i}.norm2"] = vec(w, mean=1)
        units = [("", mlp.get("ff"))]
        if mlp["kind"] == "moe":
            E = mlp["router"]["experts"]
            # spread-out logits: an expert near the edge of being chosen weighs little
            W[f"l{i}.mlp.router"], W[f"l{i}.mlp.router.b"] = t(E, w, gain=4.0), vec(E)
            units = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(E)]
            units += [("shared.", mlp["shared"]["ff"])] if mlp["shared"] else []
        for n, ff in units:
            W[f"l{i}.mlp.{n}gate"], W[f"l{i}.mlp.{n}up"] = t(ff, w, gain=1.5), t(ff, w)
            W[f"l{i}.mlp.{n}down"] = t(w, ff)
    return W


def write_checkpoint(path, cfg, W):
    save_file(W, str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return str(path)


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
    """name -> (folder, config, float64 weights)"""
    out = {}
    for n, (name, (cfg, buckets)) in enumerate(CONFIGS.items()):
        W = make_weights(cfg, buckets, seed=n)
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
    assert read_architecture(path) == cfg.architecture == "Lobuvik"
    assert (cfg.vocab_size, cfg.hidden_size, cfg.rms_eps, cfg.embed_scale) == (311, 42, 0.03, 0.7)
    a, b, c = (cfg.layers[i].mixer for i in (1, 2, 0))
    assert isinstance(a, GroupedAttentionSpec) and isinstance(b, LatentAttentionSpec)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.conv, a.window, a.sigmoid) == (
        4, 2, 12, 6, 3, None, True)
    assert (a.distance_bias.buckets, a.distance_bias.reach) == (10, 40)
    assert (a.q_temp.coef, a.q_temp.every) == (0.6, 9)
    assert (b.heads, b.dim, b.rot_dim, b.vdim, b.kv_rank, b.window, b.sink, b.q_rank) == (
        3, 10, 6, 14, 20, 23, True, None)
    assert b.rope_scaling == YarnScaling(4.0, 64, 8.0, 0.5) and b.rope_half and not b.head_gate
    assert (c.window, c.softcap, c.rotary.dims, c.head_temp, c.head_gate) == (7, 6.0, 6, True, True)
    assert c.rotary.scaling == WavelengthScaling(5.0, 0.7, 3.0, 90)
    assert cfg.layers[1].mlp == ExpertsSpec(5, 2, ClampedGluSpec(9, 1.2), ClampedGluSpec(21, 1.0))
    assert cfg.layers[2].mlp.shared is None and cfg.layers[3].mlp is None
    assert cfg.params_bytes(1) == sum(v.numel() for v in W.values())


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="attention_9"),
    lambda d: d["layers"][0]["mlp"].update(kind="sparse"),
    lambda d: d["layers"][1]["mlp"]["router"].update(top=6),
    lambda d: d["layers"][1]["mixer"].update(bias_max=5),
    lambda d: d["layers"][1]["mixer"].update(kv_heads=3),
    lambda d: d["layers"][2]["mixer"]["rot"].update(dims=4),
    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=12),
    lambda d: d.update(architecture="Other"),
])
def test_config_reader_refuses(checkpoints, tmp_path, change):
    path, cfg, W = checkpoints["odd"]
    d = json.loads(json.dumps(cfg))
    change(d)
    write_checkpoint(tmp_path, d, {k: v.bfloat16() for k, v in W.items()})
    with pytest.raises(ValueError):
        read_model_config(str(tmp_path))


@pytest.mark.parametrize("name", ["l1.mlp.e4.down", "l1.mix.k.conv", "l2.mix.sink", "head"])
def test_loader_refuses_wrong_shape(checkpoints, tmp_path, name):
    _, cfg, W = checkpoints["odd"]
    W = {k: v.bfloat16() for k, v in W.items()}
    W[name] = W[name][:-1].contiguous()
    with pytest.raises(ValueError, match=name):
        make_engine(write_checkpoint(tmp_path, cfg, W), "cpu")


def test_checkpoint_round_trip(checkpoints, tmp_path):
    """Export undoes the padded, paired, fused layout exactly."""
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
def test_residual_after_every_layer(checkpoints, device, name):
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


def assert_near(got, want, dtype):
    """assert_close(), tighter in bf16: these models leave its rounding little to amplify."""
    if dtype == "float32":
        return assert_close(got, want)
    d = got.double() - want.double()
    err = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.double().std()
    assert err.max() < 0.12, (err.max().item(), err.argmax().item())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("name", CONFIGS)
def test_portions(checkpoints, device, name, cuts, dtype):
    """However the prompt is cut, decoded tail included, the logits are the whole
    sequence's: windows of 1 to 50, convolutions and pages of 16 pass by."""
    path, cfg, W = checkpoints[name]
    ids = tokens(150, cfg)
    replay = TraceReplay(make_engine(path, device, dtype))
    got = feed(replay, "a", ids, CUTS[cuts](len(ids)))
    assert_near(got, oracle.forward(cfg, W, ids), dtype)
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
    at, queue, live, rows = {r: 0 for r in ids}, list(lens), [], {r: [] for r in ids}
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
        for e in entries:
            n, r = len(e["tokens"]), e["id"]
            rows[r].append(got[:n])
            got = got[n:]
            at[r] += n
        for r in end:
            live.remove(r)
    for r in ids:
        assert_near(torch.cat(rows[r]), want[r], dtype)
    assert eng.bm.free_blocks == 19 and eng.states.free == 3


def test_first_tokens(checkpoints, device):
    for name, (path, cfg, W) in checkpoints.items():
        replay = TraceReplay(make_engine(path, device))
        for n in (1, 2, 3):
            ids = tokens(n, cfg, seed=n)
            got = feed(replay, f"{name}{n}", ids, [1] * n)
            assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("kind", ["latent", "rotated"])
@pytest.mark.parametrize("decode", [False, True])
def test_window_edges_through_the_model(tmp_path, device, decode, kind):
    """One layer with a window of 9: changing a token moves its own logits and those of
    the 8 tokens after it, and no others."""
    layer = latent(2, 8, 8, 8, 16, 9) if kind == "latent" else rotated(2, 1, 8, 8, 4, 9)
    cfg = config(280, 32, [layer])
    path = write_checkpoint(tmp_path, cfg, make_weights(cfg, {}, seed=5))
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(60, cfg)
    cuts = [14] + [1] * 46 if decode else [60]
    base = feed(replay, "a", ids, cuts)
    for j in (0, 1, 15, 16, 40):  # the first tokens, a page's last and first
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-6
        assert moved[j : j + 9].all() and not moved[:j].any() and not moved[j + 9 :].any(), j


@pytest.mark.parametrize("decode", [False, True])
def test_far_keys_and_convolution_through_the_model(tmp_path, device, decode):
    """One layer of biased attention without a window: a changed token moves every later
    position, however far, and none before it."""
    cfg = config(280, 32, [biased(2, 1, 8, 8, 4, 20)])
    W = make_weights(cfg, {0: 8}, seed=6)
    W["l0.mix.rel"][-1] = 3.0  # far keys weigh
    path = write_checkpoint(tmp_path, cfg, W)
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(300, cfg)
    cuts = [14, 2, 2] + [1] * 282 if decode else [300]
    base = feed(replay, "a", ids, cuts)
    assert_close(base, oracle.forward(cfg, {k: v.double() for k, v in W.items()}, ids))
    for j in (0, 13, 16, 40):
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-6
        assert moved[j:].float().mean() > 0.98 and not moved[:j].any(), j


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    ids = tokens(400, cfg, seed=3)
    got = feed(TraceReplay(make_engine(path, device)), "a", ids, [5] + [1] * 395)
    assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompts_that_fill_expert_tiles(checkpoints, device, dtype):
    """Prompts long enough for the tiled expert products, beside decoded tokens."""
    path, cfg, W = checkpoints["wide"]
    long, short = tokens(700, cfg, seed=1), tokens(30, cfg, seed=2)
    replay = TraceReplay(make_engine(path, device, dtype))
    replay.step([{"id": "s", "tokens": short[:29], "want": []}], [])
    got = replay.step([{"id": "l", "tokens": long, "want": list(range(700))},
                       {"id": "s", "tokens": short[29:], "want": [0]}], ["l", "s"])
    assert_near(got[:700], oracle.forward(cfg, W, long), dtype)
    assert_near(got[700:], oracle.forward(cfg, W, short)[-1:], dtype)


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
    # keys are split over workgroups by the captured table width: the sums round apart
    tol = 1e-3 if dtype == "float32" else 2e-2
    assert (runs[0] - runs[1]).abs().max() <= tol * runs[1].abs().max()


def test_models_without_convolutions_keep_no_state(tmp_path, device):
    cfg = config(280, 32, [latent(2, 8, 8, 8, 16, 9), rotated(2, 1, 8, 8, 4, 9, dense(20))])
    W = make_weights(cfg, {}, seed=8)
    eng = make_engine(write_checkpoint(tmp_path, cfg, W), device)
    assert eng.states is None and eng.model.state_slot_bytes == 0
    ids = tokens(40, cfg)
    got = feed(TraceReplay(eng), "a", ids, [17, 3] + [1] * 20)
    assert_close(got, oracle.forward(cfg, {k: v.double() for k, v in W.items()}, ids))


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
        assert eng.states.free == slots - len(eng.scheduler.retired)
    finally:
        eng.stop()


def test_presets_and_random_init(device):
    cfg = EngineConfig(model="tiny-lobuvik", device=device, num_kv_blocks=64, max_batch_size=8)
    eng = InferenceEngine(cfg)
    try:
        res = eng.chat([{"role": "user", "content": "hello"}],
                       sampling=SamplingParams(max_tokens=6, temperature=0.8))
        assert res.completion_tokens <= 6 and res.finish_reason in ("stop", "length")
    finally:
        eng.stop()
    for name in ("lobuvik-8b", "lobuvik-2b"):
        p = PRESETS[name]
        assert {x.mlp.width for x in p.layers} == {p.intermediate_size}  # per token, all alike


# ---------------------------------------------------------- tensor parallel

SHARDED = config(300, 32, [
    biased(4, 2, 8, 6, 3, 30, moe(4, 2, 12, 1.5, 10)),
    latent(4, 8, 4, 6, 12, 17, dense(26)),
    rotated(2, 2, 8, 6, 4, 11, moe(3, 1, 8)),
], eps=1e-2)


def _tp_worker(rank, path, prompt, q):
    try:
        os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT="29549")
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
    """Two ranks, each with its heads, convolution channels and feed-forward columns: one
    model, its output bias added once."""
    import torch.multiprocessing as mp

    W = make_weights(SHARDED, {0: 8}, seed=4)
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
    assert got[0] == want and got[1] == [2, 2, 1], got


# -------------------------------------------------- command line, trace runner


def test_serve_takes_the_checkpoint_configuration(checkpoints):
    from argparse import Namespace

    from agentcontrolplane_amd.__main__ import _engine_config

    args = Namespace(model=None, checkpoint=checkpoints["wide"][0], dtype="float32", kv_blocks=64)
    cfg = _engine_config(args, "cpu").model_config()
    assert cfg.architecture == "Lobuvik" and cfg.dtype == "float32" and cfg.vocab_size == 400


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
