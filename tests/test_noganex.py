"""Noganex end to end against the plain oracle: checkpoints in the design's own config
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

import noganex_oracle as oracle
from agentcontrolplane_amd.engine.config import (
    PRESETS, EngineConfig, GatedDeltaSpec, GroupedAttentionSpec, YarnScaling, gelu_glu, silu_glu,
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


def moe(experts, top, ff, scale=1.3, shared=None):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "scale": scale},
            "shared": {"ff": shared} if shared else None}


def attention(heads, kv, dim, vdim, dims, size, mlp=None, scale=0.3, base=300.0, factor=3.0,
              original=90, fast=8.0, slow=0.5):
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
        "mask": {"size": size}, "rot": {"base": base, "dims": dims, "scaling": {
            "factor": factor, "original": original, "fast": fast, "slow": slow}}}}


def delta(heads, kv, dim, vdim, conv, mlp=None):
    return {"type": "delta", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def again(layers, j):
    return {**layers[j], "weights_of": j}


def config(vocab, width, layers, eps=1e-5, scale=0.7):
    return {"architecture": "Noganex", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "logit_scale": scale, "layers": layers}


# odd sizes, no two owners alike, layers without a feed-forward or a shared expert; both
# kinds of layers used again, before and after others
_ODD = [
    delta(4, 2, 12, 18, 3, moe(5, 2, 9, 1.7, 21)),
    attention(6, 2, 10, 14, 6, 7, dense(33)),
    delta(3, 3, 9, 20, 5),
    attention(3, 1, 8, 6, 8, 40, moe(3, 3, 17)),
]
_ODD += [again(_ODD, 1), again(_ODD, 0)]
# head, group and inner sizes the matrix-core kernels take unpadded
_WIDE = [
    attention(16, 4, 64, 128, 32, 50, dense(96), scale=0.15),
    delta(4, 2, 64, 64, 4, moe(8, 3, 64, 0.8, 128)),
    attention(4, 4, 128, 64, 128, 33, moe(4, 2, 128, 2.0, 96), scale=0.1),
    delta(8, 8, 32, 128, 4, dense(64)),
]
_WIDE += [again(_WIDE, 1), again(_WIDE, 0)]
CONFIGS = {
    "odd": config(311, 42, _ODD, eps=0.03),
    "wide": config(400, 128, _WIDE, scale=1.4),
    # beyond the matrix-core kernels' sizes
    "large": config(290, 64, [
        attention(4, 2, 260, 20, 24, 20, dense(64), scale=0.06),
        delta(2, 1, 20, 270, 4, moe(3, 1, 20, 1.0, 16)),
        attention(10, 5, 24, 270, 24, 30, moe(2, 2, 30)),
    ], eps=1e-3),
    # nothing repeated: one head, the fewest dimensions, one tap, one expert, chunks of one token
    "ones": config(270, 16, [
        attention(1, 1, 2, 1, 2, 1, moe(1, 1, 1, 1.0, 1)),
        delta(1, 1, 1, 1, 1, dense(1)),
        attention(1, 1, 2, 1, 2, 3),
    ], eps=0.5, scale=1.0),
}


def make_weights(cfg, seed=0):
    """bf16 tensors with scores, gates, decays and routes that vary."""
    g = torch.Generator().manual_seed(seed)
    w, V = cfg["width"], cfg["vocab"]

    def t(*shape, gain=1.0):
        return (torch.randn(*shape, generator=g) * gain * shape[-1] ** -0.5).bfloat16()

    def vec(*shape, mean=0.0, spread=0.3):
        return (mean + spread * torch.randn(*shape, generator=g)).bfloat16()

    W = {"embed": t(V, w, gain=w ** 0.5), "final.norm": vec(w, mean=1), "head": t(V, w)}
    for i, spec in enumerate(cfg["layers"]):
        if "weights_of" in spec:
            continue
        m, p, H, G = spec["mixer"], f"l{i}.mix.", *(spec["mixer"][n] for n in ("heads", "kv_heads"))
        mlp = spec["mlp"]
        for n in ("1", "2") if mlp else ("1",):
            # in 16 bits a close call among experts may go either way: it weighs little
            routed = n == "2" and mlp["kind"] == "moe"
            W[f"l{i}.norm{n}"] = vec(w, mean=0.25 if routed else 1, spread=0.1 if routed else 0.3)
            W[f"l{i}.rg{n}"], W[f"l{i}.rg{n}.b"] = t(w, w), vec(w)
        for n, size in (("q", (H if spec["type"] == "attention" else G) * m["dim"]),
                        ("k", G * m["dim"]),
                        ("v", (G if spec["type"] == "attention" else H) * m["vdim"])):
            W[p + n] = t(size, w)
            if spec["type"] == "delta":
                W[p + n + ".conv"] = t(size, m["conv"], gain=1.5)
        W[p + "o"] = t(w, H * m["vdim"])
        if spec["type"] == "attention":
            W[p + "q.norm"], W[p + "k.norm"] = (vec(len(W[p + n]), mean=1) for n in "qk")
            W[p + "talk"] = (torch.eye(H) + 0.4 * torch.randn(H, H, generator=g)).bfloat16()
        else:
            W[p + "b"], W[p + "a"], W[p + "g"] = t(H, w), t(H, w), t(H * m["vdim"], w)
            W[p + "A_log"], W[p + "dt_bias"] = vec(H, spread=1.0), vec(H, mean=-2, spread=1.0)
            W[p + "norm"] = vec(m["vdim"], mean=1)
        if not mlp:
            continue
        units = [("", mlp.get("ff"))]
        if mlp["kind"] == "moe":
            E = mlp["router"]["experts"]
            # scores near zero or one: the corrections decide among equals, few calls are close
            W[f"l{i}.mlp.router"], W[f"l{i}.mlp.correction"] = t(E, w, gain=8.0), vec(E)
            units = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(E)]
            units += [("shared.", mlp["shared"]["ff"])] if mlp["shared"] else []
        for n, ff in units:
            for name, rows, cols in (("gate", ff, w), ("up", ff, w), ("down", w, ff)):
                W[f"l{i}.mlp.{n}{name}"] = t(rows, cols)
                if mlp["kind"] == "dense":
                    W[f"l{i}.mlp.{n}{name}.b"] = vec(rows)
    return W


def write_checkpoint(path, cfg, W):
    save_file(W, str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return str(path)


def doubles(W):
    return {k: v.double() for k, v in W.items()}


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
    """name -> (folder, config, float64 weights)"""
    out = {}
    for n, (name, cfg) in enumerate(CONFIGS.items()):
        W = make_weights(cfg, seed=n)
        out[name] = (write_checkpoint(tmp_path_factory.mktemp(name), cfg, W), cfg, doubles(W))
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
    assert read_architecture(path) == cfg.architecture == "Noganex"
    assert (cfg.vocab_size, cfg.hidden_size, cfg.rms_eps, cfg.logit_scale) == (311, 42, 0.03, 0.7)
    a, b = cfg.layers[1].mixer, cfg.layers[0].mixer
    assert isinstance(a, GroupedAttentionSpec) and isinstance(b, GatedDeltaSpec)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.chunk, a.scale) == (6, 2, 10, 14, 7, 0.3)
    assert a.talk and a.row_norm and a.window is None and not (a.bias or a.sink or a.qk_norm)
    assert (a.rotary.base, a.rotary.dims) == (300.0, 6)
    assert a.rotary.scaling == YarnScaling(3.0, 90, 8.0, 0.5)
    assert (b.heads, b.kv_heads, b.dim, b.vdim, b.conv, b.decays) == (4, 2, 12, 18, 3, 4)
    assert b.head_decay and b.gate_silu
    m = cfg.layers[0].mlp
    assert (m.experts, m.top, m.scale, m.sigmoid, m.correction) == (5, 2, 1.7, True, True)
    assert m.expert == silu_glu(9) and m.shared == silu_glu(21)
    assert cfg.layers[1].mlp == gelu_glu(33, bias=True)
    assert cfg.layers[3].mlp.shared is None and cfg.layers[2].mlp is None
    assert [x.weights_of for x in cfg.layers] == [None] * 4 + [1, 0]
    assert cfg.params_bytes(1) == sum(v.numel() for v in W.values())


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="delta_9"),
    lambda d: d["layers"][1]["mlp"].update(kind="sparse"),
    lambda d: d["layers"][0]["mlp"]["router"].update(top=6),
    lambda d: d["layers"][0]["mixer"].update(kv_heads=3),
    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=12),
    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=5),
    lambda d: d["layers"][4].update(weights_of=5),
    lambda d: d["layers"][4].update(weights_of=9),
    lambda d: d["layers"][4].update(weights_of=3),
    lambda d: d.update(architecture="Other"),
])
def test_config_reader_refuses(checkpoints, tmp_path, change):
    path, cfg, W = checkpoints["odd"]
    d = json.loads(json.dumps(cfg))
    change(d)
    write_checkpoint(tmp_path, d, {k: v.bfloat16() for k, v in W.items()})
    with pytest.raises(ValueError):
        read_model_config(str(tmp_path))


@pytest.mark.parametrize("name", [
    "l0.mlp.e4.down", "l0.mix.k.conv", "l1.mix.talk", "l1.mix.q.norm", "l1.rg2.b", "head"])
def test_loader_refuses_wrong_shape(checkpoints, tmp_path, name):
    _, cfg, W = checkpoints["odd"]
    W = {k: v.bfloat16() for k, v in W.items()}
    W[name] = W[name][:-1].contiguous()
    with pytest.raises(ValueError, match=name):
        make_engine(write_checkpoint(tmp_path, cfg, W), "cpu")


def test_checkpoint_round_trip(checkpoints, tmp_path):
    """Export undoes the padded, paired, stacked layout exactly; layers that use another
    one's weights write none."""
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


def test_shared_weights_have_stores_of_their_own(checkpoints):
    m = make_engine(checkpoints["odd"][0], "cpu").model
    assert m.layers[4] is m.layers[1] and m.layers[5] is m.layers[0]
    assert len({t.data_ptr() for t in m.caches}) == 6 and len({t.data_ptr() for t in m.states}) == 6


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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("name", CONFIGS)
def test_portions(checkpoints, device, name, cuts, dtype):
    """However the prompt is cut, decoded tail included, the logits are the whole
    sequence's: chunks of 1 to 50, convolutions and pages of 16 pass by."""
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
        assert_close(torch.cat(rows[r]), want[r], dtype)
    assert eng.bm.free_blocks == 19 and eng.states.free == 3


def test_first_tokens(checkpoints, device):
    for name, (path, cfg, W) in checkpoints.items():
        replay = TraceReplay(make_engine(path, device))
        for n in (1, 2, 3):
            ids = tokens(n, cfg, seed=n)
            got = feed(replay, f"{name}{n}", ids, [1] * n)
            assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("cuts", [[60], [14] + [1] * 46, [2] * 30], ids=["whole", "decode", "twos"])
def test_chunk_edges_through_the_model(tmp_path, device, cuts):
    """One layer with chunks of 9: changing a token moves its own logits and those of the
    later tokens of its chunk, and no others, wherever the prompt was cut."""
    cfg = config(280, 32, [attention(4, 2, 8, 8, 4, 9)])
    path = write_checkpoint(tmp_path, cfg, make_weights(cfg, seed=5))
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(60, cfg)
    base = feed(replay, "a", ids, cuts)
    for j in (0, 1, 8, 9, 15, 16, 17, 40, 53):  # chunks' and pages' last and first tokens
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-6
        end = (j // 9 + 1) * 9
        assert moved[j:end].all() and not moved[:j].any() and not moved[end:].any(), j


@pytest.mark.parametrize("cuts", [[300], [14, 2, 2] + [1] * 282], ids=["whole", "decode"])
def test_far_tokens_through_the_model(tmp_path, device, cuts):
    """One delta layer with slow decays: a changed token moves every later position,
    however far, and none before it."""
    cfg = config(280, 32, [delta(2, 1, 8, 8, 4)])
    W = make_weights(cfg, seed=6)
    W["l0.mix.A_log"].fill_(-7.0)
    path = write_checkpoint(tmp_path, cfg, W)
    replay = TraceReplay(make_engine(path, device))
    ids = tokens(300, cfg)
    base = feed(replay, "a", ids, cuts)
    assert_close(base, oracle.forward(cfg, doubles(W), ids))
    for j in (0, 13, 16, 40):
        other = list(ids)
        other[j] = (other[j] + 1) % 280
        moved = (feed(replay, f"b{j}", other, cuts) - base).abs().amax(-1) > 1e-6
        assert moved[j:].float().mean() > 0.9 and not moved[:j].any(), j


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_long_decoding(checkpoints, device, name):
    path, cfg, W = checkpoints[name]
    ids = tokens(400, cfg, seed=3)
    got = feed(TraceReplay(make_engine(path, device)), "a", ids, [5] + [1] * 395)
    assert_close(got, oracle.forward(cfg, W, ids))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_chunks(tmp_path, device, dtype):
    """Chunks longer than a prompt's portions and a decode split's keys."""
    cfg = config(300, 64, [attention(8, 4, 64, 64, 64, 500, dense(32), scale=0.15), delta(2, 2, 16, 16, 4),
                           attention(6, 1, 64, 64, 20, 333, scale=0.15)])
    W = make_weights(cfg, seed=12)
    ids = tokens(900, cfg, seed=1)
    replay = TraceReplay(make_engine(write_checkpoint(tmp_path, cfg, W), device, dtype))
    got = feed(replay, "a", ids, [130, 200, 2, 140, 1, 1, 40] + [1] * 20 + [330] + [1] * 36)
    assert_close(got, oracle.forward(cfg, doubles(W), ids), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompts_that_fill_expert_tiles(checkpoints, device, dtype):
    """Prompts long enough for the tiled expert products, beside decoded tokens."""
    path, cfg, W = checkpoints["wide"]
    long, short = tokens(700, cfg, seed=1), tokens(30, cfg, seed=2)
    replay = TraceReplay(make_engine(path, device, dtype))
    replay.step([{"id": "s", "tokens": short[:29], "want": []}], [])
    got = replay.step([{"id": "l", "tokens": long, "want": list(range(700))},
                       {"id": "s", "tokens": short[29:], "want": [0]}], ["l", "s"])
    assert_close(got[:700], oracle.forward(cfg, W, long), dtype)
    assert_close(got[700:], oracle.forward(cfg, W, short)[-1:], dtype)


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
    tol = 1e-3 if dtype == "float32" else 3e-2
    assert (runs[0] - runs[1]).abs().max() <= tol * runs[1].abs().max()


def test_attention_alone_keeps_no_state(tmp_path, device):
    cfg = config(280, 32, [attention(2, 1, 8, 8, 4, 9, dense(20))])
    W = make_weights(cfg, seed=8)
    eng = make_engine(write_checkpoint(tmp_path, cfg, W), device)
    assert eng.states is None and eng.model.state_slot_bytes == 0
    ids = tokens(40, cfg)
    got = feed(TraceReplay(eng), "a", ids, [17, 3] + [1] * 20)
    assert_close(got, oracle.forward(cfg, doubles(W), ids))


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
    cfg = EngineConfig(model="tiny-noganex", device=device, num_kv_blocks=64, max_batch_size=8)
    eng = InferenceEngine(cfg)
    try:
        res = eng.chat([{"role": "user", "content": "hello"}],
                       sampling=SamplingParams(max_tokens=6, temperature=0.8))
        assert res.completion_tokens <= 6 and res.finish_reason in ("stop", "length")
    finally:
        eng.stop()
    for name in ("noganex-8b", "noganex-2b"):
        p = PRESETS[name]
        assert p.layers[3].weights_of == 1 and p.layers[5].weights_of is None


# ---------------------------------------------------------- tensor parallel

_SHARDED = [
    delta(4, 2, 8, 6, 3, moe(4, 2, 12, 1.5, 10)),
    attention(3, 1, 8, 6, 4, 11, dense(26)),
    delta(2, 2, 8, 6, 4, moe(3, 1, 8)),
]
SHARDED = config(300, 32, _SHARDED + [again(_SHARDED, 0)], eps=1e-2)


def _tp_worker(rank, path, prompt, q):
    try:
        os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT="29551")
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
    """Two ranks, each with its delta heads and feed-forward columns and all attention
    heads: one model, its output biases added once."""
    import torch.multiprocessing as mp

    W = make_weights(SHARDED, seed=4)
    path = write_checkpoint(tmp_path, SHARDED, W)
    prompt = tokens(21, SHARDED)
    want = [greedy(SHARDED, doubles(W), p, 12, 261) for p in (prompt, prompt[3:])]
    ctx = mp.get_context("spawn")
    q = ctx.Queue()
    procs = [ctx.Process(target=_tp_worker, args=(r, path, prompt, q)) for r in (0, 1)]
    for p in procs:
        p.start()
    got = dict(q.get(timeout=180) for _ in procs)
    for p in procs:
        p.join(timeout=30)
    assert got[0] == want and got[1] == [2, 3, 1, 2], got


# -------------------------------------------------- command line, trace runner


def test_serve_takes_the_checkpoint_configuration(checkpoints):
    from argparse import Namespace

    from agentcontrolplane_amd.__main__ import _engine_config

    args = Namespace(model=None, checkpoint=checkpoints["wide"][0], dtype="float32", kv_blocks=64)
    cfg = _engine_config(args, "cpu").model_config()
    assert cfg.architecture == "Noganex" and cfg.dtype == "float32" and cfg.vocab_size == 400


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
