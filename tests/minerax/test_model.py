"""Whole Minerax models through the engine (scheduler, paged cache, state slots) against the slow
oracle: whole prompts, token-by-token decoding, portions, mixed batches with pages and slots
reused, window edges in prompts and in decoding, greedy generation."""
import pytest
import torch

from . import oracle
from .common import (ODD, ONES, SMALL, WIDE, alone, both, build, check, config, dense, latent, left, right,
                     run_schedule, tokens, yarn)

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [SMALL, ONES, ODD], ids=["small", "ones", "odd"])
def test_whole_prompt_and_token_by_token(device, cfg):
    eng, full = build(cfg, device)
    if device != "cpu":
        assert eng.model.w["embed"].is_cuda
    t = tokens(75, cfg["vocab"], 1)
    check(run_schedule(eng, alone(t, [])), cfg, full, {"a": t})
    check(run_schedule(eng, alone(t, [40] + [1] * 35)), cfg, full, {"a": t})


@pytest.mark.parametrize("device", DEVICES)
def test_residual_stream_after_every_layer(device):
    cfg = SMALL
    eng, full = build(cfg, device)
    t = tokens(45, cfg["vocab"], 3)
    want = []
    oracle.forward(cfg, full, t, want)
    taps, fwd = [], eng.model.forward
    eng.model.forward = lambda m: fwd(m, taps)
    try:
        run_schedule(eng, alone(t, []))
    finally:
        eng.model.forward = fwd
    assert len(taps) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(taps, want)):
        err = float((a.double().cpu() - b).abs().max() / b.abs().max())
        assert err < 1e-4, f"layer {i}: {err:.2e}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[2] * 30, [3, 2, 33, 2, 5, 31, 2], [32, 32, 1, 1, 2], [64, 2],
                                  [7, 7, 7, 7, 7, 7, 7, 7, 7, 7, 2, 1, 1]])
def test_portions(device, cuts):
    """Portions down to two tokens (shorter than the convolutions), cut inside pages and windows.
    Short ones run in the decode section (<= 32 rows), long ones in the prefill section."""
    eng, full = build(SMALL, device)
    t = tokens(90, SMALL["vocab"], 2)
    check(run_schedule(eng, alone(t, cuts)), SMALL, full, {"a": t})


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_one_token_requests(device):
    for cfg in (ONES, SMALL):
        eng, full = build(cfg, device)
        for n in (1, 2, 3, 5):
            t = tokens(n, cfg["vocab"], 10 + n)
            check(run_schedule(eng, alone(t, [])), cfg, full, {"a": t})
            check(run_schedule(eng, alone(t, [1] * n)), cfg, full, {"a": t})


@pytest.mark.parametrize("device", DEVICES)
def test_batches_of_unequal_requests(device):
    """Up to four live requests, portions beside single tokens, requests that pause, pages and
    slots given back and used again by later requests: each row as if its request ran alone."""
    cfg = SMALL
    eng, full = build(cfg, device, max_kv_blocks=14)       # 13 pages: reuse is forced
    V = cfg["vocab"]
    req = {n: tokens(L, V, 20 + i) for i, (n, L) in enumerate(
        [("a", 97), ("b", 40), ("c", 5), ("d", 66), ("e", 130), ("f", 33), ("g", 64)])}
    at = {n: 0 for n in req}

    def take(n, c):
        lo = at[n]
        at[n] = lo + c
        return (n, req[n][lo:lo + c], list(range(c)))

    plan = [
        [("a", 50), ("b", 2), ("c", 5)], [("a", 1), ("b", 33), ("d", 40)], [("a", 1), ("b", 5)],
        [("a", 45), ("d", 2)], [("d", 24), ("e", 64), ("f", 3)], [("e", 1), ("f", 30)],
        [("e", 2), ("g", 64)], [("e", 63)],
    ]
    steps = []
    for st in plan:
        entries = [take(n, c) for n, c in st]
        steps.append({"entries": entries, "end": [n for n, _ in st if at[n] == len(req[n])]})
    assert all(at[n] == len(req[n]) for n in req)
    got = run_schedule(eng, steps)
    check(got, cfg, full, req)
    assert len(got) == sum(len(t) for t in req.values())
    assert eng.core.num_free_state_slots == 4 and eng.core.num_free_blocks == 13


@pytest.mark.parametrize("device", DEVICES)
def test_slot_and_pages_reused_after_release(device):
    """One slot, pool of one request: each request runs where the last one's matrices, convolution
    inputs, latents and keys still lie."""
    cfg = SMALL
    eng, full = build(cfg, device, max_num_seqs=1, max_kv_blocks=4)
    for i in range(3):
        t = tokens(70 + i, cfg["vocab"], 40 + i)
        check(run_schedule(eng, alone(t, [33, 2, 1, 1])), cfg, full, {"a": t})
    for n in (1, 2, 3):                                    # shorter than the taps
        t = tokens(n, cfg["vocab"], 45 + n)
        check(run_schedule(eng, alone(t, [1])), cfg, full, {"a": t})


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_over_page_and_window_edges(device):
    cfg = SMALL
    eng, full = build(cfg, device)
    t = tokens(140, cfg["vocab"], 50)
    check(run_schedule(eng, alone(t, [20] + [1] * 120)), cfg, full, {"a": t})


def _sharp(cfg, boost):
    """Weights with sharp scores (latent queries and the left side's query norm scaled up), so that
    a key that enters or leaves the view moves the logits visibly."""
    _, full = build(cfg, "cpu")
    full = dict(full)
    for i, ly in enumerate(cfg["layers"]):
        n = f"l{i}.mix.q" if ly["type"] == "latent_attention" else f"l{i}.mix.left.q.norm"
        full[n] = (full[n] * boost).bfloat16().float()
    return full


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size", [1, 2, 31, 32, 33, 64, 70])
def test_window_with_sharp_scores(device, size):
    """Windows of one key, at, just under and just over the page size and a multiple of it: one key
    more or less in view shows; prompt rows and decoded rows."""
    def cfg_of(n):
        return config([latent(2, 8, 8, 8, 16, n, None, scale=0.5),
                       latent(3, 8, 4, 8, 16, size + 1, dense(16), scale=0.5)], width=32, vocab=50)

    cfg = cfg_of(size)
    full = _sharp(cfg, 4.0)
    eng, _ = build(cfg, device, full=full)
    t = tokens(130, cfg["vocab"], 60 + size)
    got = run_schedule(eng, alone(t, [75, 2, 21] + [1] * 32))
    check(got, cfg, full, {"a": t})
    mine = torch.stack([got[("a", p)].double() for p in range(130)])
    # the mask matters: a window one key wider gives visibly other logits
    assert float((oracle.forward(cfg_of(size + 1), full, t) - mine).abs().max()) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_far_keys_over_many_pages(device):
    """A layer without window: sharp, capped scores over hundreds of keys across many pages, in a
    prompt and in decoding."""
    cfg = config([both(left(2, 1, 8, 8, 3, 4, softcap=9.0), right(1, 1, 8, 8, 2), dense(16)),
                  both(left(3, 3, 8, 8, 2, 8, softcap=6.0, scaling=yarn()), right(2, 1, 8, 8, 3), None)],
                 width=32, vocab=50, streams=2)
    full = _sharp(cfg, 3.0)
    eng, _ = build(cfg, device, full=full, max_kv_blocks=40, max_model_len=1024, max_batched_tokens=1024)
    t = tokens(400, cfg["vocab"], 77)
    got = run_schedule(eng, alone(t, [330, 2, 31] + [1] * 37))
    check(got, cfg, full, {"a": t})
    # the far past matters: another third token changes the last logits
    t2 = list(t)
    t2[3] = (t2[3] + 1) % cfg["vocab"]
    other = oracle.forward(cfg, full, t2)
    assert float((other[-1] - got[("a", 399)].double()).abs().max()) > 1e-4


def test_every_mechanism_shows_in_the_logits():
    """What the schedule tests rest on: a change of any one constant, in the oracle, moves the
    logits of the test models by far more than the tests' tolerance."""
    import copy

    t = tokens(60, SMALL["vocab"], 5)
    _, full = build(SMALL, "cpu")
    base = oracle.forward(SMALL, full, t)

    def moved(change, tensors=full):
        cfg = copy.deepcopy(SMALL)
        change(cfg)
        return float((oracle.forward(cfg, tensors, t) - base).abs().max() / base.abs().max())

    m = lambda c, i: c["layers"][i]["mixer"]               # noqa: E731
    changes = {
        "logit_scale": lambda c: c.update(logit_scale=0.9),
        "eps": lambda c: c["norm"].update(eps=1e-2),
        "left_scale": lambda c: m(c, 1).update(left_scale=0.8),
        "right_scale": lambda c: m(c, 1).update(right_scale=1.0),
        "scale": lambda c: m(c, 1)["left"].update(scale=0.5),
        "softcap": lambda c: m(c, 1)["left"].update(softcap=4.0),
        "left base": lambda c: m(c, 1)["left"]["rot"].update(base=900.0),
        "left dims": lambda c: m(c, 1)["left"]["rot"].update(dims=6),
        "left factor": lambda c: m(c, 1)["left"]["rot"]["scaling"].update(factor=4.0),
        "latent scale": lambda c: m(c, 0).update(scale=0.4),
        "latent window": lambda c: m(c, 0)["mask"].update(size=20),
        "latent base": lambda c: m(c, 0)["rot"].update(base=400.0),
        "latent original": lambda c: m(c, 0)["rot"]["scaling"].update(original=900),
        "latent slow": lambda c: m(c, 0)["rot"]["scaling"].update(slow=0.25),
        "latent fast": lambda c: m(c, 0)["rot"]["scaling"].update(fast=0.5),
    }
    for name, change in changes.items():
        assert moved(change) > 1e-3, name
    for name in full:
        if name == "l0.hc1.in":      # a factor on streams that are still equal: the norm takes it out
            continue
        other = dict(full)
        other[name] = full[name] * 0.8 + 0.05
        assert moved(lambda c: None, other) > 1e-4, name


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [SMALL, ODD], ids=["small", "odd"])
def test_bfloat16_close_to_oracle_and_independent_of_cuts(device, cfg):
    eng, full = build(cfg, device, dtype=torch.bfloat16)
    a, b = tokens(100, cfg["vocab"], 80), tokens(41, cfg["vocab"], 81)
    steps = [{"entries": [("a", a[:70], list(range(70))), ("b", b[:3], [0, 1, 2])], "end": []},
             {"entries": [("a", a[70:71], [0]), ("b", b[3:40], list(range(37)))], "end": []},
             {"entries": [("a", a[71:], list(range(29))), ("b", b[40:], [0])], "end": ["a", "b"]}]
    got = run_schedule(eng, steps)
    assert len(got) == 141
    ref = {"a": oracle.forward(cfg, full, a), "b": oracle.forward(cfg, full, b)}

    def err(row, want, std):
        d = row.double() - want.double()
        d = d - d.mean()
        return float(d.pow(2).mean().sqrt() / std)

    e = sorted(err(row, ref[n][p], ref[n].std()) for (n, p), row in got.items())
    assert e[len(e) // 2] < 0.05 and e[-8] < 0.15 and e[-1] < 0.4, (e[len(e) // 2], e[-8:])
    whole = run_schedule(eng, alone(a, []))
    e = sorted(err(whole[("a", p)], got[("a", p)], ref["a"].std()) for p in range(100))
    assert e[50] < 0.05 and e[-6] < 0.15 and e[-1] < 0.4, (e[50], e[-8:])


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_engine(device):
    """generate() (scheduler, sampler at temperature 0, decode steps) picks the oracle's tokens."""
    from replisense_rfq_amd.engine.sequence import SamplingParams

    cfg = SMALL
    eng, full = build(cfg, device)
    prompts = [tokens(n, cfg["vocab"], 70 + n) for n in (9, 35, 2)]
    seqs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, grammar=False))
    for p, s in zip(prompts, seqs):
        assert s.output_ids == oracle.greedy(cfg, full, p, 10)
    assert eng.core.num_free_state_slots == 4


@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_folder_round_trip(device, tmp_path):
    """config.json + model.safetensors written to a folder choose the model class and load."""
    import json

    from safetensors.torch import save_file

    from replisense_rfq_amd.engine.engine import LLMEngine
    from replisense_rfq_amd.utils.config import EngineConfig

    cfg = ODD if device == "cpu" else SMALL
    _, full = build(cfg, "cpu")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in full.items()},
              str(tmp_path / "model.safetensors"))
    eng = LLMEngine(EngineConfig(model="x", weights_path=str(tmp_path), dtype="float32", device=str(device),
                                 max_num_seqs=2, max_kv_blocks=8, max_batched_tokens=128,
                                 max_model_len=128, use_graphs=False, grammar=False,
                                 prefix_cache=False, warm_prefix=False, tune_gemm=False,
                                 jump_forward=False))
    assert type(eng.model).__name__ == "MineraxLM"
    t = tokens(20, cfg["vocab"], 5)
    check(run_schedule(eng, alone(t, [9, 2])), cfg, full, {"a": t})


def test_trace_replay_from_the_command_line(tmp_path):
    """bin/trace_run chooses the model by the folder's config.json and writes the wanted logits."""
    import json
    import os
    import subprocess

    import numpy as np
    from safetensors.torch import save_file

    cfg = SMALL
    _, full = build(cfg, "cpu")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in full.items()},
              str(tmp_path / "model.safetensors"))
    a, b = tokens(60, cfg["vocab"], 1), tokens(9, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]},
                                     {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [6]},
                                     {"id": "a", "tokens": a[40:], "want": [19]}], "end": ["a", "b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": b, "want": [8]}], "end": ["a"]}]    # name reused
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    p = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128", "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                       capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    ra, rb = oracle.forward(cfg, full, a), oracle.forward(cfg, full, b)
    for n, rows in {0: [ra[0], ra[39]], 1: [rb[8], ra[59]], 2: [rb[8]]}.items():
        got = np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"])
        for g, r in zip(got, rows):
            assert float(np.abs(g - r.numpy()).max() / r.abs().max()) < 3e-4


def test_named_configuration_and_registry():
    from replisense_rfq_amd.models import layered_model_class
    from replisense_rfq_amd.models.config import get_config

    c = get_config("tiny-minerax")
    assert c.architecture == "Minerax" and c.streams == 3
    assert layered_model_class("Minerax").__name__ == "MineraxLM"
    assert c.params() > 0
    m, lat = c.layers[0].mixer, c.layers[1].mixer
    a, b = m.parts
    assert c.kv_bytes_per_token() == 2 * (2 * a.kv_heads * (a.dim + a.vdim) + lat.kv_rank + lat.rot_dim)
    assert c.state_shapes(0) == {
        "0.conv": (a.conv - 1, a.heads * a.dim + a.kv_heads * (a.dim + a.vdim)),
        "1.S": (b.heads, b.dim, b.vdim),
        "1.conv": (b.conv - 1, 2 * b.kv_heads * b.dim + b.heads * b.vdim)}
    assert c.state_shapes(1) == {}


def test_configuration_errors():
    from replisense_rfq_amd.models.config import minerax_from_json

    ok = right(2, 1, 8, 8, 2)
    for layer in (both(left(3, 2, 8, 8, 2, 4), ok, None), both(left(2, 1, 8, 8, 0, 4), ok, None),
                  both(left(2, 1, 8, 8, 2, 10), ok, None), both(left(2, 1, 8, 8, 2, 3), ok, None),
                  both(left(2, 1, 8, 8, 2, 4), right(3, 2, 8, 8, 2), None),
                  latent(2, 8, 0, 8, 16, 5, None),
                  {"type": "attention", "mixer": {}, "mlp": None},
                  latent(2, 8, 4, 8, 16, 5, {"kind": "moe", "ff": 8})):
        with pytest.raises(ValueError):
            minerax_from_json(config([layer]))
    with pytest.raises(ValueError):
        minerax_from_json(config([latent(2, 8, 4, 8, 16, 5, None)], streams=0))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_decode_graphs_replayed_between_eager_steps(dtype):
    """Decode steps replay a captured hipGraph (streams, convolutions, both attentions and the
    recurrence inside it), prompts run eagerly in between: greedy generation of several waves of
    requests picks the oracle's tokens each time (fp32), and the graph was the path that ran."""
    from replisense_rfq_amd.engine.sequence import SamplingParams

    cfg = WIDE
    eng, full = build(cfg, "cuda:0", dtype=dtype, use_graphs=True, graph_buckets=(4,))
    assert eng.runner.graphs
    for wave in range(3):
        prompts = [tokens(n, cfg["vocab"], 100 + 10 * wave + n) for n in (9, 35, 2)]
        seqs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, grammar=False))
        if dtype == torch.float32:
            for p, s in zip(prompts, seqs):
                assert s.output_ids == oracle.greedy(cfg, full, p, 10), wave
    assert eng.runner.stats["graph_steps"] >= 24
    assert eng.core.num_free_state_slots == 4


@pytest.mark.gpu
def test_mfma_sized_model_in_bf16_against_fp32():
    """Head sizes of the MFMA tiles, bf16 on the GPU: prompts in portions (the first long enough
    for the recurrence's scan) and decoding, against the oracle."""
    cfg = WIDE
    eng, full = build(cfg, "cuda:0", dtype=torch.bfloat16, max_kv_blocks=40, max_model_len=640,
                      max_batched_tokens=1024)
    req = {"a": tokens(420, cfg["vocab"], 90), "b": tokens(130, cfg["vocab"], 91)}
    a, b = req["a"], req["b"]
    steps = [{"entries": [("a", a[:300], [5, 150, 299]), ("b", b[:100], [0, 99])], "end": []},
             {"entries": [("a", a[300:400], [0, 99]), ("b", b[100:101], [0])], "end": []}]
    steps += [{"entries": [("a", a[400 + i:401 + i], [0]), ("b", b[101 + i:102 + i], [0])], "end": []}
              for i in range(20)]
    ref = {n: oracle.forward(cfg, full, t) for n, t in req.items()}
    got = run_schedule(eng, steps)
    assert len(got) == 48
    e = []
    for (n, p), row in got.items():
        d = row.double() - ref[n][p]
        d = d - d.mean()
        e.append(float(d.pow(2).mean().sqrt() / ref[n].std()))
    e.sort()
    assert e[len(e) // 2] < 0.05 and e[-1] < 0.15, e[-6:]
