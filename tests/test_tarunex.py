"""Tarunex through the engine against the plain implementation.  Every test runs on the CPU
path (reference kernels, fp32) and, marked gpu, on the HIP kernels in fp32 and bf16."""
import json
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(__file__))
import tarunex_cases as sc  # noqa: E402
import plain_tarunex as plain  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
RUNS = [pytest.param(("cpu", "float32"), id="cpu"),
        pytest.param(("cuda", "float32"), id="gpu32", marks=pytest.mark.gpu),
        pytest.param(("cuda", "bfloat16"), id="gpu16", marks=pytest.mark.gpu)]
LIMIT = {"float32": 1e-4, "bfloat16": 0.06}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name, seed=0):
        if (name, seed) not in made:
            cfg = sc.CASES[name]
            W = sc.weights(cfg, seed)
            made[name, seed] = (cfg, W, sc.save(cfg, W, tmp_path_factory.mktemp(name)))
        return made[name, seed]

    return get


def check(models, name, schedule, run, **kw):
    """Replay a schedule; every position of every request equals the oracle's."""
    device, dtype = run
    cfg, W, path = models(name)
    got, rp = sc.replay(path, schedule, dtype, device, **kw)
    full: dict = {}
    for step in schedule:
        for i, t in step:
            full.setdefault(i, []).extend(t or [])
    for i, toks in full.items():
        e = sc.error(got[i], sc.oracle(name, cfg, W, toks))
        assert e < LIMIT[dtype], f"{name} {i}: {e:.2e}"
    return rp


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", sorted(sc.CASES))
def test_whole_prompt_and_decode(models, name, run):
    cfg = sc.CASES[name]
    t = sc.tokens(cfg, 150, 1)
    check(models, name, [[("a", t)]], run)  # one prefill step
    # prefill, then token by token past every page border
    check(models, name, [[("a", t[:30])]] + [[("a", [x])] for x in t[30:]], run)


@pytest.mark.parametrize("run", RUNS)
def test_residual_stream_of_every_layer_run(models, run):
    device, dtype = run
    cfg, W, path = models("mixed")
    from omnia_amd.engine.replay import TraceReplay

    rp = TraceReplay(path, dtype, 128, device)
    m, got = rp.engine.model, []
    layers = m.run_layers
    m.run_layers = lambda fb, kv: layers(fb, kv, got)
    t = sc.tokens(cfg, 70, 4)
    rp.step([{"id": "a", "tokens": t, "want": [69]}], [])
    want: list = []
    plain.forward(cfg, W, t, want)
    assert len(got) == len(want) == 6  # two layers run twice
    for i, (a, b) in enumerate(zip(got, want)):
        e = float((a.cpu().double() - b).norm() / b.norm())
        assert e < {"float32": 1e-5, "bfloat16": 0.03}[dtype], (i, e)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", sorted(sc.CASES))
def test_first_tokens(models, name, run):
    """A one-token prompt and every short length."""
    cfg = sc.CASES[name]
    t = sc.tokens(cfg, 9, 2)
    check(models, name, [[("a", [x])] for x in t], run)
    for n in (2, 3, 5):
        check(models, name, [[("a", t[:n])], [("a", t[n:])]], run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("sizes", [(2,), (3, 7), (16,), (31, 33, 1), (32, 64), (5, 2, 40)])
@pytest.mark.parametrize("name", ["mixed", "odd", "many"])
def test_portions(models, name, sizes, run):
    cfg = sc.CASES[name]
    t = sc.tokens(cfg, 131, 3)
    check(models, name, [[("a", p)] for p in sc.cut(t, sizes)], run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", ["mixed", "many", "wide"])
def test_batches_and_reuse(models, name, run):
    """Unequal requests together -- portions beside decoded tokens, requests left out of
    steps -- in a pool that makes pages be used again."""
    cfg = sc.CASES[name]
    T = {i: sc.tokens(cfg, n, 10 + k) for k, (i, n) in enumerate(
        [("a", 90), ("b", 41), ("c", 5), ("d", 70), ("e", 97), ("f", 33)])}
    sched = [[("a", T["a"][:50]), ("b", T["b"][:2])],
             [("b", T["b"][2:35]), ("c", T["c"][:1])],
             [("a", T["a"][50:51]), ("b", T["b"][35:36]), ("c", T["c"][1:2]), ("d", T["d"][:66])],
             [("a", T["a"][51:52]), ("d", T["d"][66:67]), ("c", T["c"][2:5])],
             [("d", T["d"][67:68]), ("a", T["a"][52:90]), ("b", T["b"][36:37])],
             [("a", None), ("c", None), ("b", T["b"][37:41])],
             [("b", None), ("e", T["e"][:80]), ("d", T["d"][68:69])],
             [("e", T["e"][80:81]), ("f", T["f"][:31]), ("d", T["d"][69:70])],
             [("d", None), ("f", T["f"][31:32]), ("e", T["e"][81:82])],
             [("f", T["f"][32:33]), ("e", T["e"][82:])]]
    rp = check(models, name, sched, run, max_tokens=320)
    bm = rp.engine.blocks
    held = sum(len(s.blocks) for s in rp.live.values())
    assert bm.num_free == bm.num_blocks - 1 - held
    for rid in list(rp.live):
        rp.step([], [rid])
    assert bm.num_free == bm.num_blocks - 1


@pytest.mark.parametrize("run", RUNS)
def test_long_decoding(models, run):
    cfg = sc.CASES["mixed"]
    t = sc.tokens(cfg, 330, 5)
    check(models, "mixed", [[("a", t[:3])]] + [[("a", [x])] for x in t[3:]], run)


@pytest.mark.gpu
@pytest.mark.parametrize("run", RUNS[1:])
def test_long_prompt(models, run):
    """A prompt long enough for the prefill tile GEMMs (bf16), whole, beside another one and
    in portions; then decoding."""
    cfg = sc.CASES["tile"]
    t, u = sc.tokens(cfg, 2300, 20), sc.tokens(cfg, 1900, 21)
    check(models, "tile", [[("a", t[:2270])]] + [[("a", [x])] for x in t[2270:]], run,
          max_tokens=2432)
    check(models, "tile", [[("a", t[:1100]), ("b", u[:1000])],
                           [("a", t[1100:]), ("b", u[1000:1001])], [("b", u[1001:])]], run,
          max_tokens=4608)


@pytest.mark.gpu
@pytest.mark.parametrize("run", RUNS[1:])
def test_two_streams(models, run, monkeypatch):
    """Sublayers side by side give what they give one after another: a long prompt, then
    replays of decode graphs with eager steps between."""
    from omnia_amd.models import hybrid

    cfg = sc.CASES["tile"]
    t, u = sc.tokens(cfg, 1130, 30), sc.tokens(cfg, 40, 31)
    sched = [[("a", t[:1100])]]
    for k, x in enumerate(t[1100:]):
        sched.append([("a", [x])] + ([("b", u[k:k + 2])] if k % 7 == 0 else []))
    got = []
    for rows, span in ((256, (1024, 8192)), (0, (1, 0))):
        monkeypatch.setattr(hybrid, "FORK_DECODE", rows)
        monkeypatch.setattr(hybrid, "FORK_PREFILL", span)
        z, rp = sc.replay(models("tile")[2], sched, run[1], run[0], max_tokens=1280)
        assert rp.engine.runner.stats["graph_replays"] >= 20
        got.append(z)
    for i in "ab":
        assert sc.error(got[0][i], got[1][i].double()) < 1e-6


@pytest.mark.parametrize("run", RUNS)
def test_rows_do_not_depend_on_their_batch(models, run):
    """The same prompt and decoded tokens, alone and in a full batch of strangers."""
    device, dtype = run
    cfg, W, path = models("mixed")
    t = sc.tokens(cfg, 45, 70)
    alone, _ = sc.replay(path, [[("a", t[:40])]] + [[("a", [x])] for x in t[40:]], dtype, device)
    other = {k: sc.tokens(cfg, 80, 71 + n) for n, k in enumerate("bcd")}
    sched = [[(k, o[:11 + 9 * n]) for n, (k, o) in enumerate(other.items())] + [("a", t[:40])]]
    for j, x in enumerate(t[40:]):
        step = [(k, o[11 + 9 * n + j * 7:11 + 9 * n + (j + 1) * 7] if n == 1 else
                 o[11 + 9 * n + j:12 + 9 * n + j]) for n, (k, o) in enumerate(other.items())]
        sched.append(step[:1] + [("a", [x])] + step[1:])
    mixed, _ = sc.replay(path, sched, dtype, device)
    assert sc.error(mixed["a"], alone["a"].double()) < {"float32": 2e-5, "bfloat16": 0.05}[dtype]


def greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(plain.forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


def engine(path, device, dtype="float32", **kw):
    from omnia_amd.engine.engine import EngineConfig, LLMEngine

    kw = {**dict(block_size=16, max_batch=4, max_model_len=256, num_blocks=40), **kw}
    return LLMEngine(EngineConfig(model="m", checkpoint=path, device=device, dtype=dtype, **kw))


def sampling(n, **kw):
    from omnia_amd.engine.sampling_params import SamplingParams

    return SamplingParams(temperature=0.0, max_tokens=n, ignore_eos=True, **kw)


@pytest.mark.parametrize("run", RUNS[:2])
@pytest.mark.parametrize("graphs", ["sync", "pipelined"])
@pytest.mark.parametrize("name", ["mixed", "odd", "many"])
def test_greedy_generation(models, name, graphs, run, monkeypatch):
    """The engine's entry point and scheduler: chunked prefill, mixed steps, more requests
    than the batch holds; on the CPU the pipelined loop runs on simulated graphs."""
    if graphs == "pipelined":
        monkeypatch.setenv("OMNIA_SIM_GRAPHS", "1")
    cfg, W, path = models(name)
    eng = engine(path, run[0], use_graphs=graphs == "pipelined", max_prefill_tokens=48,
                 max_batch=3, share_prefix=graphs == "pipelined")
    prompts = [sc.tokens(cfg, n, 40 + n) for n in (1, 60, 17, 33, 5)]
    seqs = eng.generate(prompts, sampling(10))
    for p, s in zip(prompts, seqs):
        assert s.output == greedy(cfg, W, p, 10)
    if graphs == "sync":  # no page is kept for a later prompt to share
        assert eng.blocks.num_free == eng.blocks.num_blocks - 1
    if run[0] == "cuda" and graphs == "pipelined":
        # nothing but kernels, copies and library GEMMs in the decode graph
        assert eng.runner.stats["captures"] and not eng.runner.stats["capture_guard_violations"]


@pytest.mark.parametrize("run", RUNS[:2])
def test_sessions_and_shared_prefixes(models, run):
    """No layer has a state: a session's next turn continues from the parked pages of every
    pass, whatever part of them it shares, and requests share prefixes across sessions."""
    cfg, W, path = models("mixed")
    eng = engine(path, run[0], use_graphs=False, max_batch=2)
    assert not eng.model_cfg.stateful
    p = sc.tokens(cfg, 50, 60)
    a = eng.generate([p], sampling(6), session_ids=["s"])[0]
    turn2 = p + a.output + sc.tokens(cfg, 4, 61)
    b = eng.generate([turn2], sampling(5), session_ids=["s"])[0]
    assert b.prefix_hit >= len(p) + 5 and b.output == greedy(cfg, W, turn2, 5)
    other = p[:40] + sc.tokens(cfg, 9, 62)
    c = eng.generate([other], sampling(5), session_ids=["s"])[0]
    assert c.prefix_hit >= 32 and c.output == greedy(cfg, W, other, 5)


@pytest.mark.parametrize("run", RUNS[:2])
def test_swapped_session(models, run):
    """An evicted session's pages come back from the host tier."""
    cfg, W, path = models("mixed")
    eng = engine(path, run[0], use_graphs=False, max_batch=1, num_blocks=8, max_model_len=112,
                 swap_gib=0.01, share_prefix=False)
    # six layer runs: key and value pages of three, latent pages of the others
    assert len(eng.kv.page_tensors()) == 3 * 2 + 3 and not eng.kv.state_tensors()
    p = sc.tokens(cfg, 50, 80)
    a = eng.generate([p], sampling(6), session_ids=["s"])[0]
    q = sc.tokens(cfg, 60, 81)
    assert eng.generate([q], sampling(4), session_ids=["t"])[0].output == greedy(cfg, W, q, 4)
    assert eng.blocks.stats["swap_out"] == 1
    turn2 = p + a.output + sc.tokens(cfg, 3, 82)
    b = eng.generate([turn2], sampling(5), session_ids=["s"])[0]
    assert eng.blocks.stats["swap_in"] == 1 and b.prefix_hit >= 55
    assert b.output == greedy(cfg, W, turn2, 5)


@pytest.mark.parametrize("run", RUNS[:2])
def test_preempted_sequence_recomputes(models, run):
    cfg, W, path = models("mixed")
    eng = engine(path, run[0], use_graphs=False, max_batch=3, num_blocks=8)
    prompts = [sc.tokens(cfg, 28, 90 + k) for k in range(3)]
    seqs = eng.generate(prompts, sampling(12))
    assert sum(s.preemptions for s in seqs) > 0
    for p, s in zip(prompts, seqs):
        assert s.output == greedy(cfg, W, p, 12)


def test_config_and_loader_errors(models, tmp_path):
    from omnia_amd.models.loader import config_from_hf, load_checkpoint

    cfg, W, path = models("mixed")
    mc = config_from_hf(path)
    assert mc.arch == "tarunex" and not mc.stateful and mc.num_layers == 6
    assert mc.logit_scale == cfg["logit_scale"] and mc.logit_softcap == cfg["logit_softcap"]
    assert mc.embed_scale == cfg["embedding"]["scale"] and not mc.tie_embeddings
    assert [l.weights_of for l in mc.layers] == [None, None, None, 1, 2, None]
    assert [l.starts for l in mc.layers] == [None, 0, None, 1, None, None]
    assert [l.mixer.kind for l in mc.layers] == [
        "attention", "attention", "latent_attention"] + ["attention"] + 2 * ["latent_attention"]
    a = mc.layers[1].mixer
    assert (a.softcap, a.sink, a.bias, a.gate, a.rotary) == (5.0, "zero", "qkv", True, None)
    # a looped layer keeps keys and values, or latents, per pass
    assert mc.kv_bytes_per_token(2) == 2 * (2 * (32 + 64) + 2 * (64 + 32) + 96 + 96 + 128)
    assert mc.num_params() == sum(t.numel() for t in W.values())
    bad = {k: v for k, v in W.items() if k != "l1.mix.r2"}
    with pytest.raises(ValueError, match="l1.mix.r2 is missing"):
        load_checkpoint(sc.save(cfg, bad, tmp_path / "a"), mc)
    bad = {**W, "loop.step": W["loop.step"][:1]}
    with pytest.raises(ValueError, match="loop.step"):
        load_checkpoint(sc.save(cfg, bad, tmp_path / "b"), mc)

    def edited(edit):
        c = json.loads(json.dumps(cfg))
        edit(c)
        return sc.save(c, {"x": W["embed"]}, tmp_path / "c")

    for edit, what in (
            (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "6 heads over 4"),
            (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "softcap -1"),
            (lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=0), "q_temp"),
            (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=6), "rot.dims 6"),
            (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top 7 of 6"),
            (lambda c: c["loop"].update(stop=5), "loop 1 .. 5"),
            (lambda c: c["layers"][1]["mlp"].update(kind="dense"), "unknown feed-forward"),
            (lambda c: c["layers"][1].update(type="delta"), "unknown mixer")):
        with pytest.raises(ValueError, match=what):
            config_from_hf(edited(edit))


def _run_cli(path, out, steps, extra, dtype="float32"):
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "256", *extra],
                       input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                       capture_output=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    return [x for x in p.stdout.splitlines() if x.startswith("done ")]


@pytest.mark.parametrize("run", RUNS)
def test_trace_run_program(models, tmp_path, run):
    import numpy as np

    cfg, W, path = models("mixed")
    t = sc.tokens(cfg, 40, 7)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:30], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": t[30:31], "want": [0]},
                                     {"id": "y", "tokens": t[:5], "want": [4, 1]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": t[31:], "want": [8]}], "end": ["x"]}]
    done = _run_cli(path, tmp_path, steps, ["--device", run[0]], run[1])
    assert done == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "0.f32").exists()
    want = sc.oracle("mixed", cfg, W, t)
    short = sc.oracle("mixed", cfg, W, t[:5])
    got = {k: torch.from_numpy(np.fromfile(tmp_path / f"{k}.f32", "<f4")).view(-1, cfg["vocab"])
           for k in (1, 2)}
    assert sc.error(got[1], torch.stack([want[30], short[4], short[1]])) < LIMIT[run[1]]
    assert sc.error(got[2], want[39:40]) < LIMIT[run[1]]


@pytest.mark.parametrize("run", RUNS[:2])
def test_generate_command(models, run, capsys):
    """``omnia generate`` on a checkpoint folder."""
    from omnia_amd.cli import main

    cfg, W, path = models("mixed")
    t = sc.tokens(cfg, 19, 8)
    main(["generate", "--checkpoint", path, "--tokens", ",".join(map(str, t)), "--max-tokens", "7",
          "--dtype", "float32", "--device", run[0], "--ignore-eos", "--max-model-len", "128",
          "--num-blocks", "32"])
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["tokens"] == greedy(cfg, W, t, 7) and out["prompt_tokens"] == 19


@pytest.mark.parametrize("run", RUNS)
def test_registered_preset_and_sampling(run):
    """The registry's random-init preset generates through the sampler; a seed repeats."""
    from omnia_amd.engine.engine import EngineConfig, LLMEngine
    from omnia_amd.engine.sampling_params import SamplingParams
    from omnia_amd.models.config import resolve

    for n, like in (("tarunex-3b", "sekazen-3b"), ("tarunex-8b", "sivadra-8b")):
        assert resolve(n).num_layers == resolve(like).num_layers
    tiny = resolve("tiny-tarunex")
    assert tiny.num_layers == 6 and [l.weights_of for l in tiny.layers] == [
        None, None, None, 1, 2, None]
    assert [l.starts for l in tiny.layers] == [None, 0, None, 1, None, None]
    eng = LLMEngine(EngineConfig(model="tiny-tarunex", device=run[0], dtype=run[1],
                                 num_blocks=40, max_batch=4, max_model_len=256,
                                 use_graphs=run[0] == "cuda"))
    p = SamplingParams(temperature=0.8, top_k=20, max_tokens=6, ignore_eos=True, seed=5)
    a, b = eng.generate(["hello there", "hello there"], p)
    assert len(a.output) == 6 and all(0 <= t < 512 for t in a.output)
    if run[0] == "cuda":
        if run[1] == "float32":  # one seed, one result, whatever the row
            assert a.output == b.output
        # nothing but kernels, copies and library GEMMs in the decode graph
        assert eng.runner.stats["captures"] and not eng.runner.stats["capture_guard_violations"]


@pytest.mark.parametrize("run", RUNS[:2])
def test_design_comparison(run):
    """The benchmark's comparison of the design with the closest family, at toy size."""
    from omnia_amd.engine import design_bench

    r = design_bench.run("tarunex", run[0], [("tiny-tarunex", "tiny-sekazen")], [(2, 40)],
                         [(2, 20)], reps=1, steps=4)
    assert [x["model"] for x in r["rows"]] == ["tiny-tarunex", "tiny-sekazen"]
    assert all(x["prefill_tok_s"]["2x40"] > 0 and x["decode_step_ms"]["b2@20"] > 0
               for x in r["rows"])
