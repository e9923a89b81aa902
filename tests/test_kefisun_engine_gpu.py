"""Models of the Kefisun design in the engine against the plain implementation: whole prompts, prefill against
token-by-token decoding, portions down to two tokens, batches of unequal requests with pages and state slots used
again, long decoding past every window, keys at a window's edge that carry the weight, the first tokens of a sequence,
random configurations, greedy generation through the serving engine and its scheduler, and the command lines.  The
configurations are the tests' own (``kefisun_models``)."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import kefisun_models as models
import traces
from plain import kefisun_plain as plain
from tolerances import BF16_REL_MEAN, BF16_REL_WORST, F32_TOL

pytestmark = pytest.mark.gpu

LENGTHS = {"main": [70, 41, 3, 55, 1, 26, 64], "odd": [45, 33, 2, 70, 17], "wide": [38, 9, 61, 1, 24]}
PAGE = {"main": 8, "odd": 4, "wide": 16}


def _engine(folder, dtype, pages, page, max_live=4):
    from zedinfer_amd.config import SchedulerConfig
    from zedinfer_amd.engine import Engine
    return Engine.from_folder(folder, dtype, SchedulerConfig(num_kv_blocks=pages, kv_block_size=page,
                                                             max_batch_requests=max_live, max_batch_tokens=4096,
                                                             max_seq_len=4096))


def _plain(folder):
    cfg, w = plain.load_folder(folder)
    return lambda toks: plain.forward(cfg, w, toks).float()


def _setup(tmp_path, name, dtype, pages, max_live=4, seed=0):
    folder = models.write_model(str(tmp_path / name), name, seed=seed,
                                dtype=torch.float32 if dtype == "float32" else torch.bfloat16)
    return _plain(folder), _engine(folder, dtype, pages, PAGE[name], max_live)


def _rows(steps, out):
    """((request, position), row of logits) of every written row."""
    fed = {}
    for st in steps:
        row = 0
        for e in st["entries"]:
            base = fed.get(e["id"], 0)
            for w in e["want"]:
                yield (e["id"], base + w), out[st["step"]][row]
                row += 1
            fed[e["id"]] = base + len(e["tokens"])
        for rid in st["end"]:
            fed.pop(rid, None)


def _check(steps, out, ref, dtype, what):
    """Every written row against the plain logits at (request, position); returns the rows compared."""
    worst = mean = scale = 0.0
    n = 0
    for (rid, pos), got in _rows(steps, out):
        r = ref[rid][pos].numpy()
        d = np.abs(got - r)
        worst, mean, scale, n = max(worst, float(d.max())), mean + float(d.mean()), max(scale, float(np.abs(r).max())), n + 1
    if dtype == "float32":
        assert worst <= F32_TOL * max(1.0, scale), (what, worst, scale)
    else:
        assert worst <= BF16_REL_WORST * scale and mean / n <= BF16_REL_MEAN * scale, (what, worst, mean / n, scale)
    return n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["main", "odd", "wide"])
def test_every_way_of_cutting_and_batching_gives_the_plain_logits(tmp_path, name, dtype):
    vocab = models.CONFIGS[name]["vocab"]
    requests = {f"r{i}": traces.random_tokens(vocab, n, seed=40 + i) for i, n in enumerate(LENGTHS[name])}
    ps = PAGE[name]
    # so few pages that the batches use them again: four live requests of the longest kind, and one page more
    pages = 4 * (-(-max(LENGTHS[name]) // ps) + 1) + 1
    forward, engine = _setup(tmp_path, name, dtype, pages)
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    total = sum(len(t) for t in requests.values())
    takes = [g.pool.takes for g in engine.cache.groups]
    for what, steps in (("whole", traces.whole(requests)), ("decode", traces.last_decoded(requests, tail=30)),
                        ("portions", traces.portions(requests, seed=1)),
                        ("portions of two", traces.portions(requests, seed=2, sizes=(2, 2, 3, 2, 1, 2))),
                        ("mixed", traces.mixed(requests, max_live=4, seed=3)),
                        ("mixed, three live", traces.mixed(requests, max_live=3, seed=4, decode_tail=20, max_portion=9))):
        out = traces.run_in_process(engine, steps)
        assert _check(steps, out, ref, dtype, what) == total
    for what, steps in (("last rows", traces.few_wanted(traces.mixed(requests, max_live=4, seed=5), seed=5)),
                        ("random rows", traces.random_wanted(traces.mixed(requests, max_live=4, seed=6), seed=6))):
        out = traces.run_in_process(engine, steps)
        _check(steps, out, ref, dtype, what)
    engine.cache.check()
    assert not engine.cache.live
    for g, before in zip(engine.cache.groups, takes):
        assert g.pool.takes - before > g.pool.total          # pages went round
    assert engine.cache.slots.takes > 4 * len(requests)       # and so did the state slots


def test_in_float32_every_cut_gives_the_same_logits_within_rounding(tmp_path):
    """A position's logits do not depend on the cut, the batch, the pages or the slots beyond float32 rounding."""
    vocab = models.MAIN["vocab"]
    requests = {f"b{i}": traces.random_tokens(vocab, n, seed=140 + i) for i, n in enumerate([33, 150, 6])}
    forward, engine = _setup(tmp_path, "main", "float32", pages=96)
    rows = {}
    for steps in (traces.whole(requests), traces.portions(requests, seed=3, sizes=(2, 5, 1, 7)), traces.mixed(requests, max_live=3, seed=9)):
        for key, row in _rows(steps, traces.run_in_process(engine, steps)):
            rows.setdefault(key, []).append(row.copy())
    assert len(rows) == 33 + 150 + 6
    for key, got in rows.items():
        assert len(got) == 3
        scale = max(1.0, float(np.abs(got[0]).max()))
        assert all(float(np.abs(o - got[0]).max()) <= 2e-5 * scale for o in got[1:]), key


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_past_every_window(tmp_path, dtype):
    """A short prompt and then 300 tokens one by one: the windows of 9, 20 and 33 pass many times, their pages come
    back, state and tails are carried 300 times."""
    toks = traces.random_tokens(models.MAIN["vocab"], 310, seed=7)
    forward, engine = _setup(tmp_path, "main", dtype, pages=44)
    ref = {"long": forward(toks)}
    from zedinfer_amd.engine import StepEntry
    seq = engine.open("held")
    engine.step([StepEntry(seq, toks[:300], [])])
    assert all(g.kind == "window" for g in engine.cache.groups) and len(engine.cache.groups) == 3
    assert all(seq.held[gi] <= 33 // 8 + 2 for gi in range(3))            # of 38 pages' worth of tokens
    engine.close(seq)
    steps = traces.last_decoded({"long": toks}, tail=300)
    assert _check(steps, traces.run_in_process(engine, steps), ref, dtype, "long decoding") == 310
    engine.cache.check()


def _loud_model(tmp_path, window, dtype, slope=0.2):
    """One attention layer whose query of token 1 points at token 2's key with a large weight (every other query and
    key is nothing): a prompt of token-0 filler with a single token 2 makes that position carry the weight whenever it
    is visible.  No tap of any convolution but the present token's."""
    W = 32
    cfg = dict(architecture="Kefisun", width=W, vocab=8, norm=dict(eps=1e-6), canon=dict(taps=2), embedding=dict(scale=1.0),
               logit_scale=1.0,
               layers=[dict(type="attention", mixer=dict(heads=1, kv_heads=1, dim=16, vdim=16, conv=2, scale=1.0, v_mix=True,
                                                         mask=dict(size=window)), mlp=None)])
    w = models.make_weights(cfg, seed=3)
    E = torch.zeros((8, W))
    for t in range(8):
        E[t, t] = 4.0
        E[t, 8 + t] = 1.0
    w["embed"] = E
    w["l0.norm1"], w["final.norm"], w["l0.canon1"] = torch.zeros(W), torch.zeros(W), torch.zeros((W, 2))
    q, k, v = torch.zeros((16, W)), torch.zeros((16, W)), torch.zeros((16, W))
    q[0, 1] = k[0, 2] = 30.0
    for t in range(8):
        v[t, t] = 3.0    # the value names the token
    w["l0.mix.q"], w["l0.mix.k"], w["l0.mix.v"] = q, k, v
    now = torch.zeros((16, 2))
    now[:, 1] = 1.0
    for x in ("q", "k", "v"):
        w[f"l0.mix.{x}.conv"] = now
    w["l0.mix.q.norm"], w["l0.mix.k.norm"] = torch.ones(16), torch.ones(16)
    w["l0.mix.r1"], w["l0.mix.r2"] = torch.tensor([slope]), torch.tensor([1.0])
    w["l0.mix.o"] = torch.randn((W, 16), generator=torch.Generator().manual_seed(5))
    folder = models.write_config(str(tmp_path / f"loud_{window}"), cfg,
                                 {n: t.to(torch.float32 if dtype == "float32" else torch.bfloat16) for n, t in w.items()})
    return folder


@pytest.mark.parametrize("window, page", [(6, 4), (8, 8), (70, 16)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_just_inside_and_just_outside_the_window(tmp_path, window, page, dtype):
    """The loud key stands at a chosen distance from the asking token: in the window's last place it takes the softmax,
    one further it is not seen; in prompts, in portions and decoded one by one, also where the loud key is a sequence's
    first token or stands at a page's border."""
    folder = _loud_model(tmp_path, window, dtype)
    forward, engine = _plain(folder), _engine(folder, dtype, pages=64, page=page)
    seen = {}
    for at in (0, 1, page - 1, page, page + 1):
        for gap in (1, window - 2, window - 1, window, window + 1):
            toks = [0] * (at + gap + 1)
            toks[at], toks[-1] = 2, 1
            ref = {"p": forward(toks)}
            for what, steps in (("whole", traces.whole({"p": toks})), ("decoded", traces.last_decoded({"p": toks}, tail=gap + 1)),
                                ("portions", traces.portions({"p": toks}, seed=at + gap, sizes=(2, 3, 5, 2)))):
                _check(steps, traces.run_in_process(engine, steps), ref, dtype, (what, at, gap))
            seen[(at, gap)] = ref["p"][-1]
    for at in (0, page):
        assert float((seen[(at, window - 1)] - seen[(at, window)]).abs().max()) > 0.5
        assert float((seen[(at, window)] - seen[(at, window + 1)]).abs().max()) < 0.05


def test_the_distance_takes_from_a_score(tmp_path):
    """Two loud keys in the window: with a steep slope the nearer one takes the softmax whatever the cut."""
    folder = _loud_model(tmp_path, 30, "float32", slope=6.0)
    forward, engine = _plain(folder), _engine(folder, "float32", pages=64, page=8)
    toks = [0] * 30
    toks[3], toks[20], toks[-1] = 2, 2, 1
    ref = {"p": forward(toks)}
    for steps in (traces.whole({"p": toks}), traces.last_decoded({"p": toks}, tail=12), traces.portions({"p": toks}, sizes=(2, 7, 3))):
        _check(steps, traces.run_in_process(engine, steps), ref, "float32", "two loud keys")
    far = list(toks)
    far[3] = 0
    assert float((forward(far)[-1] - ref["p"][-1]).abs().max()) < 0.2      # the far one hardly counts


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations_in_float32(tmp_path, seed):
    cfg = models.random_config(100 + seed)
    folder = models.write_config(str(tmp_path / "m"), cfg, models.make_weights(cfg, seed))
    forward, engine = _plain(folder), _engine(folder, "float32", pages=80, page=[4, 8, 16][seed % 3])
    requests = {f"q{i}": traces.random_tokens(cfg["vocab"], n, seed=seed * 10 + i) for i, n in enumerate([37, 5, 58, 1])}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    for what, steps in (("whole", traces.whole(requests)), ("mixed", traces.mixed(requests, max_live=3, seed=seed)),
                        ("portions", traces.portions(requests, seed=seed, sizes=(2, 9, 1, 4)))):
        _check(steps, traces.run_in_process(engine, steps), ref, "float32", (what, json.dumps(cfg)))
    engine.cache.check()


@pytest.mark.parametrize("seed", range(4))
def test_random_configurations_in_bfloat16(tmp_path, seed):
    cfg = models.random_config(200 + seed)
    folder = models.write_config(str(tmp_path / "m"), cfg, models.make_weights(cfg, seed, torch.bfloat16))
    forward, engine = _plain(folder), _engine(folder, "bfloat16", pages=80, page=16)
    requests = {f"q{i}": traces.random_tokens(cfg["vocab"], n, seed=seed * 10 + i) for i, n in enumerate([37, 5, 141, 1])}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    for what, steps in (("whole", traces.whole(requests)), ("mixed", traces.mixed(requests, max_live=3, seed=seed)),
                        ("portions", traces.portions(requests, seed=seed, sizes=(2, 9, 70, 4)))):
        _check(steps, traces.run_in_process(engine, steps), ref, "bfloat16", (what, json.dumps(cfg)))


@pytest.mark.parametrize("kind", ["attention", "channel_delta"])
def test_models_of_one_kind_of_layer_alone(tmp_path, kind):
    """Attention layers alone (such a model's steps may be padded to recurring shapes) and recurrent layers alone (no
    pages at all), decoded and in portions that come again and again, so that recorded steps are replayed."""
    cfg = dict(models.MAIN, layers=[l for l in models.MAIN["layers"] if l["type"] == kind])
    folder = models.write_config(str(tmp_path / "m"), cfg, models.make_weights(cfg, 5, torch.bfloat16))
    forward, engine = _plain(folder), _engine(folder, "bfloat16", pages=128, page=8)
    assert engine.model.padding_safe() == (kind == "attention") and engine.model.tape_safe()
    requests = {f"q{i}": traces.random_tokens(cfg["vocab"], n, seed=60 + i) for i, n in enumerate([70, 66, 90, 75, 64, 68, 71])}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    for steps in (traces.last_decoded(requests, tail=20), traces.portions(requests, seed=1, sizes=(30, 9)),
                  traces.mixed(requests, max_live=4, seed=2, decode_tail=40, max_portion=30), traces.last_decoded(requests, tail=20)):
        _check(steps, traces.run_in_process(engine, steps), ref, "bfloat16", kind)
    engine.cache.check()


def test_greedy_generation_through_the_serving_engine(tmp_path):
    """Requests of unequal lengths through ``InferenceEngine`` and its scheduler (prompts cut into portions of 16
    tokens beside decoding requests), more of them than state slots, and the command line: in float32 the tokens are
    the plain implementation's."""
    from zedinfer_amd import GenerationConfig, InferenceEngine, SchedulerConfig
    folder = models.write_model(str(tmp_path / "main"), "main", seed=2)
    cfg, w = plain.load_folder(folder)
    prompts = [traces.random_tokens(cfg["vocab"], n, seed=300 + i) for i, n in enumerate([30, 7, 52, 1, 19])]
    want = [plain.greedy_generate(cfg, w, p, 12) for p in prompts]
    ie = InferenceEngine.create(folder, "float32", SchedulerConfig(num_kv_blocks=64, kv_block_size=8,
                                                                   max_batch_requests=3, max_prefill_tokens=16))
    got = [r.output_ids for r in ie.generate(prompts, GenerationConfig(max_new_tokens=12, ignore_eos=True))]
    assert got == want
    r = subprocess.run([sys.executable, os.path.join(traces.ROOT, "bin", "ping"), folder, "--dtype", "fp32", "--prompt-ids",
                        ",".join(map(str, prompts[1])), "--max-new-tokens", "6", "--ignore-eos", "--num-kv-blocks", "32",
                        "--kv-block-size", "8", "--no-log-to-console"], capture_output=True, text=True, timeout=600,
                       env=dict(os.environ, PYTHONPATH=traces.ROOT))
    assert r.returncode == 0, r.stderr
    assert "output_ids: " + ",".join(map(str, want[1][:6])) in r.stdout, r.stdout


def test_the_replay_tool_runs_a_model_of_the_design(tmp_path):
    folder = models.write_model(str(tmp_path / "odd"), "odd", seed=4)
    forward = _plain(folder)
    requests = {f"t{i}": traces.random_tokens(150, n, seed=500 + i) for i, n in enumerate([40, 3, 66, 21, 9])}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    steps = traces.mixed(requests, max_live=4, seed=11)
    out = traces.run_tool(folder, "float32", steps, str(tmp_path / "out"), traces.max_live_tokens(steps))
    assert _check(steps, out, ref, "float32", "replay tool") == sum(len(t) for t in requests.values())


def test_command_lines_take_a_model_of_the_design(tmp_path):
    """random_model writes a folder from the design's config.json (the engine's own random weights), ping generates from
    it what the plain implementation generates, batch_bench runs its scheduler over it."""
    root = traces.ROOT
    env = dict(os.environ, PYTHONPATH=root)
    run = lambda *a: subprocess.run([sys.executable, *a], capture_output=True, text=True, env=env, timeout=300,  # noqa: E731
                                    cwd=str(tmp_path))
    (tmp_path / "cfg").mkdir()
    with open(tmp_path / "cfg" / "config.json", "w") as f:
        json.dump(models.ODD, f)
    folder = str(tmp_path / "made")
    r = run(os.path.join(root, "bin", "random_model"), str(tmp_path / "cfg"), folder, "--seed", "5", "--dtype", "float32", "--std", "0.1", "--noisy-norms")
    assert r.returncode == 0, r.stderr + r.stdout
    cfg, w = plain.load_folder(folder)
    assert set(w) == set(models.tensor_shapes(models.ODD))
    prompt = traces.random_tokens(models.ODD["vocab"], 27, seed=3)
    r = run(os.path.join(root, "bin", "ping"), folder, "--dtype", "fp32", "--prompt-ids", ",".join(map(str, prompt)),
            "--max-new-tokens", "6", "--ignore-eos", "--num-kv-blocks", "32", "--kv-block-size", "8", "--no-log-to-console")
    assert r.returncode == 0, r.stderr
    want = plain.greedy_generate(cfg, w, prompt, 6)
    assert "output_ids: " + ",".join(map(str, want)) in r.stdout, r.stdout
    r = run(os.path.join(root, "bin", "batch_bench"), str(tmp_path / "cfg"), "-b", "3", "-p", "20", "-d", "6", "--num-kv-blocks",
            "64", "--kv-block-size", "8", "--random-weights", "--seed", "4", "--no-log-to-console")
    assert r.returncode == 0 and "18 tokens generated" in r.stdout, r.stderr + r.stdout
