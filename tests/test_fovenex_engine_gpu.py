"""Models of the Fovenex design in the engine against the plain implementation: whole prompts, prefill against
token-by-token decoding, portions down to two tokens, batches of unequal requests with pages used
again, long decoding past every window, keys at a window's edge that carry the weight, the first tokens of a sequence,
random configurations, layers that read another's latents, greedy generation through the serving engine and its scheduler, and the command lines.  The
configurations are the tests' own (``fovenex_models``)."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import fovenex_models as models
import traces
from plain import fovenex_plain as plain
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
    """A short prompt and then 300 tokens one by one: the windows of 9, 20, 33 and 50 pass many times; a cache that two layers
    read holds the wider of their windows, and its pages come back."""
    toks = traces.random_tokens(models.MAIN["vocab"], 310, seed=7)
    forward, engine = _setup(tmp_path, "main", dtype, pages=44)
    ref = {"long": forward(toks)}
    from zedinfer_amd.engine import StepEntry
    seq = engine.open("held")
    engine.step([StepEntry(seq, toks[:300], [])])
    held = {(g.kind, g.window): seq.held[gi] for gi, g in enumerate(engine.cache.groups)}
    assert set(held) == {("full", 0), ("window", 20), ("window", 50)}      # 33, 9 and 50 read one cache
    assert held[("full", 0)] == 38 and held[("window", 20)] <= 20 // 8 + 2 and held[("window", 50)] <= 50 // 8 + 2
    engine.close(seq)
    steps = traces.last_decoded({"long": toks}, tail=300)
    assert _check(steps, traces.run_in_process(engine, steps), ref, dtype, "long decoding") == 310
    engine.cache.check()


# ---- keys that carry the weight ---------------------------------------------------------------------------------------
def _loud_table(W):
    """Token t's row: a number of its own at t (asking, loud) and again at 8 + t (what its value names); its mean is zero, so
    the layer norm only scales it."""
    E = torch.zeros((8, W))
    for t in range(8):
        E[t, t], E[t, 8 + t] = 4.0, 1.0
        E[t, 16:] = -5.0 / (W - 16)
    return E


def _loud_window_model(tmp_path, window, reads_wider, dtype):
    """One layer of latent attention (or a second one that reads the first's latents through a wider or narrower window) whose
    query of token 1 points at token 2's key with a large weight, every other score being nothing: a prompt of token-0 filler
    with a single token 2 makes that position carry the weight whenever it is visible.  ``reads_wider``: None, or the window
    of the first layer when the second, which has ``window``, reads its latents (the first layer's result is not used)."""
    W = 48
    layer = lambda win, src=None: models._layer("latent_attention", models._latent(1, 16, 8, 16, 24, 8, 1.0, win, kv_from=src))      # noqa: E731
    layers = [layer(window)] if reads_wider is None else [layer(reads_wider), layer(window, 0)]
    cfg = dict(architecture="Fovenex", width=W, vocab=8, norm=dict(eps=1e-6), streams=2, residual_mult=1.0, layers=layers)
    w = models.make_weights(cfg, seed=3)
    w["embed"] = _loud_table(W)
    for i in range(len(layers)):
        p = f"l{i}."
        w[p + "norm1"], w[p + "ls1"] = torch.ones(W), torch.ones(W)
        # stream 0 keeps the embedding, stream 1 takes the result; every layer reads stream 0
        w[p + "hc1.in"], w[p + "hc1.mix"] = torch.tensor([1.0, 0.0]), torch.eye(2)
        w[p + "hc1.out"] = torch.tensor([0.0, 1.0 if i == len(layers) - 1 else 0.0])
        m = p + "mix."
        dq = torch.zeros((8, W))
        dq[0, 1] = 1.0               # asks
        dq[1, :8] = 0.3              # (so that no row is nothing)
        w[m + "dq"], w[m + "dq.norm"] = dq, torch.ones(8)
        uq = torch.zeros((24, 8))
        uq[0, 0] = 30.0
        w[m + "uq"] = uq
        if i == 0:
            dkv = torch.zeros((32, W))
            dkv[0, 2] = 1.0          # loud
            for t in range(8):
                dkv[1 + t, t] = 1.0  # names the token
            w[m + "dkv"], w[m + "dkv.norm"] = dkv, torch.ones(24)
        uk, uv = torch.zeros((16, 24)), torch.zeros((16, 24))
        uk[0, 0] = 1.0
        for t in range(8):
            uv[t, 1 + t] = 1.0
        w[m + "uk"], w[m + "uv"], w[m + "g"] = uk, uv, torch.zeros((16, W))
        w[m + "o"] = torch.randn((W, 16), generator=torch.Generator().manual_seed(5))
    return models.write_config(str(tmp_path / f"loud_{window}_{reads_wider}"), cfg,
                               {n: t.to(torch.float32 if dtype == "float32" else torch.bfloat16) for n, t in w.items()})


@pytest.mark.parametrize("window, page, first", [(6, 4, None), (8, 8, None), (70, 16, None), (1, 4, None), (20, 8, 7), (7, 8, 20)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_just_inside_and_just_outside_the_window(tmp_path, window, page, first, dtype):
    """The loud key stands at a chosen distance from the asking token: in the window's last place it takes the softmax, one
    further it is not seen; in prompts, in portions and decoded one by one, also where the loud key is a sequence's first
    token or stands at a page's border, and where the latents are another layer's with a narrower or wider window."""
    folder = _loud_window_model(tmp_path, window, first, dtype)
    forward, engine = _plain(folder), _engine(folder, dtype, pages=64, page=page)
    seen = {}
    for at in (0, 1, page - 1, page, page + 1):
        for gap in sorted({1, window - 2, window - 1, window, window + 1} - {0, -1}):
            toks = [0] * (at + gap + 1)
            toks[at], toks[-1] = 2, 1
            ref = {"p": forward(toks)}
            for what, steps in (("whole", traces.whole({"p": toks})), ("decoded", traces.last_decoded({"p": toks}, tail=gap + 1)),
                                ("portions", traces.portions({"p": toks}, seed=at + gap, sizes=(2, 3, 5, 2)))):
                _check(steps, traces.run_in_process(engine, steps), ref, dtype, (what, at, gap))
            seen[(at, gap)] = ref["p"][-1]
    for at in (0, page):
        if window > 1:
            assert float((seen[(at, window - 1)] - seen[(at, window)]).abs().max()) > 0.3
        assert float((seen[(at, window)] - seen[(at, window + 1)]).abs().max()) < 0.1


@pytest.mark.parametrize("which", [0, 1])
@pytest.mark.parametrize("dtype, dim, vdim", [("float32", 16, 16), ("bfloat16", 16, 16), ("bfloat16", 64, 128), ("bfloat16", 32, 64)])
def test_a_far_key_takes_one_map_alone(tmp_path, which, dtype, dim, vdim):
    """The asking token points at the loud one in map ``which`` alone, however far back it stands, at page and block borders and
    first in the sequence: the head's difference then names the loud token (with the sign of the map)."""
    W = 48
    cfg = dict(architecture="Fovenex", width=W, vocab=8, norm=dict(eps=1e-6), streams=2, residual_mult=1.0,
               layers=[models._layer("attention", models._attn(1, 1, dim, vdim, 1.0, 0.5))])
    w = models.make_weights(cfg, seed=3)
    w["embed"] = _loud_table(W)
    w["l0.norm1"], w["l0.ls1"] = torch.ones(W), torch.ones(W)
    w["l0.hc1.in"], w["l0.hc1.mix"], w["l0.hc1.out"] = torch.tensor([1.0, 0.0]), torch.eye(2), torch.tensor([0.0, 1.0])
    q, k, v = torch.zeros((2, dim, W)), torch.zeros((2, dim, W)), torch.zeros((vdim, W))
    for m in range(2):      # every row of queries and keys is something, and no two of them meet but the loud ones
        q[m, 1, :8] = 1.0
        k[m, 2, :8] = 1.0
    q[which, 0, 1] = k[which, 0, 2] = 20.0
    for t in range(8):
        v[t, t] = 1.0
    p = "l0.mix."
    w[p + "q"], w[p + "k"], w[p + "v"] = q.view(2 * dim, W), k.view(2 * dim, W), v
    w[p + "q.norm"], w[p + "k.norm"] = torch.full((dim,), 2.0), torch.full((dim,), 2.0)
    for x in ("lq1", "lk1", "lq2", "lk2"):
        w[p + x] = torch.zeros(dim)
    w[p + "g"] = torch.zeros((1, W))
    w[p + "o"] = torch.randn((W, vdim), generator=torch.Generator().manual_seed(5))
    w["final.norm"] = torch.ones(W)
    folder = models.write_config(str(tmp_path / "m"), cfg,
                                 {n: t.to(torch.float32 if dtype == "float32" else torch.bfloat16) for n, t in w.items()})
    forward, engine = _plain(folder), _engine(folder, dtype, pages=80, page=16)
    quiet = [0] * 300
    quiet[-1] = 1
    base = forward(quiet)[-1]
    for at in (0, 1, 15, 16, 127, 128, 255, 256, 298):
        toks = list(quiet)
        toks[at] = 2
        ref = {"p": forward(toks)}
        assert float((ref["p"][-1] - base).abs().max()) > 0.3, at
        for what, steps in (("whole", traces.whole({"p": toks})), ("decoded", traces.last_decoded({"p": toks}, tail=3)),
                            ("portions", traces.portions({"p": toks}, seed=at, sizes=(130, 2, 5, 64)))):
            _check(steps, traces.run_in_process(engine, steps), ref, dtype, (what, at))


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


@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_models_of_one_kind_of_layer_alone(tmp_path, kind):
    """Layers of either kind alone, decoded and in portions that come again and again, so that recorded steps are replayed
    (every part of the design is graph- and tape-safe and its steps may be padded)."""
    layers = [l for l in models.MAIN["layers"] if l["type"] == kind]
    if kind == "latent_attention":
        layers = [dict(l, mixer={**l["mixer"], **({"kv_from": 0} if "kv_from" in l["mixer"] else {})}) for l in layers]
    cfg = dict(models.MAIN, layers=layers)
    folder = models.write_config(str(tmp_path / "m"), cfg, models.make_weights(cfg, 5, torch.bfloat16))
    forward, engine = _plain(folder), _engine(folder, "bfloat16", pages=128, page=8)
    assert engine.model.padding_safe() and engine.model.tape_safe() and engine.model.graph_safe()
    requests = {f"q{i}": traces.random_tokens(cfg["vocab"], n, seed=60 + i) for i, n in enumerate([70, 66, 90, 75, 64, 68, 71])}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    for steps in (traces.last_decoded(requests, tail=20), traces.portions(requests, seed=1, sizes=(30, 9)),
                  traces.mixed(requests, max_live=4, seed=2, decode_tail=40, max_portion=30), traces.last_decoded(requests, tail=20)):
        _check(steps, traces.run_in_process(engine, steps), ref, "bfloat16", kind)
    engine.cache.check()


def test_a_long_prompt_beside_decoding_requests(tmp_path):
    """Steps of several hundred tokens (the kernels for many tokens), portions beside single tokens, and more than 2,048 keys."""
    cfg = dict(models.MAIN, layers=models.MAIN["layers"][4:6])
    folder = models.write_config(str(tmp_path / "m"), cfg, models.make_weights(cfg, 6, torch.bfloat16))
    forward, engine = _plain(folder), _engine(folder, "bfloat16", pages=420, page=16)
    requests = {"long": traces.random_tokens(cfg["vocab"], 2300, seed=1), "a": traces.random_tokens(cfg["vocab"], 400, seed=2),
                "b": traces.random_tokens(cfg["vocab"], 90, seed=3)}
    ref = {rid: forward(toks) for rid, toks in requests.items()}
    for steps in (traces.few_wanted(traces.whole(requests), none=0.0),
                  traces.random_wanted(traces.mixed(requests, max_live=3, seed=2, decode_tail=30, max_portion=700), seed=4)):
        _check(steps, traces.run_in_process(engine, steps), ref, "bfloat16", "long prompt")


def test_the_stream_after_every_layer(tmp_path):
    """In float32 the sum of the streams after each layer is the plain implementation's (an error in one layer shows there)."""
    from zedinfer_amd.engine import StepEntry
    for name in ("main", "odd", "wide"):
        forward, engine = _setup(tmp_path, name, "float32", pages=64)
        cfg, w = plain.load_folder(str(tmp_path / name))
        toks = traces.random_tokens(cfg["vocab"], 40, seed=9)
        _, want = plain.forward(cfg, w, toks, return_layers=True)
        after = []
        for block in engine.model.blocks:
            run = block.forward

            def watched(resid, delta, batch, memory, run=run):
                out = run(resid, delta, batch, memory)
                con, y = out
                s = resid.count
                X = resid.values if resid.values.dim() == 3 else torch.stack([resid.values] * s)
                y = (y.sum(0) if y.dim() == 3 else y) * con.scale
                new = torch.stack([sum(con.write[a * s + t] * X[a] for a in range(s)) + con.write[s * s + t] * y for t in range(s)])
                after.append(new.sum(0).double().cpu())
                return out
            block.forward = watched
        seq = engine.open("a")
        engine.step([StepEntry(seq, toks, [0])])
        engine.close(seq)
        assert len(after) == len(want)
        for i, (a, b) in enumerate(zip(after, want)):
            assert float((a[:40] - b).abs().max()) <= 2e-5 * max(1.0, float(b.abs().max())), (name, i)


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
