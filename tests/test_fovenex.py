"""The Fovenex design on the CPU: its config.json reader, its description in parts, and the plain implementation's own
mechanisms held against each other (one stream that is kept whole is the ordinary residual sum; a second map that counts
for nothing is plain attention; a turn keeps lengths; a window that covers everything is causal attention)."""
import copy
import math

import pytest
import torch

import fovenex_models as models
from plain import fovenex_plain as plain

F64 = torch.float64


def _config(d):
    from zedinfer_amd.config import find_architecture
    arch = find_architecture(d)
    return arch, arch.config_cls.from_dict(d)


def test_the_registry_knows_the_design_and_every_size_comes_from_the_config():
    from zedinfer_amd.models import expected_weights
    for cfg in list(models.CONFIGS.values()) + [models.random_config(s) for s in range(40)]:
        arch, c = _config(cfg)
        assert arch.name == "Fovenex" and c.hidden_size == cfg["width"] and c.vocab_size == cfg["vocab"]
        fc = arch.forward_config(c)
        want, got = models.tensor_shapes(cfg), expected_weights(fc)
        assert set(got) == set(want)
        assert all(tuple(got[k].shape) == tuple(want[k]) for k in want), cfg
        assert fc.streams == cfg["streams"] and [l.block for l in fc.layers] == ["connected"] * len(cfg["layers"])
        kinds = {"attention": "difference_attention", "latent_attention": "latent_attention"}
        assert [l.mixer.kind for l in fc.layers] == [kinds[x["type"]] for x in cfg["layers"]]
        for st, layer in zip(fc.schedule, cfg["layers"]):
            src = layer["mixer"].get("kv_from")
            assert st.writes_cache == (src is None) and st.cache == (st.layer if src is None else src)
        assert c.to_dict()["layers"] == cfg["layers"]
        assert {k: c.to_dict()[k] for k in ("streams", "residual_mult", "norm")} == {k: cfg[k] for k in ("streams", "residual_mult", "norm")}


def test_constants_of_a_layer_reach_its_part():
    arch, c = _config(models.MAIN)
    fc = arch.forward_config(c)
    a = fc.layers[0].mixer.params
    assert (a["num_heads"], a["num_kv_heads"], a["head_dim"], a["value_dim"], a["scale"], a["diff"], a["eps"]) == (4, 2, 32, 64, 0.2, 0.35, 3e-6)
    assert a["position"].params == dict(head_dim=32, rotary_dim=32, theta=500.0, scaling=models.RAMP)
    l = fc.layers[3].mixer.params
    assert (l["heads"], l["dim"], l["rot_dim"], l["vdim"], l["kv_rank"], l["q_rank"], l["window"]) == (5, 16, 8, 24, 48, 40, 9)
    assert l["shares_cache"] and l["gate"] and l["pairing"] == "halves" and not fc.layers[1].mixer.params["shares_cache"]
    con = fc.layers[1].connections["feed_forward"]
    assert con.params == dict(streams=3, hidden_size=96, mult=0.7, scale=True)
    assert con.weights == {"in": "l1.hc2.in", "out": "l1.hc2.out", "mix": "l1.hc2.mix", "scale": "l1.ls2"}
    assert fc.layers[2].feed_forward.kind == fc.layers[2].norms["post_mixer"].kind == fc.layers[2].connections["feed_forward"].kind == "none"
    assert fc.layers[0].feed_forward.params == dict(hidden_size=96, intermediate_size=136, activation="gelu_tanh")
    # the query latents' size is the checkpoint's own when the config does not name it
    cfg = copy.deepcopy(models.MAIN)
    cfg["layers"][1]["mixer"].pop("q_rank")
    from zedinfer_amd.models import expected_weights
    arch, c = _config(cfg)
    w = expected_weights(arch.forward_config(c))
    assert w["l1.mix.dq"].shape == (-1, 96) and w["l1.mix.uq"].shape == (96, -1)


def test_a_layer_without_a_feed_forward_may_carry_what_would_stand_around_it():
    from zedinfer_amd.models import expected_weights
    from zedinfer_amd.weights.loader import check_names
    arch, c = _config(models.MAIN)
    fc = arch.forward_config(c)
    found = dict(models.tensor_shapes(models.MAIN))
    found.update({"l2.norm2": (96,), "l2.ls2": (96,), "l2.hc2.in": (3,), "l2.hc2.out": (3,), "l2.hc2.mix": (3, 3)})
    check_names(expected_weights(fc), found, fc.ignorable_tensors)
    found["l2.mlp.up"] = (4, 96)
    with pytest.raises(ValueError):
        check_names(expected_weights(fc), found, fc.ignorable_tensors)


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("norm"), "norm"), (lambda c: c.pop("streams"), "streams"), (lambda c: c.update(streams=0), "streams"),
    (lambda c: c.update(streams=40), "streams"), (lambda c: c["layers"][0].update(type="conv"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_heads"), "kv_heads"), (lambda c: c["layers"][0]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][0]["mixer"].update(heads=5), "kv_heads"), (lambda c: c["layers"][1]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"), (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mlp"].update(ff=0), "ff"), (lambda c: c["layers"][1]["mixer"].update(dim=0), "positive"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34), "rot.dims"), (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][1]["mixer"].update(rot_dim=10), "rot_dim"), (lambda c: c["layers"][3]["mixer"].update(kv_rank=40), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "kv_from"), (lambda c: c["layers"][3]["mixer"].update(kv_from=4), "kv_from"),
    (lambda c: c["layers"][6]["mixer"].update(kv_from=3), "kv_from"), (lambda c: c.update(layers=[]), "layers")])
def test_a_config_that_cannot_be_built_is_refused_with_the_key_named(change, word):
    from zedinfer_amd.config import ConfigError
    cfg = copy.deepcopy(models.MAIN)
    change(cfg)
    with pytest.raises(ConfigError) as e:
        _config(cfg)
    assert word in str(e.value)


def test_blocks_and_streams_must_agree():
    from zedinfer_amd.config import PartSpec, ScheduleStep
    import dataclasses
    arch, c = _config(models.MAIN)
    fc = arch.forward_config(c)
    with pytest.raises(ValueError):
        dataclasses.replace(fc, streams=0).validate()
    with pytest.raises(ValueError):
        dataclasses.replace(fc, layers=tuple(dataclasses.replace(l, connections={}) for l in fc.layers)).validate()
    with pytest.raises(ValueError):
        dataclasses.replace(fc, schedule=tuple(ScheduleStep(s.layer, s.cache, s.writes_cache, PartSpec("reenter", {})) for s in fc.schedule)).validate()


def test_plain_mechanisms_agree_with_each_other():
    g = torch.Generator().manual_seed(3)
    T, H, G, d, dv = 25, 4, 2, 6, 5
    q, k = torch.randn((T, H, 2, d), generator=g, dtype=F64), torch.randn((T, G, 2, d), generator=g, dtype=F64)
    v = torch.randn((T, G, dv), generator=g, dtype=F64)
    att = []
    for m in range(2):
        s = torch.einsum("thd,shd->hts", q[:, :, m], k[:, :, m].repeat_interleave(H // G, dim=1)) * 0.3
        s = s.masked_fill(torch.triu(torch.ones((T, T), dtype=torch.bool), diagonal=1), float("-inf"))
        att.append(torch.einsum("hts,shv->thv", torch.softmax(s, -1), v.repeat_interleave(H // G, dim=1)))
    # the second map not counted: plain attention under the head's norm; counted: the difference
    assert float((plain.difference_of_maps(q, k, v, 0.3, 0.0, 0.0, 1e-9) - plain.rms(att[0], 1e-9)).abs().max()) < 1e-12
    got = plain.difference_of_maps(q, k, v, 0.3, 0.4, 0.25, 1e-6)
    assert float((got - 0.75 * plain.rms(att[0] - 0.4 * att[1], 1e-6)).abs().max()) < 1e-12
    assert abs(plain.mixing_weight(torch.zeros(3), torch.ones(3), torch.zeros(3), torch.ones(3), 0.3) - 0.3) < 1e-15
    one = plain.mixing_weight(torch.tensor([0.5]), torch.tensor([2.0]), torch.tensor([1.0]), torch.tensor([-1.0]), 0.1)
    assert abs(one - (math.e - 1.0 / math.e + 0.1)) < 1e-6
    # a window that covers everything, one that is a token short, one of the token alone
    sc = torch.randn((T, T), generator=g, dtype=F64)
    assert torch.equal(plain.softmax_map(sc, T), plain.softmax_map(sc, None))
    assert not torch.equal(plain.softmax_map(sc, T - 1), plain.softmax_map(sc, None))
    assert torch.equal(plain.softmax_map(sc, 1), torch.eye(T, dtype=F64))
    # one stream that is kept whole is the ordinary sum; a permutation moves whole streams
    X, y = torch.randn((3, T, 7), generator=g, dtype=F64), torch.randn((T, 7), generator=g, dtype=F64)
    assert torch.allclose(plain.write_streams(X[:1], torch.ones((1, 1), dtype=F64), torch.ones(1, dtype=F64), y, 0.5)[0], X[0] + 0.5 * y)
    P = torch.zeros((3, 3), dtype=F64)
    P[0, 1] = P[1, 2] = P[2, 0] = 1.0          # from 0 to 1, from 1 to 2, from 2 to 0
    moved = plain.write_streams(X, P, torch.zeros(3, dtype=F64), y, 1.0)
    assert torch.equal(moved[1], X[0]) and torch.equal(moved[2], X[1]) and torch.equal(moved[0], X[2])
    assert torch.allclose(plain.read_streams(X, torch.tensor([1.0, 0.0, 2.0], dtype=F64)), X[0] + 2 * X[2])
    # a turn keeps every pair's length (times the magnitude) and the products of equal distances
    f, mag = plain.pair_frequencies(4, 100.0)
    assert mag == 1.0 and f == [1.0, 0.1]
    x = torch.randn((T, 1, d), generator=g, dtype=F64)
    assert torch.allclose(plain.turn(x, f).norm(dim=-1), x.norm(dim=-1)) and torch.equal(plain.turn(x, f)[..., 4:], x[..., 4:])
    same = x[:1].expand(T, 1, d)
    t = plain.turn(same, f)[:, 0]
    assert abs(float(t[3] @ t[7]) - float(t[10] @ t[14])) < 1e-12
    # frequencies outside the ramp: kept, or divided
    f0, _ = plain.pair_frequencies(64, 10000.0)
    f1, m1 = plain.pair_frequencies(64, 10000.0, dict(factor=4.0, original=2048, fast=32.0, slow=1.0))
    assert f1[0] == f0[0] and abs(f1[-1] - f0[-1] / 4.0) < 1e-18 and abs(m1 - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    assert torch.allclose(plain.gelu(torch.tensor([-3.0, 0.0, 1.0, 9.0], dtype=F64)),
                          torch.nn.functional.gelu(torch.tensor([-3.0, 0.0, 1.0, 9.0], dtype=F64), approximate="tanh"), atol=1e-12)
    z = torch.randn((T, 9), generator=g, dtype=F64)
    assert torch.allclose(plain.layer_norm(z, torch.ones(9, dtype=F64), 1e-5), torch.nn.functional.layer_norm(z, (9,), eps=1e-5))


def test_the_frequencies_of_the_engine_are_the_plain_ones():
    from zedinfer_amd.parts.positions import ramped_frequencies
    for dims, base, sc in ((24, 10000.0, dict(factor=4.0, original=2048, fast=32.0, slow=1.0)), (32, 500.0, models.RAMP), (8, 100.0, None),
                           (64, 250000.0, dict(factor=40.0, original=20, fast=1.0, slow=1.0)), (2, 10.0, dict(factor=3.0, original=7, fast=2.0, slow=1.0))):
        f, mag = ramped_frequencies(dims, base, sc)
        want, wmag = plain.pair_frequencies(dims, base, sc)
        assert max(abs(float(a) - b) / b for a, b in zip(f, want)) < 1e-6 and abs(mag - wmag) < 1e-12


def test_the_plain_model_reads_a_folder_and_is_causal(tmp_path):
    folder = models.write_model(str(tmp_path / "m"), "odd", seed=1)
    cfg, w = plain.load_folder(folder)
    toks = [3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8, 9, 7]
    full, layers = plain.forward(cfg, w, toks, return_layers=True)
    assert full.shape == (len(toks), 150) and layers.shape == (4, len(toks), 83) and torch.isfinite(full).all()
    assert float((plain.forward(cfg, w, toks[:9]) - full[:9]).abs().max()) < 1e-9
    out = plain.greedy_generate(cfg, w, toks[:5], 3)
    assert len(out) == 3 and out[0] == int(torch.argmax(plain.forward(cfg, w, toks[:5])[-1]))


def test_every_part_of_a_layer_shows_in_the_logits(tmp_path):
    """The tests' weights let no mechanism hide: leaving one out, in the plain model, moves the logits."""
    folder = models.write_model(str(tmp_path / "m"), "main", seed=2)
    cfg, w = plain.load_folder(folder)
    g = torch.Generator().manual_seed(1)
    toks = [int(t) for t in torch.randint(0, 310, (60,), generator=g)]
    ref = plain.forward(cfg, w, toks)
    scale = float(ref.abs().max())

    def moved(change_w=None, change_cfg=None):
        c2, w2 = copy.deepcopy(cfg), dict(w)
        if change_w:
            change_w(w2)
        if change_cfg:
            change_cfg(c2)
        return float((plain.forward(c2, w2, toks) - ref).abs().max()) / scale
    cases = {
        "the matrix is from-to": (lambda x: x.update({"l1.hc1.mix": x["l1.hc1.mix"].T}), None),
        "what a sublayer reads": (lambda x: x.update({"l1.hc2.in": x["l1.hc2.in"].flip(0)}), None),
        "where a result goes": (lambda x: x.update({"l4.hc1.out": x["l4.hc1.out"].flip(0)}), None),
        "layer scale of the mixer": (lambda x: x.update({"l2.ls1": 0 * x["l2.ls1"] + 1}), None),
        "layer scale of the feed-forward": (lambda x: x.update({"l0.ls2": 0 * x["l0.ls2"] + 1}), None),
        "the gate of a head": (lambda x: x.update({"l0.mix.g": 0 * x["l0.mix.g"]}), None),
        "the elementwise gate": (lambda x: x.update({"l1.mix.g": 0 * x["l1.mix.g"]}), None),
        "the maps' weight": (lambda x: x.update({"l0.mix.lq1": 0 * x["l0.mix.lq1"]}), None),
        "query norm": (lambda x: x.update({"l5.mix.q.norm": 0 * x["l5.mix.q.norm"] + 1}), None),
        "query latents' norm": (lambda x: x.update({"l3.mix.dq.norm": 0 * x["l3.mix.dq.norm"] + 1}), None),
        "window": (None, lambda c: c["layers"][3]["mixer"]["mask"].update(size=10)),
        "whose latents": (None, lambda c: c["layers"][6]["mixer"]["rot"].update(base=900.0)),
        "slowed frequencies": (None, lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling")),
        "diff": (None, lambda c: c["layers"][0]["mixer"].update(diff=0.4)),
        "residual constant": (None, lambda c: c.update(residual_mult=0.72)),
        "eps": (None, lambda c: c["norm"].update(eps=2e-2)),
    }
    for what, (cw, cc) in cases.items():
        assert moved(cw, cc) > 2e-3, what      # float32's tolerance is 2e-4
