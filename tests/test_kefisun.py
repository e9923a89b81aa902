"""The Kefisun design on the CPU: its config.json reader, its description in parts, and the plain implementation's own
mechanisms held against each other (a decay of one for every channel is the plain delta rule; a cut of a sequence
through the state; a slope of nothing is plain attention; a convolution cut in two)."""
import copy
import math

import pytest
import torch

import kefisun_models as models
from plain import kefisun_plain as plain

F64 = torch.float64


def _config(d):
    from zedinfer_amd.config import find_architecture
    arch = find_architecture(d)
    return arch, arch.config_cls.from_dict(d)


def test_the_registry_knows_the_design_and_every_size_comes_from_the_config():
    from zedinfer_amd.models import expected_weights
    for cfg in list(models.CONFIGS.values()) + [models.random_config(s) for s in range(40)]:
        arch, c = _config(cfg)
        assert arch.name == "Kefisun" and c.hidden_size == cfg["width"] and c.vocab_size == cfg["vocab"]
        fc = arch.forward_config(c)
        want, got = models.tensor_shapes(cfg), expected_weights(fc)
        assert set(got) == set(want)
        assert all(tuple(got[k].shape) == tuple(want[k]) for k in want), cfg
        assert [l.block for l in fc.layers] == ["prenorm"] * len(cfg["layers"])
        kinds = {"attention": "conv_attention", "channel_delta": "channel_delta_rule"}
        assert [l.mixer.kind for l in fc.layers] == ["input_convolution"] * len(cfg["layers"])
        assert [l.mixer.params["mixer"].kind for l in fc.layers] == [kinds[x["type"]] for x in cfg["layers"]]
        assert c.to_dict()["layers"] == cfg["layers"]
        assert {k: c.to_dict()[k] for k in ("canon", "embedding", "logit_scale")} == {k: cfg[k] for k in ("canon", "embedding", "logit_scale")}


def test_constants_of_a_layer_reach_its_part():
    arch, c = _config(models.MAIN)
    fc = arch.forward_config(c)
    inner = [l.mixer.params["mixer"].params for l in fc.layers]
    assert [p.get("value_mix") for p in inner] == [None, "first", None, "mix", None, "mix"]
    assert [p.get("window") for p in inner] == [33, 20, None, 9, None, 20]
    a = inner[1]
    assert (a["num_heads"], a["num_kv_heads"], a["head_dim"], a["value_dim"], a["conv"], a["scale"]) == (6, 2, 32, 16, 4, 0.15)
    assert not a["bias"] and not a["sink"] and a["log_distance"] and a["gate"] and a["eps"] == 3e-6
    d = inner[2]
    assert (d["heads"], d["kv_heads"], d["dim"], d["vdim"], d["conv"], d["decay_rank"], d["gate_rank"]) == (4, 2, 16, 24, 2, 10, 7)
    assert all(l.mixer.params["taps"] == 3 for l in fc.layers)
    assert fc.layers[1].feed_forward.params == dict(hidden_size=96, intermediate_size=72, limit=0.6, bias=True)
    assert fc.layers[3].feed_forward.kind == "none" and fc.layers[3].norms["post_mixer"].kind == "none"
    assert fc.embedding.params["scale"] == 5.5 and fc.final_norm.params["gain_scale"] == 1.7
    assert fc.lm_head.weights["weight"] == fc.embedding.weights["weight"] == "embed"
    # the ranks are the checkpoint's own when the config does not name them
    cfg = copy.deepcopy(models.MAIN)
    for k in ("decay_rank", "gate_rank"):
        cfg["layers"][2]["mixer"].pop(k)
    arch, c = _config(cfg)
    from zedinfer_amd.models import expected_weights
    w = expected_weights(arch.forward_config(c))
    assert w["l2.mix.a1"].shape == (-1, 96) and w["l2.mix.g2"].shape == (96, -1)


def test_a_model_may_carry_the_share_that_its_first_mixing_layer_never_uses():
    from zedinfer_amd.models import expected_weights
    from zedinfer_amd.weights.loader import check_names
    arch, c = _config(models.MAIN)
    fc = arch.forward_config(c)
    found = dict(models.tensor_shapes(models.MAIN))
    found["l1.mix.vmix"] = ()
    check_names(expected_weights(fc), found, fc.ignorable_tensors)
    found["l1.mix.other"] = ()
    with pytest.raises(ValueError):
        check_names(expected_weights(fc), found, fc.ignorable_tensors)


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("norm"), "norm"), (lambda c: c.pop("canon"), "canon"), (lambda c: c["canon"].pop("taps"), "taps"),
    (lambda c: c["canon"].update(taps=0), "canon.taps"), (lambda c: c["layers"][0].update(type="conv"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_heads"), "kv_heads"), (lambda c: c["layers"][2]["mixer"].pop("conv"), "conv"),
    (lambda c: c["layers"][1]["mixer"].update(heads=5), "kv_heads"), (lambda c: c["layers"][1]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"), (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mlp"].update(limit=0), "limit"), (lambda c: c["layers"][2]["mixer"].update(dim=0), "positive"),
    (lambda c: c["layers"][3]["mixer"].update(vdim=40), "mix values"), (lambda c: c.update(layers=[]), "layers")])
def test_a_config_that_cannot_be_built_is_refused_with_the_key_named(change, word):
    from zedinfer_amd.config import ConfigError
    cfg = copy.deepcopy(models.MAIN)
    change(cfg)
    with pytest.raises(ConfigError) as e:
        _config(cfg)
    assert word in str(e.value)


def test_plain_mechanisms_agree_with_each_other():
    g = torch.Generator().manual_seed(3)
    T, H, G, d, dv = 25, 4, 2, 6, 5
    q, k, v = torch.randn((T, H, d), generator=g, dtype=F64), torch.randn((T, G, d), generator=g, dtype=F64), torch.randn((T, G, dv), generator=g, dtype=F64)
    none, r1, r2 = torch.zeros(H, dtype=F64), torch.rand(H, generator=g, dtype=F64) + 0.5, torch.rand(H, generator=g, dtype=F64) + 0.5
    s = torch.einsum("thd,shd->hts", q, k.repeat_interleave(H // G, dim=1)) * 0.3
    s = s.masked_fill(torch.triu(torch.ones((T, T), dtype=torch.bool), diagonal=1), float("-inf"))
    causal = torch.einsum("hts,shv->thv", torch.softmax(s, -1), v.repeat_interleave(H // G, dim=1))
    # no slope (or a rate of nothing) and no window, or one that covers everything: causal attention
    assert float((plain.distance_biased_attention(q, k, v, 0.3, none, r2, None) - causal).abs().max()) < 1e-12
    assert float((plain.distance_biased_attention(q, k, v, 0.3, r1, none, T) - causal).abs().max()) < 1e-12
    # the bias by distance as a matrix
    dist = (torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)).clamp(min=0).to(F64)
    sb = s - r1.view(H, 1, 1) * torch.log1p(r2.view(H, 1, 1) * dist)
    sb = sb.masked_fill(dist.view(1, T, T) >= 7, float("-inf"))
    biased = torch.einsum("hts,shv->thv", torch.softmax(sb, -1), v.repeat_interleave(H // G, dim=1))
    assert float((plain.distance_biased_attention(q, k, v, 0.3, r1, r2, 7) - biased).abs().max()) < 1e-12
    assert float((plain.distance_biased_attention(q, k, v, 0.3, r1, r2, 8) - biased).abs().max()) > 1e-3
    # the delta rule with one decay for every channel, written with the scalar outside
    kk, qq = plain.unit(torch.randn((T, 2, d), generator=g, dtype=F64)), plain.unit(torch.randn((T, 2, d), generator=g, dtype=F64))
    vv, beta = torch.randn((T, 4, dv), generator=g, dtype=F64), torch.rand((T, 4), generator=g, dtype=F64)
    gg = torch.rand((T, 4, 1), generator=g, dtype=F64)
    out, S = plain.channel_delta_rule(qq, kk, vv, beta, gg.expand(T, 4, d))
    M = torch.zeros((4, d, dv), dtype=F64)
    for t in range(T):
        for h in range(4):
            a = kk[t, h // 2].view(d, 1)
            M[h] = gg[t, h] * (M[h] - beta[t, h] * a @ (a.T @ M[h])) + beta[t, h] * a @ vv[t, h].view(1, dv)
            assert float((M[h].T @ qq[t, h // 2] - out[t, h]).abs().max()) < 1e-12
    assert float((M - S).abs().max()) < 1e-12
    # cut in two through the state
    decay = torch.rand((T, 4, d), generator=g, dtype=F64)
    whole, end = plain.channel_delta_rule(qq, kk, vv, beta, decay)
    a, mid = plain.channel_delta_rule(qq[:9], kk[:9], vv[:9], beta[:9], decay[:9])
    b, end2 = plain.channel_delta_rule(qq[9:], kk[9:], vv[9:], beta[9:], decay[9:], mid)
    assert float((torch.cat([a, b]) - whole).abs().max()) < 1e-12 and float((end - end2).abs().max()) < 1e-12
    # softplus far out on both sides
    z = torch.tensor([-200.0, -1.0, 0.0, 1.0, 40.0, 800.0], dtype=F64)
    assert torch.allclose(plain.softplus(z), torch.nn.functional.softplus(z, threshold=60.0), atol=1e-12)
    # one tap alone is a scaling of the present row
    x = torch.randn((6, 3), generator=g, dtype=F64)
    assert torch.equal(plain.input_convolution(x, torch.full((3, 1), 0.5, dtype=F64)), 1.5 * x)


def test_the_clamps_of_the_feed_forward():
    g = torch.tensor([-9.0, -0.5, 0.5, 9.0], dtype=F64)
    u = torch.tensor([-9.0, 9.0, 0.2, -0.3], dtype=F64)
    got = plain.clamped_glu(g, u, 2.0)
    want = [-9.0 / (1 + math.exp(1.702 * 9)) * (-2 + 1), -0.5 / (1 + math.exp(1.702 * 0.5)) * 3, 0.5 / (1 + math.exp(-1.702 * 0.5)) * 1.2,
            2.0 / (1 + math.exp(-1.702 * 2)) * 0.7]
    assert torch.allclose(got, torch.tensor(want, dtype=F64), atol=1e-12)


def test_the_plain_model_reads_a_folder_and_is_causal(tmp_path):
    folder = models.write_model(str(tmp_path / "m"), "odd", seed=1)
    cfg, w = plain.load_folder(folder)
    toks = [3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8, 9, 7]
    full, layers = plain.forward(cfg, w, toks, return_layers=True)
    assert full.shape == (len(toks), 150) and layers.shape == (3, len(toks), 83) and torch.isfinite(full).all()
    assert float((plain.forward(cfg, w, toks[:9]) - full[:9]).abs().max()) < 1e-9
    out = plain.greedy_generate(cfg, w, toks[:5], 3)
    assert len(out) == 3 and out[0] == int(torch.argmax(plain.forward(cfg, w, toks[:5])[-1]))


def test_every_part_of_a_layer_shows_in_the_logits(tmp_path):
    """The tests' weights let no mechanism hide: leaving one out, in the plain model, moves the logits."""
    folder = models.write_model(str(tmp_path / "m"), "main", seed=2)
    cfg, w = plain.load_folder(folder)
    g = torch.Generator().manual_seed(1)
    toks = [int(t) for t in torch.randint(0, 310, (40,), generator=g)]
    ref = plain.forward(cfg, w, toks)
    scale = float(ref.abs().max())

    def moved(change_w=None, change_cfg=None):
        c2, w2 = copy.deepcopy(cfg), dict(w)
        if change_w:
            change_w(w2)
        if change_cfg:
            change_cfg(c2)
        return float((plain.forward(c2, w2, toks) - ref).abs().max()) / scale
    tail = w["l2.canon1"].clone()
    tail[:, 0] = 0
    cases = {
        "input convolution's oldest tap": (lambda x: x.update({"l2.canon1": tail}), None),
        "value share": (lambda x: x.update({"l3.mix.vmix": x["l3.mix.vmix"] + 0.1}), None),
        "slope": (lambda x: x.update({"l1.mix.r1": 0.5 * x["l1.mix.r1"]}), None),
        "rate": (lambda x: x.update({"l1.mix.r2": 0.5 * x["l1.mix.r2"]}), None),
        "decay bias": (lambda x: x.update({"l4.mix.dt_bias": x["l4.mix.dt_bias"] + 0.3}), None),
        "biases": (lambda x: x.update({"l5.mlp.down.b": 0 * x["l5.mlp.down.b"]}), None),
        "window": (None, lambda c: c["layers"][1]["mixer"]["mask"].update(size=21)),
        "limit": (None, lambda c: c["layers"][1]["mlp"].update(limit=0.7)),
        "embedding scale": (None, lambda c: c["embedding"].update(scale=5.6)),
        "logit scale": (None, lambda c: c.update(logit_scale=1.71)),
    }
    for what, (cw, cc) in cases.items():
        assert moved(cw, cc) > 2e-3, what      # float32's tolerance is 2e-4
