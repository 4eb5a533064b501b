"""The plain Fiterax pinned by hand-made cases and closed forms, its configuration and what the engine makes of it
(parts, tensor names, schedule, caches); no GPU."""
import copy
import math

import pytest
import torch

import plain_fiterax as plain
import tiny_fiterax as tiny

F = torch.float64


def test_grouped_norm_takes_every_part_by_itself():
    x = torch.tensor([[3.0, 4.0, 0.0, 10.0]], dtype=F)
    y = plain.group_rms(x, torch.tensor([1.0, 2.0, 1.0, 1.0], dtype=F), 2, 0.0)[0]
    r1, r2 = math.sqrt(12.5), math.sqrt(50.0)
    assert y.tolist() == pytest.approx([3 / r1, 8 / r1, 0.0, 10 / r2])
    assert torch.allclose(plain.group_rms(x, torch.ones(4, dtype=F), 1, 0.5), plain.rms(x, 0.5))
    # eps is inside the root
    assert plain.rms(torch.zeros(1, 2, dtype=F), 0.25).abs().sum() == 0
    assert plain.rms(torch.ones(1, 2, dtype=F), 3.0)[0, 0].item() == pytest.approx(0.5)


def test_input_filter_adds_to_its_input_and_its_last_column_meets_the_row_itself():
    h = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    assert plain.input_conv(h, torch.tensor([[0.0, 0.0, 2.0]], dtype=F)).view(-1).tolist() == [3.0, 30.0, 300.0]
    assert plain.input_conv(h, torch.tensor([[1.0, 0.0, 0.0]], dtype=F)).view(-1).tolist() == [1.0, 10.0, 101.0]
    assert plain.input_conv(h, torch.tensor([[0.0, 1.0, 0.0]], dtype=F)).view(-1).tolist() == [1.0, 11.0, 110.0]
    assert plain.input_conv(h, torch.tensor([[0.5]], dtype=F)).view(-1).tolist() == [1.5, 15.0, 150.0]


def test_the_turn_pairs_halves_and_leaves_the_rest():
    x = torch.zeros(6, 1, 5, dtype=F)
    x[5, 0] = torch.tensor([1.0, 0.0, 0.0, 2.0, 9.0], dtype=F)
    y = plain.turn_halves(x, 4, 100.0)[5, 0]
    a0, a1 = 5.0, 5.0 * 100.0 ** -0.5
    assert y.tolist() == pytest.approx([math.cos(a0), -2.0 * math.sin(a1), math.sin(a0), 2.0 * math.cos(a1), 9.0])


def _attention_weights(H, G, d, vd, W, g):
    r = lambda *s: torch.randn(*s, generator=g, dtype=F)
    return {"q": r(H * d, W), "q.b": r(H * d), "k": r(G * d, W), "k.b": r(G * d), "v": r(G * vd, W), "v.b": r(G * vd),
            "temp": torch.ones(H, dtype=F), "g": torch.zeros(H, W, dtype=F), "o": torch.eye(H * vd, dtype=F),
            "o.b": torch.zeros(H * vd, dtype=F)}


def test_attention_averages_at_scale_zero_gates_a_head_and_caps_its_scores():
    g = torch.Generator().manual_seed(0)
    T, W, H, G, d, vd = 7, 6, 4, 2, 4, 3
    h = torch.randn(T, W, generator=g, dtype=F)
    w = _attention_weights(H, G, d, vd, W, g)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": vd, "scale": 0.0, "rot": {"dims": 2, "base": 10.0}}
    out = plain.attention(h, w, m, 1e-6).view(T, H, vd)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, vd)
    for t in range(T):                    # every visible key weighs the same; the gate's logits are zero
        for n in range(H):
            assert torch.allclose(out[t, n], 0.5 * v[:t + 1, n // 2].mean(0))
    w["g"] = torch.randn(H, W, generator=g, dtype=F)
    gated = plain.attention(h, w, m, 1e-6).view(T, H, vd)
    assert torch.allclose(gated, 2.0 * out * torch.sigmoid(h @ w["g"].T)[:, :, None])
    # a factor a head acts as its scale does; a cap far above the scores changes nothing, a low one does
    m1 = dict(m, scale=0.7)
    w["temp"] = torch.full((H,), 2.0, dtype=F)
    twice = plain.attention(h, w, m1, 1e-6)
    w["temp"] = torch.ones(H, dtype=F)
    assert torch.allclose(twice, plain.attention(h, w, dict(m, scale=1.4), 1e-6))
    assert torch.allclose(plain.attention(h, w, dict(m1, softcap=1e6), 1e-6), plain.attention(h, w, m1, 1e-6))
    assert not torch.allclose(plain.attention(h, w, dict(m1, softcap=0.3), 1e-6), plain.attention(h, w, m1, 1e-6))
    # queries and keys have unit length: their size does not matter
    big = dict(w, q=w["q"] * 5, **{"q.b": w["q.b"] * 5})
    assert torch.allclose(plain.attention(h, big, m1, 0.0), plain.attention(h, w, m1, 0.0))


def test_memory_by_hand_and_independent_of_the_running_maximum():
    one = lambda *v: torch.tensor(v, dtype=F)
    # one channel, one head: two tokens
    i, f = one(0.3, -1.0).view(2, 1), one(-0.2, -0.7).view(2, 1)
    q, k, v = one(1.0, 2.0).view(2, 1, 1), one(0.5, -3.0).view(2, 1, 1), one(4.0, 5.0).view(2, 1, 1)
    out = plain.mlstm_memory(q, k, v, i, f).view(-1)
    m1 = max(-0.2 + 0.0, 0.3)
    s1, n1 = math.exp(0.3 - m1) * 0.5 * 4.0, math.exp(0.3 - m1) * 0.5
    assert out[0].item() == pytest.approx(s1 / (max(abs(n1), math.exp(-m1)) + 1e-6))
    m2 = max(-0.7 + m1, -1.0)
    keep, add = math.exp(-0.7 + m1 - m2), math.exp(-1.0 - m2)
    s2, n2 = keep * s1 + add * -3.0 * 5.0, keep * n1 + add * -3.0
    assert out[1].item() == pytest.approx(2.0 * s2 / (max(abs(2.0 * n2), math.exp(-m2)) + 1e-6))
    # without the maximum: S = sum of e^(sum of f) e^i k v, the denominator at least 1 (the small constant apart)
    g = torch.Generator().manual_seed(1)
    T, d, vd = 9, 4, 3
    r = lambda *s: torch.randn(*s, generator=g, dtype=F)
    q, k, v, i = r(T, 1, d), r(T, 1, d), r(T, 1, vd), r(T, 1) * 2.0
    f = torch.nn.functional.logsigmoid(r(T, 1))
    out = plain.mlstm_memory(q, k, v, i, f)
    t = T - 1
    wgt = torch.stack([torch.exp(f[j + 1:t + 1].sum() + i[j, 0]) for j in range(T)])
    num = ((wgt * (k[:, 0] @ q[t, 0]))[:, None] * v[:, 0]).sum(0)
    den = max(abs(float((wgt * (k[:, 0] @ q[t, 0])).sum())), 1.0)
    assert torch.allclose(out[t, 0], num / den, rtol=1e-4)


def test_gates_are_capped_and_the_forget_gate_is_a_log_sigmoid():
    h = torch.tensor([[100.0], [-100.0], [0.0]], dtype=F)
    w = {"i": torch.ones(1, 1, dtype=F), "f": torch.ones(1, 1, dtype=F), "i.b": torch.zeros(1, dtype=F),
         "f.b": torch.zeros(1, dtype=F)}
    i, f = plain.log_gates(h, w, 5.0)
    assert i.view(-1).tolist() == pytest.approx([5.0, -5.0, 0.0])
    assert f.view(-1).tolist() == pytest.approx([-math.log1p(math.exp(-5.0)), -5.0 - math.log1p(math.exp(-5.0)), -math.log(2.0)])


def test_routing_chooses_by_the_corrected_score_and_weighs_by_the_plain_one():
    z = torch.tensor([2.0, 0.0, 1.0, -1.0], dtype=F)
    s = torch.sigmoid(z).tolist()
    r = plain.route(z, torch.zeros(4, dtype=F), 2, 3.0)
    assert [e for e, _ in r] == [0, 2] and r[0][1] == pytest.approx(3.0 * s[0] / (s[0] + s[2]))
    r = plain.route(z, torch.tensor([0.0, 0.0, 0.0, 1.0], dtype=F), 2, 1.0)
    assert [e for e, _ in r] == [3, 0]
    assert r[0][1] == pytest.approx(s[3] / (s[3] + s[0])) and sum(x for _, x in r) == pytest.approx(1.0)


def test_gelu_is_the_exact_one():
    z = torch.linspace(-4, 4, 33, dtype=F)
    assert torch.allclose(plain.gelu(z), torch.nn.functional.gelu(z))


@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_a_longer_sequence_leaves_earlier_logits_and_every_mechanism_moves_them(name):
    cfg = tiny.CONFIGS[name]
    w = tiny.make_weights(cfg, 13)
    seq = tiny.prompt(20, cfg["vocab"], 3)
    a, b = plain.logits(cfg, w, seq), plain.logits(cfg, w, seq[:11])
    assert torch.allclose(a[:11], b)
    moves = lambda change: float((plain.logits(cfg, {**w, **change}, seq)[-1] - a[-1]).abs().max())
    for key, t in w.items():
        if key.endswith((".temp", ".g", ".correction", "canon1", "canon2", ".b", "mix.i", "mix.f", "norm")):
            if key.endswith("correction") and all(not L.get("mlp") or L["mlp"]["router"]["top"] in (L["mlp"]["router"]["experts"],)
                                                  for L in cfg["layers"]):
                continue                                        # all experts a token: no choice to correct
            if "canon" in key and t.shape[1] > 1:
                t = t.clone()
                t[:, :-1] = 0.0                                 # (the taps before the row's own)
                assert moves({key: t}) > 1e-3, key
            elif key.endswith("correction"):
                assert max(moves({key: torch.roll(t, s)}) for s in range(1, t.shape[0])) > 1e-3, key
            else:
                assert moves({key: t + 0.5}) > 1e-3, key


@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_no_router_choice_of_the_test_models_is_a_close_call(name, monkeypatch):
    cfg = tiny.CONFIGS[name]
    w = tiny.make_weights(cfg, 13)
    gaps = []
    orig = plain.route

    def spy(z, correction, top, scale):
        c = torch.sort(torch.sigmoid(z) + correction, descending=True).values
        if top < c.shape[0]:
            gaps.append(float(c[top - 1] - c[top]))
        return orig(z, correction, top, scale)
    monkeypatch.setattr(plain, "route", spy)
    plain.logits(cfg, w, list(range(cfg["vocab"])))
    if gaps:
        assert min(gaps) > 0.015, min(gaps)


@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_configuration_round_trip_spec_and_caches(name):
    from swifttransformer_amd.config.fiterax_param import FiteraxHyperParam
    from swifttransformer_amd.models import build_model
    from swifttransformer_amd.models.decoder import conv_cache_id, ffn_conv_cache_id
    cfg = tiny.CONFIGS[name]
    hp = FiteraxHyperParam.from_dict(cfg)
    assert FiteraxHyperParam.from_dict(hp.to_config_dict()) == hp
    model = build_model(hp, torch.float32)
    w = tiny.make_weights(cfg, 0)
    specs = {s.name: tuple(s.shape) for s in model.tensor_specs() if not s.optional}
    assert specs == {k: tuple(v.shape) for k, v in w.items()}
    needs = model.cache_needs()
    taps, W = (cfg.get("canon") or {}).get("taps", 0), cfg["width"]
    for i, L in enumerate(cfg["layers"]):
        m = L["mixer"]
        if L["type"] == "mlstm":
            assert needs[i].kind == "state"
            assert needs[i].state_shape[0] >= m["heads"] * (m["dim"] * m["vdim"] + m["dim"] + 1)
        else:
            assert needs[i].kind == "paged_kv" and needs[i].num_kv_heads == m["kv_heads"]
            assert needs[i].head_dim % 16 == 0 and needs[i].head_dim >= max(m["dim"], m["vdim"]) and not needs[i].window
        for cid, there in ((conv_cache_id(i), taps > 0), (ffn_conv_cache_id(i), taps > 0 and L["mlp"] is not None)):
            assert (cid in needs) == there
            if there:
                assert needs[cid].state_shape == (taps - 1, W)


def test_configuration_errors_name_the_key():
    from swifttransformer_amd.config.fiterax_param import FiteraxHyperParam
    from swifttransformer_amd.config.hyper_param import ConfigError
    base = tiny.CONFIGS["A"]

    def broken(change):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError) as e:
            FiteraxHyperParam.from_dict(cfg)
        return str(e.value)
    assert "layers[0].mixer.heads" in broken(lambda c: c["layers"][0]["mixer"].update(heads=3))
    assert "vdim" in broken(lambda c: c["layers"][0]["mixer"].pop("vdim"))
    assert "dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5))
    assert "dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18))
    assert "gate_cap" in broken(lambda c: c["layers"][1]["mixer"].update(gate_cap=0))
    assert "dim" in broken(lambda c: c["layers"][1]["mixer"].update(dim=300))
    assert "top" in broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    assert "scale" in broken(lambda c: c["layers"][0]["mlp"]["router"].pop("scale"))
    assert "kind" in broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    assert "type" in broken(lambda c: c["layers"][0].update(type="other"))
    assert "groups" in broken(lambda c: c["norm"].update(groups=5))
    assert "taps" in broken(lambda c: c["canon"].update(taps=9))
    assert "residual_mult" in broken(lambda c: c.pop("residual_mult"))


def test_a_layer_without_feed_forward_may_keep_its_second_norm_and_filter_in_the_file():
    from swifttransformer_amd.config.fiterax_param import FiteraxHyperParam
    from swifttransformer_amd.models import build_model
    from swifttransformer_amd.weights.loader import match_specs
    cfg = tiny.CONFIGS["A"]
    model = build_model(FiteraxHyperParam.from_dict(cfg), torch.float32)
    shapes = {k: tuple(v.shape) for k, v in tiny.make_weights(cfg, 0).items()}
    match_specs(model.tensor_specs(), shapes)
    shapes.update({"l2.norm2": (cfg["width"],), "l2.canon2": (cfg["width"], cfg["canon"]["taps"])})
    match_specs(model.tensor_specs(), shapes)


def test_named_sizes():
    from swifttransformer_amd.config.registry import hyper_param_by_name
    hp = hyper_param_by_name("fiterax_1.3b", num_layers=6)
    assert hp.width == 2048 and [L["type"] for L in hp.layers] == ["mlstm", "attention", "attention"] * 2
    with pytest.raises(KeyError):
        hyper_param_by_name("fiterax_3b")
