"""The plain Fefozen pinned by hand and by closed forms; its configuration, layout and the test models, all on the CPU."""
import copy
import math

import pytest
import torch

import plain_fefozen as plain
import tiny_fefozen as tiny

F = torch.float64


def test_norm_with_a_weight_around_zero():
    x = torch.tensor([[3.0, 4.0]], dtype=F)
    r = math.sqrt(12.5 + 0.5)
    got = plain.shifted_rms(x, torch.tensor([0.0, -1.0], dtype=F), 0.5)
    assert torch.allclose(got, torch.tensor([[3.0 / r, 0.0]], dtype=F))


def test_gelu_is_the_tanh_form():
    z = torch.linspace(-4, 4, 33, dtype=F)
    assert torch.allclose(plain.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))


def test_turned_pairs_of_both_layouts():
    x = torch.zeros(3, 6, dtype=F)
    x[:, 0], x[:, 2] = 1.0, 2.0
    a = plain.turn(x, 4, 100.0, True)            # pairs (0, 1) by the position, (2, 3) by position / 10; 4 and 5 stay
    assert torch.allclose(a[2], torch.tensor([math.cos(2), math.sin(2), 2 * math.cos(0.2), 2 * math.sin(0.2), 0, 0], dtype=F))
    b = plain.turn(x, 4, 100.0, False)           # pairs (0, 2) by the position, (1, 3) by position / 10
    u, v = 1.0, 2.0
    assert torch.allclose(b[1], torch.tensor([u * math.cos(1) - v * math.sin(1), 0, v * math.cos(1) + u * math.sin(1), 0, 0, 0], dtype=F))
    assert torch.equal(a[0], x[0]) and torch.equal(b[0], x[0])


def test_a_sink_is_one_more_term_of_the_denominator():
    s = torch.tensor([[[0.0, float("-inf")], [1.0, 1.0]]], dtype=F)
    p = plain.softmax_with_sink(s, torch.tensor([math.log(3.0)], dtype=F))
    assert torch.allclose(p[0], torch.tensor([[0.25, 0.0], [math.e / (2 * math.e + 3)] * 2], dtype=F))
    assert torch.allclose(plain.softmax_with_sink(s)[0, 1], torch.tensor([0.5, 0.5], dtype=F))
    # a large sink overflows nothing
    assert float(plain.softmax_with_sink(s, torch.tensor([900.0], dtype=F)).sum()) == 0.0


def _latent_case(scale=0.0, **extra):
    g = torch.Generator().manual_seed(1)
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "q_rank": 5, "kv_rank": 6, "scale": scale, "rot": {"dims": 2, "base": 10.0}, **extra}
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F)
    w = {"dq": rnd(5, 8), "dq.norm": rnd(5), "uq": rnd(10, 5), "dkv": rnd(8, 8), "dkv.norm": rnd(6), "uk": rnd(6, 6), "uv": rnd(8, 6),
         "g": rnd(8, 8), "o": rnd(8, 8)}
    return m, w, rnd(7, 8)


def test_latent_attention_with_a_scale_of_zero_averages_the_values():
    m, w, h = _latent_case()
    c, kr = plain.latent(h, w, m, 1e-5, True)
    got = plain.latent_attention(h, w, m, 1e-5, (c, kr), True)
    v = c @ w["uv"].T
    for t in range(7):
        want = (v[:t + 1].mean(0) * torch.sigmoid(w["g"] @ h[t])) @ w["o"].T
        assert torch.allclose(got[t], want)
    # a sink of zero counts as one more key without a value
    got = plain.latent_attention(h, w, m, 1e-5, (c, kr), True, torch.zeros(2, dtype=F))
    want = (v[:3].sum(0) / 4 * torch.sigmoid(w["g"] @ h[2])) @ w["o"].T
    assert torch.allclose(got[2], want)


def test_latent_attention_of_the_first_token_and_by_explicit_keys():
    m, w, h = _latent_case(0.7)
    for neighbours in (True, False):
        cached = plain.latent(h, w, m, 1e-5, neighbours)
        got = plain.latent_attention(h, w, m, 1e-5, cached, neighbours)
        v = cached[0] @ w["uv"].T
        assert torch.allclose(got[0], (v[0] * torch.sigmoid(w["g"] @ h[0])) @ w["o"].T)
        cq = h @ w["dq"].T
        q = ((cq / torch.sqrt((cq ** 2).mean(-1, keepdim=True) + 1e-5) * w["dq.norm"]) @ w["uq"].T).view(7, 2, 5)
        t, head = 4, 1
        keys = (cached[0] @ w["uk"].T).view(7, 2, 3)
        s = []
        for j in range(t + 1):
            a = (t - j) * 1.0                                     # the pair's angle between query and key
            raw = (h @ w["dkv"].T)[j, 6:]
            u, x = q[t, head, 3], q[t, head, 4]
            turned = u * (raw[0] * math.cos(a) + raw[1] * math.sin(a)) + x * (raw[1] * math.cos(a) - raw[0] * math.sin(a))
            s.append(0.7 * (q[t, head, :3] @ keys[j, head] + turned))
        p = torch.softmax(torch.stack(s), 0)
        o = p @ v.view(7, 2, 4)[:t + 1, head]
        mine = torch.linalg.lstsq(w["o"], got[t]).solution / torch.sigmoid(w["g"] @ h[t])
        assert torch.allclose(mine[4:], o, atol=1e-8)


def test_filter_is_causal_and_its_last_column_meets_the_token():
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=F)
    silu = lambda z: z / (1 + math.exp(-z))
    got = plain.short_filter(x, torch.tensor([[0.1, 0.02, 0.003]], dtype=F))
    assert torch.allclose(got[:, 0], torch.tensor([silu(0.003), silu(0.02 + 0.03), silu(0.1 + 0.2 + 0.3)], dtype=F))


def test_delta_memory_of_two_tokens_by_hand():
    q, k, v = (torch.tensor(t, dtype=F).view(2, 1, -1) for t in ([[1.0, 0.0], [0.6, 0.8]], [[1.0, 0.0], [0.6, 0.8]], [[2.0], [5.0]]))
    beta, g = torch.tensor([[0.5], [0.25]], dtype=F), torch.tensor([[0.9], [0.8]], dtype=F)
    o = plain.delta_memory(q, k, v, beta, g)
    assert math.isclose(float(o[0]), 1.0)                       # S = k * 0.5 * 2
    # S <- 0.8 S: [0.8, 0]; S^T k = 0.48; u = 0.25 (5 - 0.48); read along k: 0.48 + u
    assert math.isclose(float(o[1]), 0.48 + 0.25 * 4.52)
    # a strength of one stores the value exactly: reading along the same key gives it back
    o = plain.delta_memory(k, k, v, torch.ones(2, 1, dtype=F), g)
    assert torch.allclose(o.flatten(), torch.tensor([2.0, 5.0], dtype=F))


def test_chunked_form_of_the_delta_rule():
    """The triangular system that the kernels solve for a chunk, from a state that is not zero, against the recurrence."""
    g_ = torch.Generator().manual_seed(2)
    T, d, vd = 9, 4, 3
    rnd = lambda *s: torch.randn(*s, generator=g_, dtype=F)
    q, k, v = plain.unit_vector(rnd(T, 1, d)), plain.unit_vector(rnd(T, 1, d)), rnd(T, 1, vd)
    beta, g = torch.sigmoid(rnd(T, 1)), torch.sigmoid(rnd(T, 1))
    want = plain.delta_memory(q, k, v, beta, g)
    S = torch.zeros(d, vd, dtype=F)
    outs = []
    for a, e in ((0, 4), (4, 9)):
        K, Q, V, b = k[a:e, 0], q[a:e, 0], v[a:e, 0], beta[a:e]
        G = torch.cumsum(torch.log(g[a:e, 0]), 0)
        W = torch.exp(G[:, None] - G[None, :])
        A = torch.tril(b * W * (K @ K.T), -1)
        solve = lambda r: torch.linalg.solve(torch.eye(e - a, dtype=F) + A, r)
        U = solve(b * V) - solve(b * torch.exp(G)[:, None] * K) @ S
        outs.append(torch.exp(G)[:, None] * (Q @ S) + torch.tril(W * (Q @ K.T)) @ U)
        S = torch.exp(G[-1]) * S + (torch.exp(G[-1] - G)[:, None] * K).T @ U
    assert torch.allclose(torch.cat(outs), want[:, 0])


def test_routing_and_clamped_experts_by_hand():
    z = torch.log(torch.tensor([0.5, 0.3, 0.2], dtype=F))
    assert [(e, round(s, 9)) for e, s in plain.route(z, torch.zeros(3, dtype=F), 2)] == [(0, 0.5), (1, 0.3)]
    # the correction moves the choice, not the weight
    assert [(e, round(s, 9)) for e, s in plain.route(z, torch.tensor([0.0, -0.2, 0.4], dtype=F), 2)] == [(2, 0.2), (0, 0.5)]
    one = torch.ones(1, 1, dtype=F)
    h = torch.tensor([3.0], dtype=F)
    a = 2.0                                                      # the gate is cut from above, the other input on both sides
    assert math.isclose(float(plain.expert(h, one, -one, one, 2.0)), a / (1 + math.exp(-1.702 * a)) * (-2.0 + 1.0))
    a = -3.0
    assert math.isclose(float(plain.expert(h, -one, 0.1 * one, one, 2.0)), a / (1 + math.exp(-1.702 * a)) * 1.3, rel_tol=1e-12)


def test_identity_experts_give_the_input_back():
    w = {"router": torch.tensor([[0.0], [4.0]], dtype=F), "correction": torch.zeros(2, dtype=F),
         **{f"e0.{n}": torch.ones(1, 1, dtype=F) for n in ("gate", "up", "down")}}
    mlp = {"router": {"experts": 1, "identity": 1, "top": 1}, "expert": {"limit": 1.0}}
    h = torch.tensor([[1.0]], dtype=F)
    assert torch.allclose(plain.moe(h, w, mlp), torch.sigmoid(torch.tensor([[4.0]], dtype=F)))


@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_a_longer_sequence_leaves_earlier_logits_and_every_mechanism_moves_them(name):
    cfg = tiny.CONFIGS[name]
    w = tiny.make_weights(cfg, 13)
    seq = tiny.prompt(20, cfg["vocab"], 3)
    a, b = plain.logits(cfg, w, seq), plain.logits(cfg, w, seq[:11])
    assert torch.allclose(a[:11], b)
    moves = lambda change: float((plain.logits(cfg, {**w, **change}, seq) - a).abs().max())
    for key, t in w.items():
        if key.endswith("correction"):
            r = [L["mlp"]["router"] for L in cfg["layers"] if (L.get("mlp") or {}).get("kind") == "moe"][0]
            if r["top"] < t.shape[0]:                            # (else every choice is taken: nothing to correct)
                assert max(moves({key: torch.roll(t, s)}) for s in range(1, t.shape[0])) > 1e-3, key
        elif ".conv" in key:
            t = t.clone()
            t[:, :-1] = 0.0                                      # (the taps before the row's own)
            assert w[key].shape[1] == 1 or moves({key: t}) > 1e-3, key
        elif ".e" not in key:
            # (a constant on every router logit changes nothing, and one expert's weight alone goes in the norm behind)
            assert moves({key: torch.roll(t, 1, 0) if key.endswith("router") else t + 0.5}) > 1e-3, key


@pytest.mark.parametrize("name", [n for n in tiny.CONFIGS if tiny.reserved(tiny.CONFIGS[n])])
def test_no_router_choice_of_the_test_models_is_a_close_call(name, monkeypatch):
    cfg = tiny.CONFIGS[name]
    w = tiny.make_weights(cfg, 13)
    gaps, chosen = [], set()
    orig = plain.route

    def spy(z, correction, top):
        c = torch.sort(torch.softmax(z, 0) + correction, descending=True).values
        if top < c.shape[0]:
            gaps.append(float(c[top - 1] - c[top]))
        out = orig(z, correction, top)
        chosen.update(e for e, _ in out)
        return out
    monkeypatch.setattr(plain, "route", spy)
    plain.logits(cfg, w, list(range(cfg["vocab"])))
    assert not gaps or min(gaps) > 0.015, min(gaps)
    assert len(chosen) >= max(tiny.router_outputs(L["mlp"]) for L in cfg["layers"] if L["mlp"] and L["mlp"]["kind"] == "moe") - 1


@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_configuration_round_trip_spec_and_caches(name):
    from swifttransformer_amd.config.fefozen_param import FefozenHyperParam
    from swifttransformer_amd.models import build_model
    cfg = tiny.CONFIGS[name]
    hp = FefozenHyperParam.from_dict(cfg)
    assert FefozenHyperParam.from_dict(hp.to_config_dict()) == hp
    model = build_model(hp, torch.float32)
    w = tiny.make_weights(cfg, 0)
    specs = {s.name: tuple(s.shape) for s in model.tensor_specs() if not s.optional}
    assert specs == {k: tuple(v.shape) for k, v in w.items()}
    needs = model.cache_needs()
    for i, L in enumerate(cfg["layers"]):
        m, e = L["mixer"], model.schedule[i]
        if L["type"] == "delta":
            G, H = m["kv_heads"], m["heads"]
            assert needs[i].kind == "state"
            inputs = m["conv"] if m["vdim"] <= 256 else m["conv"] - 1       # (a ring, or the last ones, of the filter)
            assert needs[i].state_shape[0] >= inputs * (2 * G * m["dim"] + H * m["vdim"]) + H * m["dim"] * m["vdim"]
        elif m.get("kv_from") is None:
            assert e.write and needs[i].kind == "paged_kv" and needs[i].num_kv_heads == 1 and not needs[i].values
            assert needs[i].head_dim % 16 == 0 and needs[i].head_dim >= m["kv_rank"] + m["rot_dim"] and not needs[i].window
        else:
            assert i not in needs and not e.write and e.cache == m["kv_from"]


def test_a_layout_of_halves_is_one_of_neighbours_with_reordered_rows():
    """What the mixer does when its weights are bound: the same turned products for reordered coordinates."""
    from swifttransformer_amd.parts.gated_latent import GatedLatentAttention
    from swifttransformer_amd.parts.spec import PartSpec
    params = {"num_heads": 1, "key_dim": 4, "value_dim": 4, "q_rank": 4, "rank": 4, "rot_dim": 10, "rot_dims": 6, "rot_base": 30.0,
              "scale": 1.0, "eps": 1e-5, "rot_layout": "halves"}
    order = GatedLatentAttention(PartSpec("gated_latent_attention", params, {}), 8, torch.float32).pair_order
    assert sorted(order) == list(range(10)) and order[6:] == [6, 7, 8, 9]
    g = torch.Generator().manual_seed(0)
    x = torch.randn(7, 10, generator=g, dtype=F)
    assert torch.allclose(plain.turn(x, 6, 30.0, False)[:, order], plain.turn(x[:, order], 6, 30.0, True))


def test_configuration_errors_name_the_key():
    from swifttransformer_amd.config.fefozen_param import FefozenHyperParam
    from swifttransformer_amd.config.hyper_param import ConfigError
    base = tiny.CONFIGS["A"]

    def broken(change):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(ConfigError) as e:
            FefozenHyperParam.from_dict(cfg)
        return str(e.value)
    assert "layers[0].mixer.heads" in broken(lambda c: c["layers"][0]["mixer"].update(heads=3))
    assert "conv" in broken(lambda c: c["layers"][0]["mixer"].update(conv=9))
    assert "dim" in broken(lambda c: c["layers"][0]["mixer"].update(dim=300))
    assert "vdim" in broken(lambda c: c["layers"][0]["mixer"].pop("vdim"))
    assert "q_rank" in broken(lambda c: c["layers"][1]["mixer"].pop("q_rank"))
    assert "scale" in broken(lambda c: c["layers"][1]["mixer"].pop("scale"))
    assert "rot_dim" in broken(lambda c: c["layers"][1]["mixer"].update(kv_rank=600))
    assert "dims" in broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=12))
    assert "kv_from" in broken(lambda c: c["layers"][3]["mixer"].update(kv_from=3))
    assert "kv_from" in broken(lambda c: c["layers"][3]["mixer"].update(kv_from=2))          # of the other kind
    assert "kv_rank" in broken(lambda c: c["layers"][3]["mixer"].update(kv_rank=40))
    assert "rot" in broken(lambda c: c["layers"][3]["mixer"]["rot"].update(base=77.0))
    assert "top" in broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=9))
    assert "limit" in broken(lambda c: c["layers"][1]["mlp"]["expert"].pop("limit"))
    assert "kind" in broken(lambda c: c["layers"][1]["mlp"].update(kind="other"))
    assert "ff" in broken(lambda c: c["layers"][0]["mlp"].pop("ff"))
    assert "type" in broken(lambda c: c["layers"][0].update(type="other"))
    assert "eps" in broken(lambda c: c["norm"].pop("eps"))


def test_a_layer_without_feed_forward_may_keep_its_second_norms_in_the_file():
    from swifttransformer_amd.config.fefozen_param import FefozenHyperParam
    from swifttransformer_amd.models import build_model
    from swifttransformer_amd.weights.loader import match_specs
    cfg = tiny.CONFIGS["A"]
    model = build_model(FefozenHyperParam.from_dict(cfg), torch.float32)
    shapes = {k: tuple(v.shape) for k, v in tiny.make_weights(cfg, 0).items()}
    match_specs(model.tensor_specs(), shapes)
    shapes.update({"l3.norm2": (cfg["width"],), "l3.norm2b": (cfg["width"],)})
    match_specs(model.tensor_specs(), shapes)


def test_named_sizes():
    from swifttransformer_amd.config.registry import hyper_param_by_name
    hp = hyper_param_by_name("fefozen_1.3b", num_layers=8)
    assert hp.width == 2048 and [L["type"] for L in hp.layers] == ["delta", "delta", "latent_attention", "latent_attention_2"] * 2
    assert hp.layers[7]["mixer"]["kv_from"] == 3 and "kv_from" not in hp.layers[3]["mixer"]
    with pytest.raises(KeyError):
        hyper_param_by_name("fefozen_3b")
