"""Fefozen: a decoder of sandwich layers (a root-mean-square norm before and after each sublayer) whose mixers are gated delta
rules or latent attentions with a query latent and gated heads, with or without a learned sink, some reading the cache of an
earlier layer; feed-forwards are dense or routed experts with clamped units and identity experts.

This module turns its config.json into a ``ModelSpec`` and registers it; the parts themselves know nothing of it.  Tensor names
of the folder's safetensors file: ``embed``, ``final.norm`` and per layer i ``l<i>.norm1|norm1b|norm2|norm2b``, ``l<i>.mix.*``,
``l<i>.mlp.*``."""
from __future__ import annotations

from ..config.fefozen_param import ARCHITECTURE, FefozenHyperParam
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _norm(hp: FefozenHyperParam, name: str) -> PartSpec:
    return PartSpec("layer_norm", {"eps": hp.norm_eps, "center": False, "bias": False, "gain_offset": 1.0}, {"weight": name})


def _mixer(hp: FefozenHyperParam, kind: str, p: str, mx: dict) -> PartSpec:
    if kind == "delta":
        return PartSpec("gated_delta",
                        {"num_heads": mx["heads"], "num_qk_heads": mx["kv_heads"], "key_dim": mx["dim"], "value_dim": mx["vdim"],
                         "taps": mx["conv"], "eps": hp.norm_eps, "unit_eps": 1e-6},
                        {"q": f"{p}.q", "k": f"{p}.k", "v": f"{p}.v", "gate": f"{p}.g", "q_conv": f"{p}.q.conv",
                         "k_conv": f"{p}.k.conv", "v_conv": f"{p}.v.conv", "write": f"{p}.b", "decay": f"{p}.a",
                         "a_log": f"{p}.A_log", "dt_bias": f"{p}.dt_bias", "norm": f"{p}.norm", "out": f"{p}.o"})
    rot = mx.get("rot") or {}
    return PartSpec("gated_latent_attention",
                    {"num_heads": mx["heads"], "key_dim": mx["dim"], "value_dim": mx["vdim"], "q_rank": mx["q_rank"],
                     "rank": mx["kv_rank"], "rot_dim": mx["rot_dim"], "rot_dims": int(rot.get("dims", 0)),
                     "rot_base": float(rot.get("base", 10000.0)), "scale": float(mx["scale"]), "eps": hp.norm_eps,
                     "rot_layout": "interleaved" if kind == "latent_attention" else "halves",
                     "sink": kind == "latent_attention", "gate": True, "own_latent": mx.get("kv_from") is None},
                    {"q_down": f"{p}.dq", "q_norm": f"{p}.dq.norm", "q_up": f"{p}.uq", "down": f"{p}.dkv",
                     "down_norm": f"{p}.dkv.norm", "up_k": f"{p}.uk", "up_v": f"{p}.uv", "gate": f"{p}.g", "sink": f"{p}.sink",
                     "out": f"{p}.o"})


def _feed_forward(p: str, mlp):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return PartSpec("dense", {"inner": mlp["ff"], "activation": "gelu_tanh", "bias": False},
                        {"fc1.weight": f"{p}.up", "fc2.weight": f"{p}.down"})
    r, e = mlp["router"], mlp["expert"]
    return PartSpec("routed_experts",
                    {"experts": r["experts"], "identity": int(r.get("identity") or 0), "top": r["top"], "inner": e["ff"],
                     "style": "softmax_corrected", "clamped": True, "limit": float(e["limit"])},
                    {"router": f"{p}.router", "correction": f"{p}.correction", "gate": p + ".e{e}.gate", "up": p + ".e{e}.up",
                     "down": p + ".e{e}.down"})


def build_fefozen_spec(hp: FefozenHyperParam) -> ModelSpec:
    hp.validate()
    layers, schedule = [], []
    for i, L in enumerate(hp.layers):
        p = f"l{i}"
        ffn = _feed_forward(f"{p}.mlp", L.get("mlp"))
        unused = {} if ffn is not None else {"unused_norm": f"{p}.norm2", "unused_out_norm": f"{p}.norm2b"}
        layers.append(LayerSpec(
            arrangement=PartSpec("sandwich", {"feed_forward": ffn is not None}, unused),
            mixer_norm=_norm(hp, f"{p}.norm1"), mixer=_mixer(hp, L["type"], f"{p}.mix", L["mixer"]),
            mixer_out_norm=_norm(hp, f"{p}.norm1b"),
            ffn_norm=_norm(hp, f"{p}.norm2") if ffn is not None else None, feed_forward=ffn,
            ffn_out_norm=_norm(hp, f"{p}.norm2b") if ffn is not None else None))
        src = L["mixer"].get("kv_from")
        # (a layer that borrows reads the entries which an earlier layer of the same step has written)
        schedule.append(ScheduleEntry(layer=i, cache=i) if src is None else ScheduleEntry(layer=i, cache=src, write=False))
    return ModelSpec(
        hidden_size=hp.width, vocab_size=hp.vocab, max_positions=hp.max_positions,
        embedding=PartSpec("token", {"vocab_size": hp.vocab, "embed_dim": hp.width}, {"weight": "embed"}),
        position=PartSpec("none"),
        layers=layers, schedule=schedule,
        final_norm=_norm(hp, "final.norm"),
        head=PartSpec("linear", {"vocab_size": hp.vocab, "embed_dim": hp.width, "tied_to": "embed"}, {"weight": "head"}),
        eos_token_id=hp.eos_token_id,
    ).validate()


def _presets(name: str, **overrides) -> FefozenHyperParam:
    from ..config.presets import fefozen_preset
    return fefozen_preset(name, **overrides)


register_architecture(ARCHITECTURE, FefozenHyperParam, build_fefozen_spec, short_name="fefozen", presets=_presets)
