"""Fiterax: a decoder of layers whose mixer and feed-forward run side by side on one stream, each behind a grouped
root-mean-square norm and a short causal filter; mixers are grouped attention with turned, unit-length queries and keys,
capped scores and a gate a head, or a matrix memory with exponential gates (mLSTM); feed-forwards are routed experts
without gates, weighted by normalised sigmoids.

This module turns its config.json into a ``ModelSpec`` and registers it; the parts themselves know nothing of it.
Tensor names of the folder's safetensors file: ``embed``, ``head``, ``final.norm`` and per layer i ``l<i>.norm1|norm2``,
``l<i>.canon1|canon2``, ``l<i>.mix.*``, ``l<i>.mlp.*``."""
from __future__ import annotations

from ..config.fiterax_param import ARCHITECTURE, FiteraxHyperParam
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _norm(hp: FiteraxHyperParam, name: str) -> PartSpec:
    return PartSpec("group_rms", {"eps": hp.norm_eps, "groups": hp.norm_groups}, {"weight": name})


def _filter(hp: FiteraxHyperParam, name: str):
    return PartSpec("causal", {"taps": hp.taps}, {"weight": name}) if hp.taps else None


def _mixer(hp: FiteraxHyperParam, kind: str, p: str, mx: dict) -> PartSpec:
    if kind == "attention":
        rot = mx.get("rot") or {}
        return PartSpec("unit_qk_attention",
                        {"num_heads": mx["heads"], "num_kv_heads": mx["kv_heads"], "key_dim": mx["dim"],
                         "value_dim": mx["vdim"], "scale": float(mx["scale"]), "eps": hp.norm_eps,
                         "softcap": float(mx.get("softcap") or 0.0), "bias": True, "out_bias": True,
                         "rot_dims": int(rot.get("dims", 0)), "rot_base": float(rot.get("base", 10000.0)),
                         "head_scale": True, "gate": True, "out_scale": hp.residual_mult},
                        {"q": f"{p}.q", "q_bias": f"{p}.q.b", "k": f"{p}.k", "k_bias": f"{p}.k.b", "v": f"{p}.v",
                         "v_bias": f"{p}.v.b", "head_scale": f"{p}.temp", "gate": f"{p}.g", "out": f"{p}.o",
                         "out_bias": f"{p}.o.b"})
    return PartSpec("matrix_memory",
                    {"num_heads": mx["heads"], "key_dim": mx["dim"], "value_dim": mx["vdim"], "eps": hp.norm_eps,
                     "gate_cap": float(mx["gate_cap"]), "out_scale": hp.residual_mult},
                    {"q": f"{p}.q", "k": f"{p}.k", "v": f"{p}.v", "gate": f"{p}.g", "in_gate": f"{p}.i",
                     "in_gate_bias": f"{p}.i.b", "forget_gate": f"{p}.f", "forget_gate_bias": f"{p}.f.b",
                     "norm": f"{p}.norm", "out": f"{p}.o"})


def _feed_forward(hp: FiteraxHyperParam, p: str, mlp):
    if mlp is None:
        return None
    r = mlp["router"]
    return PartSpec("routed_experts",
                    {"experts": r["experts"], "top": r["top"], "inner": mlp["expert"]["ff"], "style": "sigmoid_output",
                     "gated": False, "scale": float(r["scale"]), "residual_scale": hp.residual_mult},
                    {"router": f"{p}.router", "correction": f"{p}.correction", "up": p + ".e{e}.up",
                     "down": p + ".e{e}.down"})


def build_fiterax_spec(hp: FiteraxHyperParam) -> ModelSpec:
    hp.validate()
    layers = []
    for i, L in enumerate(hp.layers):
        p = f"l{i}"
        ffn = _feed_forward(hp, f"{p}.mlp", L.get("mlp"))
        unused = {}
        if ffn is None:       # a file may still hold the second sublayer's norm and filter
            unused = {"unused_norm": f"{p}.norm2", "unused_filter": f"{p}.canon2"}
        layers.append(LayerSpec(
            arrangement=PartSpec("parallel_residual", {"feed_forward": ffn is not None, "taps": hp.taps}, unused),
            mixer_norm=_norm(hp, f"{p}.norm1"), mixer_conv=_filter(hp, f"{p}.canon1"),
            mixer=_mixer(hp, L["type"], f"{p}.mix", L["mixer"]),
            ffn_norm=_norm(hp, f"{p}.norm2") if ffn is not None else None,
            ffn_conv=_filter(hp, f"{p}.canon2") if ffn is not None else None,
            feed_forward=ffn))
    return ModelSpec(
        hidden_size=hp.width, vocab_size=hp.vocab, max_positions=hp.max_positions,
        embedding=PartSpec("hashed_pairs", {"vocab_size": hp.vocab, "scale": hp.embedding_scale, "buckets": 0},
                           {"weight": "embed"}),
        position=PartSpec("none"),
        layers=layers, schedule=[ScheduleEntry(layer=i, cache=i) for i in range(len(layers))],
        final_norm=_norm(hp, "final.norm"),
        head=PartSpec("linear", {"vocab_size": hp.vocab, "embed_dim": hp.width, "tied_to": None}, {"weight": "head"}),
        eos_token_id=hp.eos_token_id,
    ).validate()


def _presets(name: str, **overrides) -> FiteraxHyperParam:
    from ..config.presets import fiterax_preset
    return fiterax_preset(name, **overrides)


register_architecture(ARCHITECTURE, FiteraxHyperParam, build_fiterax_spec, short_name="fiterax", presets=_presets)
