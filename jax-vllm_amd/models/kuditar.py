"""Kuditar: a decoder whose layers are listed one by one in ``config.json``, each with one of three token mixers and a
feed-forward (or none), under layer norms on the sublayers' inputs; the embedding's rows carry a constant, the head is the
embedding table without it.  This file reads that configuration and turns it into a ``ModelSpec``; the mechanisms are parts
of their own:

* layers: ``parts/block.py: PreNormBlock`` with ``parts/norm.py: LayerNorm``;
* ``attention``: ``parts/attention.py`` with a weightless q/k norm, scores under a soft cap, an output gate and values blended
  with those of the first layer that blends; ``parts/rotary.py`` with one factor on every frequency;
* ``parallel``: ``parts/recurrent.py: ParallelMixer`` with norms on the results, of ``parts/attention.py`` (input biases, a
  q/k norm per head, scores under a soft cap, a window that keeps the first tokens, learned sinks) and
  ``parts/recurrent.py: GatedDeltaMixer``;
* ``parallel_2``: the same pair of ``parts/attention.py`` (input biases, a q/k norm per head, no rotation, blocks of
  positions) and ``parts/recurrent.py: GatedLinearAttention``;
* feed-forwards: ``parts/mlp.py: GatedMLP`` and ``parts/moe.py`` with the clamped activation; the experts are chosen by their
  corrected sigmoid and weighed by it times a constant.

``config.json``: ``architecture`` "Kuditar", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale`` (default 1) and ``layers``:
a list of ``{type, mixer, mlp}`` with

* type "attention": mixer ``{heads, kv_heads, dim, vdim, scale, rot: {base, dims, scaling: {factor} (optional)} (optional),
  softcap (optional), v_mix (optional)}``;
* type "parallel": mixer ``{left: {heads, kv_heads, dim, vdim, scale, rot (optional), softcap (optional), mask: {size,
  keep_first (default 0)} (optional)}, right: {heads, kv_heads, dim, vdim, conv}}``;
* type "parallel_2": mixer ``{left: {heads, kv_heads, dim, vdim, scale, softcap (optional), mask: {size} (optional)}, right:
  {heads, dim, vdim, tau, decay_rank (optional: otherwise the checkpoint's tensors give it)}}``;
* mlp ``{kind: "dense", ff, limit}``, ``{kind: "moe", router: {experts, top, scale (default 1)}, expert: {ff, limit}}`` or null.

Tensor names: ``embed``, ``final.norm``, and per layer ``l<i>.{norm1,norm2}``, ``l<i>.mix.{q,k,v,vmix,g,o}`` (attention),
``l<i>.mix.left.{q,k,v,q.norm,k.norm,sink,o,out}``, ``l<i>.mix.right.{q,k,v,q.conv,k.conv,v.conv,b,a,A_log,dt_bias,g,norm,o,out}``
or ``l<i>.mix.right.{q,k,v,a1,a2,g,norm,o,out}``, ``l<i>.mlp.{gate,up,down}`` or ``l<i>.mlp.{router,correction,e<j>.gate,
e<j>.up,e<j>.down}``; a bias has its weight's name with ``.b`` behind it.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional

from ..config.errors import ConfigError
from ..config.model import config_value, read_config_json
from ..config.registry import register_architecture
from ..parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

MIXERS = ("attention", "parallel", "parallel_2")
GLU_SLOPE = 1.702        # of the clamped activation's sigmoid


def _positive(where: str, c: Mapping, key: str) -> int:
    v = config_value(c, key, int)
    if v <= 0:
        raise ConfigError(f"{where}.{key} must be positive, got {v}")
    return v


def _positive_number(where: str, c: Mapping, key: str, required: bool = True) -> Optional[float]:
    v = config_value(c, key, float, required=required)
    if v is not None and not v > 0:
        raise ConfigError(f"{where}.{key} must be positive, got {v}")
    return v


def _section(where: str, c: Mapping, key: str, required: bool = True) -> Optional[Mapping]:
    v = c.get(key)
    if v is None:
        if required:
            raise ConfigError(f"config.json lacks {where}.{key}")
        return None
    if not isinstance(v, Mapping):
        raise ConfigError(f"{where}.{key} must be an object")
    return v


@dataclass(frozen=True)
class KuditarLayer:
    kind: str                       # one of MIXERS
    mixer: Mapping[str, Any]        # the mixer's sizes and constants, checked
    mlp: Optional[Mapping[str, Any]]


@dataclass(frozen=True)
class KuditarConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    layers: tuple
    raw: Mapping[str, Any]

    @classmethod
    def from_dict(cls, c: Mapping[str, Any]) -> "KuditarConfig":
        vocab, width = _positive("config", c, "vocab"), _positive("config", c, "width")
        eps = config_value(_section("config", c, "norm"), "eps", float)
        if not eps >= 0.0:
            raise ConfigError("norm.eps must be non-negative")
        emb = _section("config", c, "embedding", required=False) or {}
        scale = config_value(emb, "scale", float, default=1.0, required=False)
        listed = c.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json needs a non-empty list 'layers'")
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            if not isinstance(entry, Mapping):
                raise ConfigError(f"{where} must be an object")
            kind = config_value(entry, "type", str)
            if kind not in MIXERS:
                raise ConfigError(f"{where}.type {kind!r} is not one of {MIXERS}")
            m = _section(where, entry, "mixer")
            _CHECKS[kind](where + ".mixer", m)
            mlp = _section(where, entry, "mlp", required=False)
            if mlp is not None:
                _check_mlp(where + ".mlp", mlp)
            layers.append(KuditarLayer(kind, m, mlp))
        blending = {(layer.mixer["kv_heads"], layer.mixer["vdim"]) for layer in layers if _blends(layer)}
        if len(blending) > 1:
            raise ConfigError(f"layers with v_mix must agree in kv_heads and vdim, there are {sorted(blending)}")
        return cls(vocab, width, eps, scale, tuple(layers), dict(c))

    @classmethod
    def from_folder(cls, path) -> "KuditarConfig":
        return cls.from_dict(read_config_json(path))

    def to_dict(self) -> dict:
        return dict(self.raw)


def _blends(layer: KuditarLayer) -> bool:
    return layer.kind == "attention" and bool(layer.mixer.get("v_mix"))


def _check_heads(where: str, m: Mapping) -> None:
    heads, kv = _positive(where, m, "heads"), _positive(where, m, "kv_heads")
    if heads % kv:
        raise ConfigError(f"{where}.heads = {heads} is not a multiple of kv_heads = {kv}")
    _positive(where, m, "dim")
    _positive(where, m, "vdim")


def _check_softmax_attention(where: str, m: Mapping) -> None:
    _check_heads(where, m)
    _positive_number(where, m, "scale")
    _positive_number(where, m, "softcap", required=False)
    rot = _section(where, m, "rot", required=False)
    if rot is not None:
        dims = config_value(rot, "dims", int)
        if dims < 0 or dims % 2 or dims > m["dim"]:
            raise ConfigError(f"{where}.rot.dims must be even and at most dim = {m['dim']}, got {dims}")
        if not config_value(rot, "base", float) > 1.0:
            raise ConfigError(f"{where}.rot.base must be above 1")
        scaling = _section(where + ".rot", rot, "scaling", required=False)
        if scaling is not None:
            _positive_number(where + ".rot.scaling", scaling, "factor")
    mask = _section(where, m, "mask", required=False)
    if mask is not None:
        _positive(where + ".mask", mask, "size")
        if config_value(mask, "keep_first", int, default=0, required=False) < 0:
            raise ConfigError(f"{where}.mask.keep_first must not be negative")


def _check_attention(where: str, m: Mapping) -> None:
    _check_softmax_attention(where, m)
    if not isinstance(m.get("v_mix", False), bool):
        raise ConfigError(f"{where}.v_mix must be true or false")


def _check_parallel(where: str, m: Mapping) -> None:
    _check_softmax_attention(where + ".left", _section(where, m, "left"))
    right = _section(where, m, "right")
    _check_heads(where + ".right", right)
    _positive(where + ".right", right, "conv")


def _check_parallel_2(where: str, m: Mapping) -> None:
    _check_softmax_attention(where + ".left", _section(where, m, "left"))
    right = _section(where, m, "right")
    for key in ("heads", "dim", "vdim"):
        _positive(where + ".right", right, key)
    _positive_number(where + ".right", right, "tau")


_CHECKS = {"attention": _check_attention, "parallel": _check_parallel, "parallel_2": _check_parallel_2}


def _check_mlp(where: str, f: Mapping) -> None:
    kind = f.get("kind", "dense")
    if kind == "dense":
        _positive(where, f, "ff")
        _positive_number(where, f, "limit")
        return
    if kind != "moe":
        raise ConfigError(f"{where}.kind {kind!r}: this architecture's feed-forward is 'dense' or 'moe'")
    router, expert = _section(where, f, "router"), _section(where, f, "expert")
    experts, top = _positive(where + ".router", router, "experts"), _positive(where + ".router", router, "top")
    if top > experts:
        raise ConfigError(f"{where}.router.top = {top} exceeds its {experts} experts")
    config_value(router, "scale", float, default=1.0, required=False)
    _positive(where + ".expert", expert, "ff")
    _positive_number(where + ".expert", expert, "limit")


def _rotary(m: Mapping) -> Optional[PartSpec]:
    rot = m.get("rot")
    if not rot or not rot["dims"]:
        return None
    scaling = rot.get("scaling")
    return PartSpec("rotary", {"head_dim": m["dim"], "theta": float(rot["base"]), "rotary_dim": rot["dims"],
                               "linear_factor": float(scaling["factor"]) if scaling else 1.0})


def _attention_params(cfg: KuditarConfig, m: Mapping) -> dict:
    return {"hidden_size": cfg.width, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "v_head_dim": m["vdim"], "qk_norm_eps": cfg.eps, "qk_norm": "head", "scale": float(m["scale"]),
            "softcap": m.get("softcap")}


def _attention(cfg: KuditarConfig, m: Mapping, first_blend: bool):
    blend = ("first" if first_blend else "later") if m.get("v_mix") else None
    spec = PartSpec("gqa_attention", dict(_attention_params(cfg, m), position=_rotary(m), qk_norm_weight=False, output_gate=True,
                                          value_blend=blend))
    names = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate.weight": "g", "o_proj.weight": "o"}
    if blend:
        names["value_blend"] = "vmix"
    return spec, names


_SIDE_NAMES = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "q_proj.bias": "q.b", "k_proj.bias": "k.b",
               "v_proj.bias": "v.b", "q_norm.weight": "q.norm", "k_norm.weight": "k.norm", "o_proj.weight": "o"}


def _window_side(cfg: KuditarConfig, m: Mapping):
    mask = m.get("mask") or {}
    spec = PartSpec("gqa_attention", dict(_attention_params(cfg, m), position=_rotary(m), qkv_bias=True, sinks=True,
                                          window=mask.get("size"), keep_first=mask.get("keep_first") or 0 if mask else 0))
    return spec, dict(_SIDE_NAMES, sinks="sink")


def _block_side(cfg: KuditarConfig, m: Mapping):
    spec = PartSpec("gqa_attention", dict(_attention_params(cfg, m), qkv_bias=True, chunk=(m.get("mask") or {}).get("size")))
    return spec, dict(_SIDE_NAMES)


def _delta_side(cfg: KuditarConfig, m: Mapping):
    spec = PartSpec("gated_delta", {
        "hidden_size": cfg.width, "num_heads": m["heads"], "num_qk_heads": m["kv_heads"], "head_dim": m["dim"],
        "v_dim": m["vdim"], "conv_taps": m["conv"], "norm_eps": cfg.eps, "unit_eps": 1e-6})
    names = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "q_conv.weight": "q.conv",
             "k_conv.weight": "k.conv", "v_conv.weight": "v.conv", "beta_proj.weight": "b", "decay_proj.weight": "a",
             "gate.weight": "g", "norm.weight": "norm", "o_proj.weight": "o"}
    return spec, names


def _linear_side(cfg: KuditarConfig, m: Mapping):
    spec = PartSpec("gated_linear_attention", {
        "hidden_size": cfg.width, "num_heads": m["heads"], "head_dim": m["dim"], "v_dim": m["vdim"], "tau": float(m["tau"]),
        "norm_eps": cfg.eps, "decay_rank": m.get("decay_rank")})
    names = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate.weight": "g", "decay_down.weight": "a1",
             "decay_up.weight": "a2", "decay_up.bias": "a2.b", "norm.weight": "norm", "o_proj.weight": "o"}
    return spec, names


def _pair(cfg: KuditarConfig, m: Mapping, left_side, right_side):
    left, left_names = left_side(cfg, m["left"])
    right, right_names = right_side(cfg, m["right"])
    spec = PartSpec("parallel", {"left": left, "right": right, "left_scale": 0.5, "right_scale": 0.5,
                                 "out_norm_eps": cfg.eps, "hidden_size": cfg.width})
    names = {"left." + k: "left." + v for k, v in left_names.items()}
    names.update({"right." + k: "right." + v for k, v in right_names.items()})
    names.update({"left.out.weight": "left.out", "right.out.weight": "right.out"})
    return spec, names


def _mixer_spec(cfg: KuditarConfig, layer: KuditarLayer, first_blend: bool):
    """(PartSpec of the mixer, local tensor name -> name below the layer's prefix)."""
    if layer.kind == "attention":
        return _attention(cfg, layer.mixer, first_blend)
    if layer.kind == "parallel":
        return _pair(cfg, layer.mixer, _window_side, _delta_side)
    return _pair(cfg, layer.mixer, _block_side, _linear_side)


def _mlp_spec(cfg: KuditarConfig, f: Mapping):
    if f.get("kind", "dense") == "dense":
        spec = PartSpec("gated_mlp", {"hidden_size": cfg.width, "intermediate_size": f["ff"],
                                      "activation": ("clamped", float(f["limit"]), GLU_SLOPE)})
        return spec, {"gate_proj.weight": "gate", "up_proj.weight": "up", "down_proj.weight": "down"}
    router, expert = f["router"], f["expert"]
    scale = router.get("scale")
    spec = PartSpec("routed_experts", {
        "hidden_size": cfg.width, "num_experts": router["experts"], "top": router["top"], "expert_size": expert["ff"],
        "activation": ("clamped", float(expert["limit"]), GLU_SLOPE), "weight_on_input": False, "score": "sigmoid_corrected",
        "choice_correction": True, "weight_scale": 1.0 if scale is None else float(scale)})
    names = {"router.weight": "router", "router.correction": "correction"}
    for e in range(router["experts"]):
        for part in ("gate", "up", "down"):
            names[f"experts.{e}.{part}.weight"] = f"e{e}.{part}"
    return spec, names


def build_spec(cfg: KuditarConfig) -> ModelSpec:
    norm = PartSpec("layernorm", {"size": cfg.width, "eps": cfg.eps})
    first_blend = next((i for i, layer in enumerate(cfg.layers) if _blends(layer)), None)
    layers = []
    for i, layer in enumerate(cfg.layers):
        mixer, mixer_names = _mixer_spec(cfg, layer, i == first_blend)
        rename = {"mix." + k: "mix." + v for k, v in mixer_names.items()}
        ffn = None
        if layer.mlp is not None:
            ffn, ffn_names = _mlp_spec(cfg, layer.mlp)
            rename.update({"mlp." + k: "mlp." + v for k, v in ffn_names.items()})
        for name in ("norm1", "norm2"):
            rename.update({name + ".weight": name, name + ".bias": name + ".b"})
        block = PartSpec("prenorm", {"norm": norm, "mixer_norm_name": "norm1", "feed_forward_norm_name": "norm2",
                                     "has_feed_forward": ffn is not None})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ffn, block=block, mixer_prefix="mix.",
                                feed_forward_prefix="mlp.", rename=rename))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": cfg.embedding_scale}),
        embedding_prefix="embed.", final_norm=norm, final_norm_prefix="final.norm.",
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width}), head_prefix="head.",
        layers=layers, schedule=[LayerRun(i) for i in range(len(layers))], tie_head_to_embedding=True,
        rename={"embed.weight": "embed", "final.norm.weight": "final.norm", "final.norm.bias": "final.norm.b"},
    )


register_architecture("Kuditar", KuditarConfig.from_dict, build_spec)
