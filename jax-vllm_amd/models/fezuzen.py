"""Fezuzen: a decoder whose layers are listed one by one in ``config.json``, every layer with one of two token mixers
and routed experts (or no feed-forward).  Norms on both sides of every sublayer; what a sublayer reads is its normed
input plus a short causal filter of it over time; a final norm and a linear head whose logits carry a constant.  This
file reads that configuration and turns it into a ``ModelSpec``; the mechanisms are parts of their own:

* layers: ``parts/block.py: SandwichBlock`` with ``input_taps`` (the filters' state belongs to the block);
* ``attention``: ``parts/attention.py`` with filters over time on q, k and v, rotation of adjacent pairs, values turned
  by their position and results turned back, blocks of positions instead of a window, one added to the softmax
  denominator, an output gate;
* ``latent_attention``: ``parts/latent_attention.py`` with a query latent, rescaled rotary frequencies, a sliding window,
  no gate; a layer with ``kv_from`` j has no down-projection and reads layer j's cache (``LayerRun.cache_of``);
* feed-forward: ``parts/moe.py`` with the softmax over all experts as weights, a choice limited to the best groups of
  neighbouring experts, experts without a gate (square of relu) and a shared expert;
* ``logit_scale``: a constant on the final norm's weight (the head is linear, so it is a constant on the logits).

``config.json``: ``architecture`` "Fezuzen", ``vocab``, ``width``, ``norm.eps``, ``canon.taps``, ``logit_scale`` (default 1) and
``layers``: a list of ``{type, mixer, mlp}`` with

* type "attention": mixer ``{heads, kv_heads, dim, vdim (default dim), scale, rot: {base, dims, scaling (optional)},
  conv (taps, optional), mask: {size} (optional)}``;
* type "latent_attention": mixer ``{heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot: {base, dims, scaling: {factor,
  original, fast, slow} (optional)}, mask: {size} (optional), kv_from (optional)}``;
* mlp ``{kind: "moe", router: {experts, top, groups: {count, keep} (optional)}, expert: {ff}, shared: {ff} (optional)}``
  or null.

Tensor names: ``embed``, ``final.norm``, ``head``, and per layer ``l<i>.{norm1,norm1b,norm2,norm2b,canon1,canon2}``,
``l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,g,o}`` (attention), ``l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}`` (latent
attention), ``l<i>.mlp.{router,e<j>.up,e<j>.down,shared.up,shared.down}``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping, Optional

from ..config.errors import ConfigError
from ..config.model import config_value, read_config_json
from ..config.registry import register_architecture
from ..parts.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

MIXERS = ("attention", "latent_attention")


def _positive(where: str, c: Mapping, key: str) -> int:
    v = config_value(c, key, int)
    if v <= 0:
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
class FezuzenLayer:
    kind: str                       # one of MIXERS
    mixer: Mapping[str, Any]        # the mixer's sizes and constants, checked
    mlp: Optional[Mapping[str, Any]]


@dataclass(frozen=True)
class FezuzenConfig:
    vocab: int
    width: int
    eps: float
    taps: int                       # of the filters on the sublayers' inputs
    logit_scale: float
    layers: tuple
    raw: Mapping[str, Any]

    @classmethod
    def from_dict(cls, c: Mapping[str, Any]) -> "FezuzenConfig":
        vocab, width = _positive("config", c, "vocab"), _positive("config", c, "width")
        eps = config_value(_section("config", c, "norm"), "eps", float)
        if not eps >= 0.0:
            raise ConfigError("norm.eps must be non-negative")
        taps = _positive("canon", _section("config", c, "canon"), "taps")
        scale = config_value(c, "logit_scale", float, default=1.0, required=False)
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
            (_check_attention if kind == "attention" else _check_latent)(where + ".mixer", m)
            mlp = _section(where, entry, "mlp", required=False)
            if mlp is not None:
                _check_mlp(where + ".mlp", mlp)
            layers.append(FezuzenLayer(kind, m, mlp))
        for i, layer in enumerate(layers):
            if layer.kind == "latent_attention" and layer.mixer.get("kv_from") is not None:
                _check_kv_from(i, layers)
        return cls(vocab, width, eps, taps, scale, tuple(layers), dict(c))

    @classmethod
    def from_folder(cls, path) -> "FezuzenConfig":
        return cls.from_dict(read_config_json(path))

    def to_dict(self) -> dict:
        return dict(self.raw)


def _check_rot(where: str, m: Mapping, most: int) -> None:
    rot = _section(where, m, "rot", required=most > 0)
    if rot is None:
        return
    dims = config_value(rot, "dims", int)
    if dims < 0 or dims % 2 or dims > most:
        raise ConfigError(f"{where}.rot.dims must be even and at most {most}, got {dims}")
    if not config_value(rot, "base", float) > 1.0:
        raise ConfigError(f"{where}.rot.base must be above 1")
    s = _section(where + ".rot", rot, "scaling", required=False)
    if s is not None:
        for key in ("factor", "original", "fast", "slow"):
            if not config_value(s, key, float) > 0:
                raise ConfigError(f"{where}.rot.scaling.{key} must be positive")


def _check_common(where: str, m: Mapping) -> None:
    if not config_value(m, "scale", float) > 0:
        raise ConfigError(f"{where}.scale must be positive")
    mask = _section(where, m, "mask", required=False)
    if mask is not None:
        _positive(where + ".mask", mask, "size")


def _check_attention(where: str, m: Mapping) -> None:
    heads, kv = _positive(where, m, "heads"), _positive(where, m, "kv_heads")
    if heads % kv:
        raise ConfigError(f"{where}.heads = {heads} is not a multiple of kv_heads = {kv}")
    dim = _positive(where, m, "dim")
    vdim = config_value(m, "vdim", int, default=dim, required=False)
    if vdim <= 0 or vdim % 2 or dim % 2:
        raise ConfigError(f"{where}: dim and vdim turn in pairs, so they are positive and even, not {dim} and {vdim}")
    if m.get("conv") is not None:
        _positive(where, m, "conv")
    _check_rot(where, m, dim)
    _check_common(where, m)


def _check_latent(where: str, m: Mapping) -> None:
    for key in ("heads", "dim", "vdim", "q_rank", "kv_rank"):
        _positive(where, m, key)
    rot_dim = config_value(m, "rot_dim", int)
    if rot_dim < 0:
        raise ConfigError(f"{where}.rot_dim must not be negative")
    _check_rot(where, m, rot_dim)
    _check_common(where, m)
    if m.get("kv_from") is not None:
        config_value(m, "kv_from", int)


def _check_kv_from(i: int, layers: list) -> None:
    m = layers[i].mixer
    j = m["kv_from"]
    where = f"layers[{i}].mixer.kv_from"
    if not 0 <= j < i:
        raise ConfigError(f"{where} = {j} must name an earlier layer")
    other = layers[j]
    if other.kind != "latent_attention" or other.mixer.get("kv_from") is not None:
        raise ConfigError(f"{where} = {j}: that layer keeps no latent cache of its own")
    for key in ("kv_rank", "rot_dim", "rot"):
        if other.mixer.get(key) != m.get(key):
            raise ConfigError(f"{where} = {j}: {key} differs between the two layers")


def _check_mlp(where: str, f: Mapping) -> None:
    kind = f.get("kind", "moe")
    if kind != "moe":
        raise ConfigError(f"{where}.kind {kind!r}: this architecture's feed-forward is 'moe' or null")
    router = _section(where, f, "router")
    experts, top = _positive(where + ".router", router, "experts"), _positive(where + ".router", router, "top")
    if top > experts:
        raise ConfigError(f"{where}.router.top = {top} exceeds its {experts} experts")
    groups = _section(where + ".router", router, "groups", required=False)
    if groups is not None:
        count, keep = _positive(where + ".router.groups", groups, "count"), _positive(where + ".router.groups", groups, "keep")
        if experts % count or keep > count or keep * (experts // count) < top:
            raise ConfigError(f"{where}.router.groups: {top} of {experts} experts cannot come from the best {keep} of {count} equal groups")
    _positive(where + ".expert", _section(where, f, "expert"), "ff")
    shared = _section(where, f, "shared", required=False)
    if shared is not None:
        _positive(where + ".shared", shared, "ff")


def _rotary(rot: Optional[Mapping], head_dim: int) -> Optional[PartSpec]:
    if not rot or not rot["dims"]:
        return None
    s = rot.get("scaling")
    rescale = {key: float(s[key]) for key in ("factor", "original", "fast", "slow")} if s else None
    return PartSpec("rotary", {"head_dim": head_dim, "theta": float(rot["base"]), "rotary_dim": rot["dims"], "interleaved": True,
                               "rescale": rescale})


def _mixer_spec(cfg: FezuzenConfig, layer: FezuzenLayer):
    """(PartSpec of the mixer, local tensor name -> name below the layer's prefix)."""
    m = layer.mixer
    size = (m.get("mask") or {}).get("size")
    if layer.kind == "attention":
        vdim = m.get("vdim", m["dim"])
        taps = m.get("conv")
        spec = PartSpec("gqa_attention", {
            "hidden_size": cfg.width, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "v_head_dim": vdim, "scale": float(m["scale"]), "position": _rotary(m["rot"], m["dim"]), "chunk": size,
            "filter_taps": taps, "softmax_plus_one": True, "output_gate": True,
            "value_position": PartSpec("rotary", {"head_dim": vdim, "theta": float(m["rot"]["base"]), "interleaved": True})})
        names = {"q_proj.weight": "q", "k_proj.weight": "k", "v_proj.weight": "v", "gate.weight": "g", "o_proj.weight": "o"}
        if taps:
            names.update({f"{s}_filter.weight": f"{s}.conv" for s in "qkv"})
        return spec, names
    own = m.get("kv_from") is None
    spec = PartSpec("latent_attention", {
        "hidden_size": cfg.width, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"], "v_dim": m["vdim"],
        "q_rank": m["q_rank"], "kv_rank": m["kv_rank"], "scale": float(m["scale"]), "norm_eps": cfg.eps,
        "position": _rotary(m.get("rot"), m["rot_dim"]), "window": size, "output_gate": None, "own_cache": own})
    names = {"q_down.weight": "dq", "q_norm.weight": "dq.norm", "q_up.weight": "uq", "k_up.weight": "uk", "v_up.weight": "uv",
             "o_proj.weight": "o"}
    if own:
        names.update({"kv_down.weight": "dkv", "kv_norm.weight": "dkv.norm"})
    return spec, names


def _mlp_spec(cfg: FezuzenConfig, f: Mapping):
    router, shared = f["router"], f.get("shared")
    groups = router.get("groups")
    spec = PartSpec("routed_experts", {
        "hidden_size": cfg.width, "num_experts": router["experts"], "top": router["top"], "expert_size": f["expert"]["ff"],
        "activation": "relu2", "gated": False, "weight_on_input": False, "score": "softmax",
        "groups": (groups["count"], groups["keep"]) if groups else None,
        "shared": PartSpec("dense_mlp", {"hidden_size": cfg.width, "intermediate_size": shared["ff"], "activation": "relu2",
                                         "bias": False}) if shared else None})
    names = {"router.weight": "router"}
    for e in range(router["experts"]):
        for part in ("up", "down"):
            names[f"experts.{e}.{part}.weight"] = f"e{e}.{part}"
    if shared:
        names.update({f"shared.{part}_proj.weight": f"shared.{part}" for part in ("up", "down")})
    return spec, names


def build_spec(cfg: FezuzenConfig) -> ModelSpec:
    norm = PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.eps})
    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        mixer, mixer_names = _mixer_spec(cfg, layer)
        rename = {"mix." + k: "mix." + v for k, v in mixer_names.items()}
        ffn = None
        if layer.mlp is not None:
            ffn, ffn_names = _mlp_spec(cfg, layer.mlp)
            rename.update({"mlp." + k: "mlp." + v for k, v in ffn_names.items()})
        for name in ("norm1", "norm1b", "norm2", "norm2b", "canon1", "canon2"):
            rename[name + ".weight"] = name
        block = PartSpec("sandwich", {"norm": norm, "has_feed_forward": ffn is not None, "input_taps": cfg.taps,
                                      "hidden_size": cfg.width})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ffn, block=block, mixer_prefix="mix.",
                                feed_forward_prefix="mlp.", rename=rename))
        schedule.append(LayerRun(i, cache_of=layer.mixer.get("kv_from") if layer.kind == "latent_attention" else None))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width}), embedding_prefix="embed.",
        final_norm=PartSpec("rmsnorm", {"size": cfg.width, "eps": cfg.eps, "gain": cfg.logit_scale}),
        final_norm_prefix="final.norm.",
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": cfg.width}),
        head_prefix="head.", layers=layers, schedule=schedule,
        rename={"embed.weight": "embed", "final.norm.weight": "final.norm", "head.weight": "head"},
    )


register_architecture("Fezuzen", FezuzenConfig.from_dict, build_spec)
