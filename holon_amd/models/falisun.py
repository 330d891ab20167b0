"""Falisun: its typed configuration, and configuration to spec.

A decoder with a norm in front of and behind each sublayer and a learned scale a channel on what joins the stream, x +=
ls1 post1(mixer(pre1(x))), x += ls2 post2(ffn(pre2(x))), RMS norms over a residual stream kept in float32; the head is
the embedding's table. Each layer names its mixer: `latent_attention` (keys and values rebuilt from a cached low-rank
latent beside one rotated key part that all heads share, rotary positions in the half-split pairing with YaRN's
rescaling, a gate a value on the heads' results; such a layer may have no latent of its own and read the one an earlier
layer cached) or `mamba2` (the state-space dual form of Mamba-2: a short causal filter with a bias over x, B and C, one
decay a head, a matrix of state by value a head, a gate in front of the grouped RMS norm). The feed-forward is a mixture
of SiLU-gated experts (a softmax over all experts' logits, groups of neighbouring experts ranked by their best score,
the chosen scores divided by their sum, an optional shared expert), or absent. config.json gives every size and
constant."""
from __future__ import annotations

import dataclasses
import json
from collections.abc import Mapping
from typing import Any

from ..config.model import ConfigError, eos_ids
from ..config.model import config_value as _get
from ..registry import register_architecture
from ..spec import LayerSpec, ModelSpec, PartRef, Run, WeightRule

NAME = "Falisun"
MIXERS = ("latent_attention", "mamba2")


def _check_mlp(at: str, mlp: Mapping[str, Any]) -> None:
    kind = mlp.get("kind", "moe")
    if kind != "moe":
        raise ConfigError(f"{at}: unknown feed-forward kind {kind!r} (moe)")
    _get(mlp, "expert.ff", int)
    experts, top = _get(mlp, "router.experts", int), _get(mlp, "router.top", int)
    if top > experts:
        raise ConfigError(f"{at}: router.top {top} exceeds router.experts {experts}")
    groups = mlp["router"].get("groups")
    if groups:
        count, keep = _get(groups, "count", int), _get(groups, "keep", int)
        if experts % count or keep > count or top > keep * (experts // count):
            raise ConfigError(f"{at}: {experts} experts do not form {count} equal groups of which {keep} can hold the "
                              f"{top} chosen")
    if mlp.get("shared"):
        _get(mlp, "shared.ff", int)


def _check_latent(at: str, i: int, m: Mapping[str, Any], layers: list) -> None:
    for key in ("heads", "dim", "vdim", "kv_rank", "rot_dim"):
        _get(m, key, int)
    _get(m, "scale", float)
    dims = _get(m, "rot.dims", int)
    _get(m, "rot.base", float)
    if dims % 2 or dims > m["rot_dim"]:
        raise ConfigError(f"{at}: rot.dims {dims} must be even and within rot_dim {m['rot_dim']}")
    if m["rot"].get("scaling"):
        for key in ("factor", "original", "fast", "slow"):
            if not _get(m, f"rot.scaling.{key}", float) > 0:
                raise ConfigError(f"{at}: rot.scaling.{key} must be positive")
    src = m.get("kv_from")
    if src is None:
        return
    if not isinstance(src, int) or isinstance(src, bool) or not 0 <= src < i:
        raise ConfigError(f"{at}: kv_from {src!r} must name an earlier layer")
    other = layers[src]
    if other.get("type") != "latent_attention" or other["mixer"].get("kv_from") is not None:
        raise ConfigError(f"{at}: kv_from {src} must name a latent_attention layer with a latent of its own")
    if any(other["mixer"].get(key) != m.get(key) for key in ("kv_rank", "rot_dim", "rot")):
        raise ConfigError(f"{at}: layer {src}'s kv_rank, rot_dim and rot must equal this layer's")


def _check_mamba2(at: str, m: Mapping[str, Any]) -> None:
    for key in ("heads", "vdim", "state", "groups", "norm_groups", "conv"):
        _get(m, key, int)
    if m["heads"] % m["groups"]:
        raise ConfigError(f"{at}: heads {m['heads']} are not a multiple of groups {m['groups']}")
    if m["heads"] * m["vdim"] % m["norm_groups"]:
        raise ConfigError(f"{at}: {m['heads']} heads of {m['vdim']} do not form {m['norm_groups']} equal norm groups")


@dataclasses.dataclass(frozen=True)
class FalisunConfig:
    width: int
    vocab: int
    eps: float
    layers: tuple                                 # per layer: its config.json entry (type, mixer, mlp), checked
    eos_token_ids: tuple[int, ...] = ()
    architecture: str = NAME

    @classmethod
    def from_dict(cls, c: Mapping[str, Any], generation: Mapping[str, Any] | None = None) -> "FalisunConfig":
        width, vocab = _get(c, "width", int), _get(c, "vocab", int)
        eps = _get(c, "norm.eps", float)
        layers = _get(c, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("`layers` must be a non-empty list")
        for i, layer in enumerate(layers):
            at = f"layers[{i}]"
            kind, m = _get(layer, "type"), _get(layer, "mixer")
            if kind not in MIXERS:
                raise ConfigError(f"{at}: unknown layer type {kind!r} ({', '.join(MIXERS)})")
            if not isinstance(m, Mapping):
                raise ConfigError(f"{at}: `mixer` must hold the mixer's sizes")
            if kind == "mamba2":
                _check_mamba2(at, m)
            else:
                _check_latent(at, i, m, layers)
            if layer.get("mlp"):
                _check_mlp(at, layer["mlp"])
        return cls(width=width, vocab=vocab, eps=eps, layers=tuple(json.loads(json.dumps(layers))),
                   eos_token_ids=eos_ids(c, generation))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "width": self.width, "vocab": self.vocab,
                               "norm": {"eps": self.eps}, "layers": list(self.layers)}
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out


def _rules() -> tuple[WeightRule, ...]:
    mix, ffn = "layers.{i}.mixer.", "layers.{i}.ffn."
    rules = [WeightRule("embed", "embed.weight"), WeightRule("final.norm", "norm.weight")]
    rules += [WeightRule(f"l{{i}}.{s}", f"layers.{{i}}.{s}.weight") for s in ("norm1", "norm1b", "norm2", "norm2b")]
    rules += [WeightRule(f"l{{i}}.{s}", f"layers.{{i}}.{s}") for s in ("ls1", "ls2")]
    # the two mixers (o is a shared name)
    rules += [WeightRule("l{i}.mix.dkv.norm", f"{mix}dkv_norm.weight"), WeightRule("l{i}.mix.in", f"{mix}in_proj.weight"),
              WeightRule("l{i}.mix.conv.b", f"{mix}conv.bias"), WeightRule("l{i}.mix.conv", f"{mix}conv.weight")]
    rules += [WeightRule(f"l{{i}}.mix.{s}", f"{mix}{s}.weight") for s in ("q", "dkv", "g", "o")]
    rules += [WeightRule(f"l{{i}}.mix.{s}", f"{mix}{s}") for s in ("uk", "uv", "dt_bias", "A_log", "D", "norm")]
    # the feed-forward
    rules += [WeightRule(f"l{{i}}.mlp.e{{e}}.{s}", f"{ffn}{s}", "e") for s in ("gate", "up", "down")]
    rules += [WeightRule(f"l{{i}}.mlp.shared.{s}", f"{ffn}shared_{s}") for s in ("gate", "up", "down")]
    rules += [WeightRule("l{i}.mlp.router", f"{ffn}router")]
    return tuple(rules)


def _mixer(c: FalisunConfig, layer: Mapping[str, Any]) -> PartRef:
    m = layer["mixer"]
    if layer["type"] == "mamba2":
        return PartRef("mixer", "mamba2", heads=m["heads"], vdim=m["vdim"], state_dim=m["state"], groups=m["groups"],
                       norm_groups=m["norm_groups"], taps=m["conv"], eps=c.eps)
    scaling = m["rot"].get("scaling")
    position = PartRef("position", "rope_yarn", theta=float(m["rot"]["base"]), rotary_dim=m["rot"]["dims"],
                       scaling=tuple(sorted(scaling.items())) if scaling else None)
    return PartRef("mixer", "latent_attention", heads=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                   rot_dim=m["rot_dim"], position=position, scale=float(m["scale"]), gate=True, entries=1,
                   own_kv=m.get("kv_from") is None, norm=PartRef("norm", "rmsnorm", eps=c.eps))


def _ffn(mlp: Mapping[str, Any] | None) -> PartRef | None:
    if not mlp:
        return None
    router = mlp["router"]
    groups = router.get("groups") or {}
    # weights of the chosen: softmax over all, divided by the chosen ones' sum = softmax over the chosen alone
    return PartRef("ffn", "moe", experts=router["experts"], top=router["top"], inter=mlp["expert"]["ff"],
                   score="softmax_top", bias=False, groups=groups.get("count", 1), keep=groups.get("keep", 1),
                   shared=(mlp.get("shared") or {}).get("ff", 0))


def recipe(c: FalisunConfig) -> ModelSpec:
    norm = PartRef("norm", "rms32", eps=c.eps)
    block = PartRef("block", "sandwich32", layer_scale=True)
    layers, skip = [], []
    for i, layer in enumerate(c.layers):
        ffn = _ffn(layer.get("mlp"))
        layers.append(LayerSpec(block=block, mixer=_mixer(c, layer), ffn=ffn, norm=norm))
        if ffn is None:                            # a layer without feed-forward may still list what goes around it
            skip += [f"l{i}.norm2", f"l{i}.ls2"]
    # every layer runs once, so a run's place in the order is its layer's number
    order = tuple(Run(i, reads=layer["mixer"].get("kv_from")) for i, layer in enumerate(c.layers))
    return ModelSpec(hidden=c.width, vocab=c.vocab, layers=tuple(layers), order=order, embed=PartRef("embed", "table"),
                     norm=norm, head=PartRef("head", "linear", tied=True), rules=_rules(), skip=tuple(skip),
                     eos_token_ids=c.eos_token_ids)


register_architecture(NAME, FalisunConfig, recipe)
