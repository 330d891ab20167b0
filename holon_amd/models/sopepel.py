"""Sopepel: its typed configuration, and configuration to spec.

A decoder with an RMS norm on each sublayer's result and none in front of it, x += norm1(mixer(x)), x += norm2(ffn(x)),
over a residual stream kept in float32. The embedding adds to a token's row the row of a second table that the token and
the one before it choose; the head is the first table, its logits times a constant. Every layer's mixer is `parallel`: grouped-query
softmax attention (biases on all four projections, an RMS norm on every query and key head, rotary positions on the first
dimensions of a head in the half-split pairing, queries that see the keys of their own chunk of positions alone, a sigmoid
gate a head) beside gated linear attention (a decay a key channel through a low-rank projection, a matrix of key by value
a head), summed with two scales. The feed-forward is dense with a gelu gate in its tanh form, or a mixture of experts with
a squared ReLU (the largest sigmoid scores chosen, each weight multiplying its expert's input, a shared expert behind a
sigmoid gate a token), or absent.

config.json gives every size and constant; the one size it does not name (the rank of the decays' projection) is the
checkpoint tensor's, unless `rank` is given beside the linear attention's other sizes (random weights need it)."""
from __future__ import annotations

import dataclasses
import json
from collections.abc import Mapping
from typing import Any

from ..config.model import ConfigError, eos_ids
from ..config.model import config_value as _get
from ..registry import register_architecture
from ..spec import LayerSpec, ModelSpec, PartRef, WeightRule, in_order

NAME = "Sopepel"


def _check_mixer(at: str, m: Mapping[str, Any]) -> None:
    for key in ("left.heads", "left.kv_heads", "left.dim", "left.vdim", "right.heads", "right.dim", "right.vdim"):
        _get(m, key, int)
    for key in ("left.scale", "left_scale", "right_scale"):
        _get(m, key, float)
    left, right = m["left"], m["right"]
    if left["heads"] % left["kv_heads"]:
        raise ConfigError(f"{at}: left heads {left['heads']} are not a multiple of kv_heads {left['kv_heads']}")
    if left.get("mask"):
        _get(left, "mask.size", int)
    if left.get("rot"):
        dims = _get(left, "rot.dims", int)
        _get(left, "rot.base", float)
        if dims % 2 or dims > left["dim"]:
            raise ConfigError(f"{at}: rot.dims {dims} must be even and within dim {left['dim']}")
    if not _get(m, "right.tau", float) > 0:
        raise ConfigError(f"{at}: tau must be positive")
    if right.get("rank") is not None:
        _get(m, "right.rank", int)


def _check_mlp(at: str, mlp: Mapping[str, Any]) -> None:
    kind = _get(mlp, "kind")
    if kind == "dense":
        _get(mlp, "ff", int)
    elif kind == "moe":
        _get(mlp, "expert.ff", int)
        experts, top = _get(mlp, "router.experts", int), _get(mlp, "router.top", int)
        if top > experts:
            raise ConfigError(f"{at}: router.top {top} exceeds router.experts {experts}")
        if mlp.get("shared"):
            _get(mlp, "shared.ff", int)
    else:
        raise ConfigError(f"{at}: unknown feed-forward kind {kind!r} (dense, moe)")


@dataclasses.dataclass(frozen=True)
class SopepelConfig:
    width: int
    vocab: int
    eps: float
    logit_scale: float
    bigram: tuple[int, int, int] | None           # (buckets, mul_prev, mul_cur); None: the plain table alone
    layers: tuple                                 # per layer: its config.json entry (type, mixer, mlp), checked
    eos_token_ids: tuple[int, ...] = ()
    architecture: str = NAME

    @classmethod
    def from_dict(cls, c: Mapping[str, Any], generation: Mapping[str, Any] | None = None) -> "SopepelConfig":
        width, vocab = _get(c, "width", int), _get(c, "vocab", int)
        eps = _get(c, "norm.eps", float)
        scale = _get(c, "logit_scale", float) if c.get("logit_scale") is not None else 1.0
        bigram = None
        if (c.get("embedding") or {}).get("bigram"):
            buckets = _get(c, "embedding.bigram.buckets", int)
            muls = [c["embedding"]["bigram"].get(key) for key in ("mul_prev", "mul_cur")]
            if any(not isinstance(v, int) or isinstance(v, bool) for v in muls):
                raise ConfigError("embedding.bigram.mul_prev and mul_cur must be whole numbers")
            bigram = (buckets, *muls)
        layers = _get(c, "layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("`layers` must be a non-empty list")
        for i, layer in enumerate(layers):
            at = f"layers[{i}]"
            kind, m = _get(layer, "type"), _get(layer, "mixer")
            if kind != "parallel":
                raise ConfigError(f"{at}: unknown layer type {kind!r} (parallel)")
            if not isinstance(m, Mapping):
                raise ConfigError(f"{at}: `mixer` must hold the mixer's sizes")
            _check_mixer(at, m)
            if layer.get("mlp"):
                _check_mlp(at, layer["mlp"])
        return cls(width=width, vocab=vocab, eps=eps, logit_scale=scale, bigram=bigram,
                   layers=tuple(json.loads(json.dumps(layers))), eos_token_ids=eos_ids(c, generation))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "width": self.width, "vocab": self.vocab,
                               "norm": {"eps": self.eps}, "logit_scale": self.logit_scale, "layers": list(self.layers)}
        if self.bigram:
            out["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), self.bigram))}
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out


def _rules() -> tuple[WeightRule, ...]:
    left, right, ffn = "layers.{i}.mixer.left.", "layers.{i}.mixer.right.", "layers.{i}.ffn."
    rules = [WeightRule("embed", "embed.weight"), WeightRule("bigram", "embed.bigram"),
             WeightRule("final.norm", "norm.weight")]
    rules += [WeightRule(f"l{{i}}.{s}", f"layers.{{i}}.{s}.weight") for s in ("norm1", "norm2")]
    rules += [WeightRule(f"l{{i}}.mix.left.{s}.b", f"{left}{s}_bias") for s in ("q", "k", "v", "o")]
    rules += [WeightRule(f"l{{i}}.mix.left.{s}.norm", f"{left}{s}_norm") for s in ("q", "k")]
    rules += [WeightRule(f"l{{i}}.mix.left.{s}", f"{left}{s}.weight") for s in ("q", "k", "v", "g", "o")]
    rules += [WeightRule("l{i}.mix.right.a2.b", f"{right}a2_bias")]
    rules += [WeightRule(f"l{{i}}.mix.right.{s}", f"{right}{s}") for s in ("a2", "norm")]
    rules += [WeightRule(f"l{{i}}.mix.right.{s}", f"{right}{s}.weight") for s in ("q", "k", "v", "g", "a1", "o")]
    rules += [WeightRule(f"l{{i}}.mlp.e{{e}}.{s}", f"{ffn}{s}", "e") for s in ("up", "down")]
    rules += [WeightRule(f"l{{i}}.mlp.shared.{s}", f"{ffn}shared_{s}") for s in ("up", "down", "sg")]
    rules += [WeightRule("l{i}.mlp.router", f"{ffn}router")]
    rules += [WeightRule(f"l{{i}}.mlp.{s}", f"{ffn}{s}_proj.weight") for s in ("gate", "up", "down")]
    return tuple(rules)


def _mixer(c: SopepelConfig, m: Mapping[str, Any]) -> PartRef:
    left, right, rot = m["left"], m["right"], m["left"].get("rot")
    position = PartRef("position", "rope_banded", theta=float(rot["base"]), rotary_dim=rot["dims"]) if rot else None
    return PartRef(
        "mixer", "parallel", left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]),
        left=PartRef("mixer", "attention", heads=left["heads"], kv_heads=left["kv_heads"], dim=left["dim"],
                     vdim=left["vdim"], scale=float(left["scale"]), qkv_bias=True, o_bias=True, head_norm=c.eps,
                     head_gate=True, chunk=left["mask"]["size"] if left.get("mask") else 0, position=position),
        right=PartRef("mixer", "gated_linear", heads=right["heads"], dim=right["dim"], vdim=right["vdim"],
                      tau=float(right["tau"]), eps=c.eps, rank=right.get("rank")))


def _ffn(mlp: Mapping[str, Any] | None) -> PartRef | None:
    if not mlp:
        return None
    if mlp["kind"] == "dense":
        return PartRef("ffn", "swiglu", inter=mlp["ff"], act="gelu_tanh")
    shared = (mlp.get("shared") or {}).get("ff", 0)
    return PartRef("ffn", "moe", experts=mlp["router"]["experts"], top=mlp["router"]["top"], inter=mlp["expert"]["ff"],
                   score="sigmoid_top", bias=False, act="relu2", weigh_input=True, shared=shared, shared_gated=bool(shared))


def recipe(c: SopepelConfig) -> ModelSpec:
    norm = PartRef("norm", "rms32", eps=c.eps)
    block = PartRef("block", "postnorm32")
    layers = tuple(LayerSpec(block=block, mixer=_mixer(c, layer["mixer"]), ffn=_ffn(layer.get("mlp")), norm=norm)
                   for layer in c.layers)
    # a layer without feed-forward may still list the norm behind it
    skip = tuple(f"l{i}.norm2" for i, layer in enumerate(c.layers) if not layer.get("mlp"))
    embed = PartRef("embed", "table") if c.bigram is None else \
        PartRef("embed", "bigram", buckets=c.bigram[0], mul_prev=c.bigram[1], mul_cur=c.bigram[2])
    return ModelSpec(hidden=c.width, vocab=c.vocab, layers=layers, order=in_order(len(layers)), embed=embed,
                     norm=PartRef("norm", "rms32", eps=c.eps, gain=c.logit_scale), head=PartRef("head", "linear", tied=True),
                     rules=_rules(), skip=skip, eos_token_ids=c.eos_token_ids)


register_architecture(NAME, SopepelConfig, recipe)
