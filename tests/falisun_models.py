"""Small Falisun configurations and checkpoints for the tests, and the plain model behind one interface.

The tensors are drawn here, by checkpoint name, from laws that make faults visible: projections keep activations of
order one, filters are far from zero, step sizes and decays range from a few tokens to hundreds, the learned scales
differ from channel to channel, gates and routers are of order one, and `sharp` scales the query side so that few keys
carry most of an attention's weight."""
from __future__ import annotations

import copy
import functools
import json
import pathlib

import torch
from safetensors import safe_open
from safetensors.torch import save_file

from tests.plain import falisun as plain


def moe(experts, top, ff, shared=None, groups=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups:
        out["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def yarn(factor, original, fast, slow):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, scaling=None, kv_from=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": {"dims": rot_dim, "base": base}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def mamba2(heads, vdim, state, groups, norm_groups, conv=4, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                    "norm_groups": norm_groups, "conv": conv}}


def model(width, vocab, layers, *, eps=1e-6):
    return {"architecture": "Falisun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


SHORT_YARN = yarn(3.0, 64, 8.0, 1.0)
# A: every mixer and branch: two layers that read the latent of layer 1, values wider than the unrotated keys, experts in
# groups and not, with and without a shared one, a layer without feed-forward; B and C shared by two heads, norm groups
# that cut across the heads.
CONFIG_A = model(64, 160, [
    mamba2(6, 8, 24, 3, 2, conv=4, mlp=moe(6, 2, 16, shared=24)),
    latent(4, 16, 8, 24, 40, 0.25, base=100.0, scaling=SHORT_YARN, mlp=moe(12, 3, 16, groups=(4, 2))),
    latent(3, 8, 8, 16, 40, 0.3, base=100.0, scaling=SHORT_YARN, kv_from=1, mlp=None),
    mamba2(4, 12, 16, 1, 3, conv=3, mlp=moe(8, 4, 24, shared=16, groups=(2, 1))),
    latent(4, 16, 8, 24, 40, 0.25, base=100.0, scaling=SHORT_YARN, kv_from=1, mlp=moe(5, 1, 16))])
# B: another order, another eps; attention first and last, plain frequencies, a state wider than the values, every expert
# chosen, one norm group, a filter of two taps.
CONFIG_B = model(96, 200, [
    latent(6, 8, 4, 8, 24, 0.35, base=500000.0, mlp=moe(4, 4, 16, shared=8)),
    mamba2(2, 40, 72, 2, 1, conv=2, mlp=moe(9, 3, 24, groups=(3, 2))),
    latent(2, 24, 16, 32, 56, 0.2, scaling=yarn(8.0, 256, 16.0, 2.0), mlp=moe(7, 3, 24, shared=40)),
    latent(2, 24, 16, 8, 56, 0.2, scaling=yarn(8.0, 256, 16.0, 2.0), kv_from=2, mlp=moe(6, 2, 16, groups=(6, 3)))], eps=1e-5)
# C: sizes that are 1 or equal: one head, one group, one state row, one tap, one expert, two rotated dimensions, a latent of
# one value, a YaRN factor of 1.
CONFIG_C = model(32, 50, [
    latent(1, 1, 2, 1, 1, 1.0, scaling=yarn(1.0, 32, 4.0, 1.0), mlp=moe(1, 1, 8, shared=8)),
    latent(1, 2, 2, 3, 1, 1.0, scaling=yarn(1.0, 32, 4.0, 1.0), kv_from=0, mlp=None),
    mamba2(1, 1, 1, 1, 1, conv=1, mlp=moe(2, 1, 8, groups=(2, 1))),
    mamba2(2, 5, 3, 1, 2, conv=4, mlp=moe(3, 3, 8, groups=(1, 1)))])
# D: sizes that are multiples of 16 and 32 (in bfloat16 on the GPU the matrix-core kernels serve them).
CONFIG_D = model(96, 120, [
    latent(4, 32, 32, 32, 96, 0.125, base=100.0, scaling=SHORT_YARN, mlp=moe(8, 2, 32, shared=32, groups=(4, 2))),
    mamba2(4, 64, 128, 2, 4, conv=4, mlp=moe(8, 2, 32)),
    latent(20, 16, 32, 16, 96, 0.15, base=100.0, scaling=SHORT_YARN, kv_from=0, mlp=moe(4, 1, 32, shared=64))])
# One mechanism at a time.
ONLY_LATENT = model(48, 90, [latent(4, 16, 8, 12, 24, 0.25, base=50.0, scaling=SHORT_YARN),
                             latent(4, 12, 8, 20, 24, 0.25, base=50.0, scaling=SHORT_YARN, kv_from=0),
                             latent(3, 8, 12, 8, 32, 0.3, base=20.0)])
ONLY_MAMBA = model(48, 90, [mamba2(4, 12, 16, 2, 2), mamba2(2, 24, 40, 1, 1, conv=3)])
ONLY_MOE = model(48, 90, [latent(1, 8, 2, 8, 8, 0.3, mlp=moe(12, 4, 16, shared=16, groups=(4, 3)))])


def tensor_shapes(c: dict) -> dict[str, tuple[int, ...]]:
    w = c["width"]
    out = {"embed": (c["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(c["layers"]):
        p, m, q = f"l{i}.", layer["mixer"], f"l{i}.mix."
        out.update({p + "norm1": (w,), p + "norm1b": (w,), p + "ls1": (w,)})
        h, v = m["heads"], m["vdim"]
        if layer["type"] == "mamba2":
            inner, channels = h * v, h * v + 2 * m["groups"] * m["state"]
            out.update({q + "in": (inner + channels + h, w), q + "conv": (channels, m["conv"]), q + "conv.b": (channels,),
                        q + "dt_bias": (h,), q + "A_log": (h,), q + "D": (h,), q + "norm": (inner,), q + "o": (w, inner)})
        else:
            out.update({q + "q": (h * (m["dim"] + m["rot_dim"]), w), q + "uk": (h * m["dim"], m["kv_rank"]),
                        q + "uv": (h * v, m["kv_rank"]), q + "g": (h * v, w), q + "o": (w, h * v)})
            if m.get("kv_from") is None:
                out.update({q + "dkv": (m["kv_rank"] + m["rot_dim"], w), q + "dkv.norm": (m["kv_rank"],)})
        mlp = layer.get("mlp")
        if not mlp:
            continue
        out.update({p + "norm2": (w,), p + "norm2b": (w,), p + "ls2": (w,)})
        f, ff, experts = p + "mlp.", mlp["expert"]["ff"], mlp["router"]["experts"]
        for e in range(experts):
            out.update({f"{f}e{e}.gate": (ff, w), f"{f}e{e}.up": (ff, w), f"{f}e{e}.down": (w, ff)})
        out[f + "router"] = (experts, w)
        if mlp.get("shared"):
            s = mlp["shared"]["ff"]
            out.update({f + "shared.gate": (s, w), f + "shared.up": (s, w), f + "shared.down": (w, s)})
    return out


def draw(name: str, shape: tuple[int, ...], g: torch.Generator, sharp: bool) -> torch.Tensor:
    n = lambda: torch.randn(shape, generator=g)               # noqa: E731
    last = name.split(".")[-1]
    if last in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
        x = 1 + 0.15 * n()
    elif last in ("ls1", "ls2"):
        x = 0.6 + 0.25 * n()
    elif last == "conv":
        x = 0.6 * n()
    elif last == "b":
        x = 0.3 * n()
    elif last == "dt_bias":
        x = -2.0 + 1.5 * n()
    elif last == "A_log":
        x = -0.5 + 1.0 * n()
    elif last == "D":
        x = 1 + 0.3 * n()
    elif last in ("router", "g"):
        x = 3.0 * n() * shape[-1] ** -0.5
    elif last == "embed":
        x = n()
    elif last == "q" and sharp:
        x = 4.0 * n() * shape[-1] ** -0.5
    else:
        x = n() * shape[-1] ** -0.5
    return x.bfloat16()


def make_folder(path: pathlib.Path, cfg: dict, seed: int, sharp: bool = False, edit=None) -> pathlib.Path:
    """A model folder for `cfg`. `edit(tensors)` may change the drawn tensors before they are stored."""
    path.mkdir(parents=True, exist_ok=True)
    g = torch.Generator().manual_seed(seed)
    tensors = {name: draw(name, shape, g, sharp) for name, shape in tensor_shapes(cfg).items()}
    if edit is not None:
        edit(tensors)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(path / "model.safetensors"))
    return path


class PlainFalisun:
    """The plain model of a folder: `logits(ids)` [T, vocab] in float64 arithmetic over the stored weights."""

    def __init__(self, folder: str | pathlib.Path, dtype: torch.dtype = torch.float64, **options) -> None:
        folder = pathlib.Path(folder)
        self.config = json.loads((folder / "config.json").read_text())
        self.dtype, self.options = dtype, options
        self.tensors = {}
        with safe_open(str(folder / "model.safetensors"), "pt") as f:
            for name in f.keys():
                self.tensors[name] = f.get_tensor(name)

    def logits(self, ids: list[int]) -> torch.Tensor:
        return self._logits(tuple(ids))

    @functools.lru_cache(maxsize=None)
    def _logits(self, ids: tuple[int, ...]) -> torch.Tensor:
        return plain.forward(self.config, self.tensors, list(ids), self.dtype, **self.options)[0].float()

    def streams(self, ids: list[int]) -> list[torch.Tensor]:
        return plain.forward(self.config, self.tensors, list(ids), self.dtype, **self.options)[1]


def variant(cfg: dict, **changes) -> dict:
    out = copy.deepcopy(cfg)
    out.update(changes)
    return out
