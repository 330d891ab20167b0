"""Small Sopepel configurations and checkpoints for the tests, and the plain model behind one interface.

The tensors are drawn here, by checkpoint name, from laws that make faults visible: projections keep activations of
order one, norm weights are spread around one, biases and gates are of order one, the second table's rows are as large as
the first's, the decays' offsets spread the decays between quick and slow, a layer's experts are alike but for a fifth, and
`sharp` scales the query side so that few keys carry most of an attention's weight."""
from __future__ import annotations

import copy
import functools
import json
import pathlib
import re

import torch
from safetensors import safe_open
from safetensors.torch import save_file

from tests.plain import sopepel as plain


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def left(heads, kv_heads, dim, vdim, scale, chunk, rot, base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": chunk},
            "rot": {"dims": rot, "base": base}}


def right(heads, dim, vdim, tau, rank):
    """(`rank` is named for the tensors drawn here and for random weights; a checkpoint's tensors say it too)"""
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}


def layer(l, r, mlp=None, scales=(0.8, 1.3)):
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": l, "right": r, "left_scale": scales[0], "right_scale": scales[1]}}


def model(width, vocab, layers, *, eps=1e-6, logit_scale=0.7, bigram=(37, 5, 3)):
    return {"architecture": "Sopepel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": layers}


# A: every feed-forward; keys and values of different widths on both sides, grouped keys, chunks that end inside pages
# and at their borders, part of a head turned, head counts that fill no tile; an expert mixture without a shared expert.
CONFIG_A = model(64, 150, [
    layer(left(4, 2, 16, 12, 0.3, 10, 8, 100.0), right(3, 12, 20, 4.0, 6), moe(6, 2, 16, shared=24)),
    layer(left(6, 3, 8, 16, 0.4, 16, 4, 50.0), right(2, 24, 8, 16.0, 5), dense(96), (1.4, 0.6)),
    layer(left(5, 5, 12, 12, 0.3, 23, 12, 1000.0), right(4, 8, 8, 1.0, 3), None, (1.0, -0.7)),
    layer(left(4, 1, 16, 8, 0.3, 7, 2, 10.0), right(1, 40, 33, 8.0, 16), moe(5, 1, 24)),
    layer(left(4, 2, 16, 12, 0.3, 10, 8, 100.0), right(3, 12, 20, 4.0, 6), dense(72))])
# B: another order, eps and logit scale, wide multipliers, more experts of which more are chosen, all of a head turned,
# rows of the table whose product passes 64 bits.
CONFIG_B = model(96, 200, [
    layer(left(3, 1, 32, 32, 0.2, 64, 32, 500000.0), right(6, 16, 32, 16.0, 16), dense(128), (0.5, 0.5)),
    layer(left(6, 6, 16, 16, 0.25, 20, 6, 1000.0), right(2, 64, 48, 16.0, 12), moe(7, 3, 24, shared=40), (2.0, 1.0)),
    layer(left(2, 2, 24, 40, 0.2, 33, 8, 20.0), right(5, 8, 24, 2.5, 4), moe(4, 4, 16, shared=8))],
    eps=1e-5, logit_scale=1.6, bigram=(101, 1 << 61, 1000003))
# C: sizes that are 1 or equal: one head, a chunk of one position (a query sees its own key alone) and of two, one turned
# pair, values of one number, a rank of one, a tau, scales and a logit scale of 1, one expert, one bucket.
CONFIG_C = model(32, 50, [
    layer(left(1, 1, 8, 1, 1.0, 1, 2), right(1, 1, 1, 1.0, 1), moe(1, 1, 8, shared=8), (1.0, 1.0)),
    layer(left(1, 1, 2, 2, 1.0, 2, 2), right(1, 4, 4, 1.0, 1), dense(32), (1.0, 1.0))], logit_scale=1.0, bigram=(1, 1, 1))
# D: heads of 64 with keys and values of one width (in bfloat16 on the GPU the matrix-core attention kernels serve them)
# over chunks of 40 and of a page; values of the linear attention that take two groups of columns.
CONFIG_D = model(128, 120, [
    layer(left(4, 2, 64, 64, 0.125, 40, 32), right(2, 32, 64, 16.0, 16), dense(128)),
    layer(left(2, 2, 64, 64, 0.125, 16, 64, 100.0), right(2, 64, 144, 16.0, 16), moe(8, 2, 32, shared=32))])
# One mechanism at a time (the other mixer's scale 0, the feed-forward absent).
ONLY_ATTENTION = model(48, 90, [layer(left(4, 2, 24, 20, 0.2, 13, 12), right(1, 4, 4, 2.0, 2), None, (1.0, 0.0)),
                                layer(left(3, 1, 8, 8, 0.35, 32, 8, 20.0), right(1, 4, 4, 2.0, 2), None, (0.6, 0.0))])
ONLY_LINEAR = model(48, 90, [layer(left(1, 1, 8, 8, 0.3, 4, 4), right(3, 20, 12, 4.0, 5), None, (0.0, 1.0)),
                             layer(left(1, 1, 8, 8, 0.3, 4, 4), right(2, 8, 28, 16.0, 7), None, (0.0, 1.7))])
ONLY_DENSE = model(48, 90, [layer(left(1, 1, 8, 8, 0.3, 4, 4), right(1, 4, 4, 2.0, 2), dense(80), (0.05, 0.05))])
ONLY_MOE = model(48, 90, [layer(left(1, 1, 8, 8, 0.3, 4, 4), right(1, 4, 4, 2.0, 2), moe(12, 4, 16, shared=16), (0.05, 0.05))])


def tensor_shapes(c: dict) -> dict[str, tuple[int, ...]]:
    w = c["width"]
    out = {"embed": (c["vocab"], w), "bigram": (c["embedding"]["bigram"]["buckets"] + 1, w), "final.norm": (w,)}
    for i, one in enumerate(c["layers"]):
        p, l, r = f"l{i}.", one["mixer"]["left"], one["mixer"]["right"]
        out[p + "norm1"] = (w,)
        q = p + "mix.left."
        for name, n in (("q", l["heads"] * l["dim"]), ("k", l["kv_heads"] * l["dim"]), ("v", l["kv_heads"] * l["vdim"])):
            out.update({q + name: (n, w), f"{q}{name}.b": (n,)})
        out.update({q + "q.norm": (l["dim"],), q + "k.norm": (l["dim"],), q + "g": (l["heads"], w),
                    q + "o": (w, l["heads"] * l["vdim"]), q + "o.b": (w,)})
        q, c_, n = p + "mix.right.", r["heads"] * r["dim"], r["heads"] * r["vdim"]
        out.update({q + "q": (c_, w), q + "k": (c_, w), q + "v": (n, w), q + "g": (n, w), q + "o": (w, n),
                    q + "norm": (r["vdim"],), q + "a1": (r["rank"], w), q + "a2": (c_, r["rank"]), q + "a2.b": (c_,)})
        mlp = one.get("mlp")
        if not mlp:
            continue
        out[p + "norm2"] = (w,)
        f = p + "mlp."
        if mlp["kind"] == "dense":
            out.update({f + "gate": (mlp["ff"], w), f + "up": (mlp["ff"], w), f + "down": (w, mlp["ff"])})
        else:
            ff, experts = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(experts):
                out.update({f"{f}e{e}.up": (ff, w), f"{f}e{e}.down": (w, ff)})
            out[f + "router"] = (experts, w)
            if mlp.get("shared"):
                s = mlp["shared"]["ff"]
                out.update({f + "shared.up": (s, w), f + "shared.down": (w, s), f + "shared.sg": (1, w)})
    return out


def draw(name: str, shape: tuple[int, ...], g: torch.Generator, sharp: bool) -> torch.Tensor:
    n = lambda: torch.randn(shape, generator=g)               # noqa: E731
    last = name.split(".")[-1]
    if name.endswith("q.norm"):
        x = (2.5 if sharp else 1.0) * (1 + 0.15 * n())
    elif last in ("norm", "norm1", "norm2"):
        x = 1 + 0.2 * n()
    elif name.endswith("a2.b"):
        x = 1.5 * n()
    elif last == "b":
        x = 0.4 * n()
    elif last in ("router", "sg", "g", "a2"):
        x = 2.5 * n() * shape[-1] ** -0.5
    elif last in ("embed", "bigram"):
        x = n()
    else:
        x = n() * shape[-1] ** -0.5
    return x.bfloat16()


def make_folder(path: pathlib.Path, cfg: dict, seed: int, sharp: bool = False, edit=None) -> pathlib.Path:
    """A model folder for `cfg`. `edit(tensors)` may change the drawn tensors before they are stored."""
    path.mkdir(parents=True, exist_ok=True)
    g = torch.Generator().manual_seed(seed)
    tensors = {name: draw(name, shape, g, sharp) for name, shape in tensor_shapes(cfg).items()}
    for name in tensors:                          # a layer's experts differ by a fifth: a close call that bfloat16 rounding
        at = re.match(r"(l\d+\.mlp\.)e\d+(\.\w+)$", name)      # decides otherwise then costs little (float32 holds the choice)
        if at and f"{at[1]}e0{at[2]}" != name:
            tensors[name] = (0.98 * tensors[f"{at[1]}e0{at[2]}"].float() + 0.2 * tensors[name].float()).bfloat16()
    if edit is not None:
        edit(tensors)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(path / "model.safetensors"))
    return path


class PlainSopepel:
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
