"""Token embedding and the output head. std/holon_std/ops/units.py:280-348 (`Embedding`, `LMHead`). Beside the plain
table an embedding with a second table by token pair (HIP form: `csrc/bigram_embedding.hip`)."""
from __future__ import annotations

import ctypes

import torch

from ..kernels.registry import KernelOp, register_kernel
from ..registry import register_part
from ..spec import PartRef
from .base import Build, EmbedPart, Part, SlotState

_P, _I, _L = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64
_DT = {torch.float32: 0, torch.bfloat16: 1}


@register_part("embed", "table")
class Embedding(EmbedPart):
    """Rows of a table. With `norm` (any registered norm whose `forward` takes `out_dtype`) the rows go through it
    and come out in float32: the start of a residual stream that is kept in 32-bit. With `scale` the rows are
    multiplied by it, in float32, and come out in float32 as well."""

    graph_safe = True

    def __init__(self, build: Build, *, vocab: int, hidden: int, norm: PartRef | None = None,
                 scale: float | None = None) -> None:
        super().__init__(build)
        self.declare("weight", (vocab, hidden))
        self.scale = None if scale is None else float(scale)
        if self.scale is not None and norm is not None:
            raise ValueError("embed table: either a norm or a scale")
        self.norm = None
        if norm is not None:
            self.attach("norm", build.make(norm, dim=hidden))

    def rows(self, ids: torch.Tensor) -> torch.Tensor:
        return self.kernels.embedding(ids, self.weight)

    def forward(self, ids: torch.Tensor, take: tuple[torch.Tensor, torch.Tensor] | None = None,
                want_stats: bool = False):
        """Rows of the table; `take`: where a token is still on the device, see the kernel contract. With
        `want_stats`: (rows, their statistics for a norm that follows, or None)."""
        if self.scale is not None:
            rows = self.kernels.scale_rows(self.kernels.embedding(ids, self.weight, take, False), self.scale)
            return (rows, None) if want_stats else rows
        if self.norm is None:
            return self.kernels.embedding(ids, self.weight, take, want_stats)
        rows = self.norm(self.kernels.embedding(ids, self.weight, take, False), out_dtype=torch.float32)
        return (rows, None) if want_stats else rows

    __call__ = forward


def bigram_embedding_plain(ids, take, table, bigram, prev, slots, starts, query_start, token_row, n_rows, mul_prev, mul_cur,
                           in_order=False):
    """ids [T] int32 -> float32 rows table[t] + bigram[(before mul_prev + t mul_cur) mod buckets] with `before` the token
    in front of t in its sequence and buckets = bigram's rows - 1; a sequence's first token takes row `buckets`. `take` =
    (take_slot [T], last_token) or None, as for `embedding`. The token before a row's first is prev[slot] ([slots] int32)
    where the row does not start at position 0; prev[slot] becomes the row's last token. `in_order`: every row has one
    token and token t is row t."""
    if take is not None:
        ids = torch.where(take[0] >= 0, take[1][take[0].clamp(min=0).long()], ids)
    n, buckets = ids.shape[0], bigram.shape[0] - 1
    qs, first = query_start.tolist()[: n_rows + 1], starts.tolist()[:n_rows]
    before = torch.cat((ids[:1], ids[:-1])).long()
    rows = (before * mul_prev + ids.long() * mul_cur) % buckets
    for b in range(n_rows):
        lo, slot = qs[b], int(slots[b])
        rows[lo] = (int(prev[slot]) * mul_prev + int(ids[lo]) * mul_cur) % buckets if first[b] > 0 else buckets
    for b in range(n_rows):
        prev[int(slots[b])] = ids[qs[b + 1] - 1]
    return table[ids.long()].float() + bigram[rows].float()


def _bigram_embedding_hip(launch, ids, take, table, bigram, prev, slots, starts, query_start, token_row, n_rows, mul_prev,
                          mul_cur, in_order=False):
    t, width = ids.shape[0], table.shape[1]
    ok = ids.is_cuda and ids.is_contiguous() and all(x.dtype == torch.int32 for x in (ids, prev, slots, starts, query_start)) \
        and table.is_contiguous() and bigram.is_contiguous() and table.dtype in _DT and bigram.dtype == table.dtype \
        and bigram.dim() == 2 and bigram.shape[1] == width and bigram.shape[0] > 1 and prev.is_contiguous() \
        and prev.dim() == 1 and slots.shape[0] >= n_rows and starts.shape[0] >= n_rows \
        and (in_order or (token_row.dtype == torch.int32 and token_row.shape[0] >= t)) \
        and (take is None or (take[0].dtype == torch.int32 and take[1].dtype == torch.int32 and take[0].shape == ids.shape))
    if not ok:
        raise ValueError(f"bigram_embedding: ids {tuple(ids.shape)}, tables {tuple(table.shape)} and {tuple(bigram.shape)} "
                         f"{table.dtype} do not fit")
    y = torch.empty((t, width), dtype=torch.float32, device=table.device)
    launch(ids.data_ptr(), take[0].data_ptr() if take is not None else None, take[1].data_ptr() if take is not None else None,
           table.data_ptr(), bigram.data_ptr(), prev.data_ptr(), slots.data_ptr(), starts.data_ptr(), query_start.data_ptr(),
           token_row.data_ptr(), y.data_ptr(), t, n_rows, width, table.shape[0], bigram.shape[0] - 1, int(mul_prev),
           int(mul_cur), prev.shape[0], _DT[table.dtype], int(bool(in_order) and t == n_rows))
    return y


register_kernel(KernelOp("bigram_embedding", bigram_embedding_plain, "holon_bigram_embedding",
                         [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _L, _L, _I, _I, _I],
                         _bigram_embedding_hip))


@register_part("embed", "bigram")
class BigramEmbedding(EmbedPart):
    """Rows of a table plus rows of a second one (`bigram`, `buckets` + 1 rows) that the token and the one before it
    choose: row (before mul_prev + token mul_cur) mod buckets, a sequence's first token the last row. The sum is float32,
    the start of a stream that is kept in 32-bit. The token before a portion's first is part of the request's state."""

    graph_safe = True

    def __init__(self, build: Build, *, vocab: int, hidden: int, buckets: int, mul_prev: int, mul_cur: int) -> None:
        super().__init__(build)
        if buckets < 1:
            raise ValueError(f"embed bigram: {buckets} buckets")
        self.mul_prev, self.mul_cur = int(mul_prev) % buckets, int(mul_cur) % buckets      # (the same rows, and no
        self.declare("weight", (vocab, hidden))                                             # product beyond 64 bits)
        self.declare("bigram", (buckets + 1, hidden))

    def state(self):
        return [SlotState("token", (), torch.int32)]

    def forward(self, ids: torch.Tensor, take: tuple[torch.Tensor, torch.Tensor] | None = None,
                want_stats: bool = False, step=None, site=None):
        rows = self.kernels.bigram_embedding(ids, take, self.weight, self.bigram, site.slot_state["token"], step.slots,
                                             step.starts, step.query_start, step.token_row, step.n_rows, self.mul_prev,
                                             self.mul_cur, step.rows.in_order)
        return (rows, None) if want_stats else rows

    __call__ = forward


@register_part("head", "linear")
class LMHead(Part):
    """Logits in float32, optionally squashed into (-softcap, softcap). A tied head owns no tensor: it reads the
    embedding's."""

    graph_safe = True

    def __init__(self, build: Build, *, vocab: int, hidden: int, tied: bool, embed: Embedding,
                 softcap: float | None = None) -> None:
        super().__init__(build)
        self.tied = tied
        self.softcap = float(softcap) if softcap else None      # logits <- cap * tanh(logits / cap)
        self._embed = [embed]                     # in a list: the embedding part keeps the one owner of the tensor
        self.tiled: torch.Tensor | None = None
        if not tied:
            self.declare("weight", (vocab, hidden))

    def _weight(self) -> torch.Tensor:
        return self._embed[0].weight if self.tied else self.weight

    def finalize(self) -> None:
        if self.build.decode_copy and self._weight() is not None:
            self.tiled = self.kernels.tile_weight(self._weight())

    def extra_tensors(self) -> list[torch.Tensor]:
        return [self.tiled] if self.tiled is not None else []

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        logits = self.kernels.linear(h, self._weight(), torch.float32, self.tiled)
        return logits if self.softcap is None else self.kernels.softcap(logits, self.softcap)

    __call__ = forward
