"""Gated linear attention: per head a matrix S [D, V] with a decay for every key channel,

    S <- diag(alpha) S + k v^T,   o = S^T q D^(-1/2),   alpha = sigmoid(W_a2 W_a1 x + b)^(1 / tau)

read after the write; each head's o is divided by its root mean square, multiplied by a weight the heads share and by
silu(W_g x), and projected. S is a float32 `SlotState`; decays, state and read-out are float32 whatever the engine's
dtype. HIP forms of the operations: `csrc/linear_attention.hip`."""
from __future__ import annotations

import ctypes

import torch

from ..kernels.registry import KernelOp, register_kernel
from ..registry import register_part
from .base import FLOAT32, Build, Part, SlotState
from .linear import Linear
from .recurrent import MAX_KEY_DIM, _need, _rows, gated_out_plain, scan_pieces

_P, _I, _L, _F = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_float
_DT = {torch.float32: 0, torch.bfloat16: 1}
PIECE, PIECES_FROM = 128, 256     # tokens a piece of a long row; the rows that are cut into pieces


def gla_decay_plain(a, w2t, bias, tau):
    """a [T, R] (columns of wider rows will do), w2t [R, C] (the second projection, transposed), bias [C] float32 ->
    sigmoid(a w2t + bias)^(1 / tau) [T, C] float32."""
    z = a.float() @ w2t.float() + bias.float()
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def _gla_decay_hip(launch, a, w2t, bias, tau):
    (t, r), c = a.shape, w2t.shape[1]
    _need(a.is_cuda and a.stride(1) == 1 and a.dtype in _DT and w2t.is_contiguous() and w2t.dtype == a.dtype
          and w2t.shape[0] == r and bias.dtype == torch.float32 and bias.shape == (c,) and r <= 1024 and tau > 0,
          "gla_decay: shapes do not fit (rank at most 1024)")
    y = torch.empty((t, c), dtype=torch.float32, device=a.device)
    launch(a.data_ptr(), a.stride(0), w2t.data_ptr(), bias.data_ptr(), 1.0 / float(tau), y.data_ptr(), t, c, r, _DT[a.dtype])
    return y


def gla_scan_plain(q, k, v, scale, alpha, state, slots, starts, query_start, n_rows, heads, pieces=None):
    """Per row and head along the row's tokens: S <- diag(alpha) S + k v^T, o = S^T (scale q). q, k [T, H D] and v
    [T, H V] (columns of wider rows will do), alpha [T, H D] float32, state [slots, H, D, V] float32, read unless the row
    starts at position 0 and written back. -> o [T, H, V] float32. `pieces` (what `scan_pieces` answers, or None) lets a
    kernel run long rows in pieces side by side; the result is the same but for the order of the sums."""
    t, dim, vdim = q.shape[0], q.shape[1] // heads, v.shape[1] // heads
    qf, kf = q.float().reshape(t, heads, dim) * scale, k.float().reshape(t, heads, dim)
    vf, af = v.float().reshape(t, heads, vdim), alpha.view(t, heads, dim)
    out = torch.empty((t, heads, vdim), dtype=torch.float32, device=q.device)
    slot_of, start_of, qs = _rows(slots, starts, query_start, n_rows)
    for b in range(n_rows):
        S = state[slot_of[b]].clone() if start_of[b] > 0 else torch.zeros_like(state[slot_of[b]])
        for i in range(qs[b], qs[b + 1]):
            S = af[i][:, :, None] * S + kf[i][:, :, None] * vf[i][:, None, :]
            out[i] = torch.einsum("hdv,hd->hv", S, qf[i])
        state[slot_of[b]] = S
    return out


def _columns(t, *tensors) -> bool:
    """Whether the tensors are columns of the same wider rows (or of rows as far apart)."""
    strides = {x.stride(0) for x in tensors} if t > 1 else {0}
    return len(strides) == 1 and all(x.is_cuda and x.stride(1) == 1 and x.dtype == tensors[0].dtype and x.shape[0] == t
                                     for x in tensors) and tensors[0].dtype in _DT


def _gla_scan_hip(launch, q, k, v, scale, alpha, state, slots, starts, query_start, n_rows, heads, pieces=None):
    t, dim, vdim = q.shape[0], q.shape[1] // heads, v.shape[1] // heads
    _need(_columns(t, q, k, v) and k.shape == q.shape and q.shape[1] == heads * dim and v.shape[1] == heads * vdim
          and alpha.is_contiguous() and alpha.dtype == torch.float32 and alpha.shape == q.shape
          and state.is_contiguous() and state.dtype == torch.float32 and tuple(state.shape[1:]) == (heads, dim, vdim),
          "gla_scan: shapes do not fit the head counts")
    _need(dim <= MAX_KEY_DIM, f"gla_scan: key size {dim} (at most {MAX_KEY_DIM})")
    out = torch.empty((t, heads, vdim), dtype=torch.float32, device=q.device)
    extra = (0, 0, None, None, None)
    if pieces is not None:
        tokens, most, base, total = pieces
        sloc = torch.empty((total, heads, dim, vdim), dtype=torch.float32, device=q.device)
        pw = torch.empty((total, heads, dim), dtype=torch.float32, device=q.device)
        extra = (tokens, most, base.data_ptr(), sloc.data_ptr(), pw.data_ptr())
    stride = q.stride(0) if t > 1 else max(q.shape[1], v.shape[1])
    launch(q.data_ptr(), k.data_ptr(), v.data_ptr(), stride, float(scale), alpha.data_ptr(), state.data_ptr(),
           out.data_ptr(), slots.data_ptr(), starts.data_ptr(), query_start.data_ptr(), n_rows, heads, dim, vdim,
           state.shape[0], _DT[q.dtype], *extra)
    return out


def gla_step_plain(q, k, v, gate, a, scale, w2t, bias, tau, weight, eps, state, slots, starts, heads):
    """A step of single tokens (row b is token b): `gla_decay`, `gla_scan` and `gated_out` one after the other ->
    [T, H V] in q's dtype."""
    t = q.shape[0]
    order = torch.arange(t + 1, dtype=torch.int32, device=q.device)
    o = gla_scan_plain(q, k, v, scale, gla_decay_plain(a, w2t, bias, tau), state, slots, starts, order, t, heads)
    return gated_out_plain(o, gate, weight, False, eps, q.dtype)


def gla_step_serves(dim: int, vdim: int) -> bool:
    """Whether the one-kernel form serves heads of these sizes (what the library's `holon_gla_step_supported` answers)."""
    if not (0 < dim <= 256 and 0 < vdim <= 1024):
        return False
    across = -(-vdim // (4 if vdim % 4 == 0 else 1))
    return -(-dim // min(1024 // across, dim)) <= 16


def _gla_step_hip(launch, q, k, v, gate, a, scale, w2t, bias, tau, weight, eps, state, slots, starts, heads):
    t, dim, vdim, rank = q.shape[0], q.shape[1] // heads, v.shape[1] // heads, a.shape[1]
    _need(_columns(t, q, k, v, gate, a) and k.shape == q.shape and gate.shape == v.shape and q.shape[1] == heads * dim
          and v.shape[1] == heads * vdim and w2t.is_contiguous() and w2t.dtype == q.dtype
          and w2t.shape == (rank, heads * dim) and bias.dtype == torch.float32 and bias.is_contiguous()
          and bias.shape == (heads * dim,) and weight.is_contiguous() and weight.dtype == q.dtype and weight.shape == (vdim,)
          and state.is_contiguous() and state.dtype == torch.float32 and tuple(state.shape[1:]) == (heads, dim, vdim)
          and slots.shape[0] >= t and starts.shape[0] >= t and rank <= 1024 and tau > 0 and gla_step_serves(dim, vdim),
          "gla_step: shapes do not fit the head counts")
    y = torch.empty((t, heads * vdim), dtype=q.dtype, device=q.device)
    stride = q.stride(0) if t > 1 else max(q.shape[1], v.shape[1])
    launch(q.data_ptr(), k.data_ptr(), v.data_ptr(), gate.data_ptr(), a.data_ptr(), stride, float(scale), w2t.data_ptr(),
           bias.data_ptr(), 1.0 / float(tau), rank, weight.data_ptr(), float(eps), state.data_ptr(), y.data_ptr(),
           slots.data_ptr(), starts.data_ptr(), t, heads, dim, vdim, state.shape[0], _DT[q.dtype])
    return y


register_kernel(KernelOp("gla_decay", gla_decay_plain, "holon_gla_decay", [_P, _L, _P, _P, _F, _P, _I, _I, _I, _I],
                         _gla_decay_hip))
register_kernel(KernelOp("gla_scan", gla_scan_plain, "holon_gla_scan",
                         [_P, _P, _P, _L, _F, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P],
                         _gla_scan_hip))
register_kernel(KernelOp("gla_step", gla_step_plain, "holon_gla_step",
                         [_P, _P, _P, _P, _P, _L, _F, _P, _P, _F, _I, _P, _F, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I],
                         _gla_step_hip))


@register_part("mixer", "gated_linear")
class GatedLinearAttention(Part):
    """Gated linear attention (see the module's text): q and k with `heads` heads of `dim`, v and the gate with heads of
    `vdim`; the decays' projection goes through `rank` values (None: the checkpoint's a1 says how many). All five
    projections of the input are one product; an owner that merges it further (`give_projection`) hands its rows to
    `forward`. `name` prefixes the state's name among its owner's."""

    graph_safe = True

    def __init__(self, build: Build, *, heads: int, dim: int, vdim: int, tau: float, eps: float, hidden: int, layer: int,
                 rank: int | None = None, name: str = "") -> None:
        super().__init__(build)
        if dim > MAX_KEY_DIM:
            raise ValueError(f"gated_linear: key size {dim} is above {MAX_KEY_DIM}")
        if not tau > 0:
            raise ValueError(f"gated_linear: tau {tau} must be positive")
        self.heads, self.dim, self.vdim, self.tau, self.eps, self.hidden = heads, dim, vdim, float(tau), float(eps), hidden
        self.scale = dim ** -0.5
        self.state_name = f"{name}.S" if name else "S"
        for nm, out in (("q", heads * dim), ("k", heads * dim), ("v", heads * vdim), ("g", heads * vdim)):
            self.attach(nm, Linear(build, inp=hidden, out=out))
        self.attach("a1", Linear(build, inp=hidden, out=-1 if rank is None else rank))
        self.declare("a2", (heads * dim, -1 if rank is None else rank), init="tap")
        self.declare("a2_bias", (heads * dim,), kind=FLOAT32, init="zero")
        self.declare("norm", (vdim,), init="norm")
        self.attach("o", Linear(build, inp=heads * vdim, out=hidden))
        self.inp: Linear | None = None
        self.a2t: torch.Tensor | None = None
        self.rank = 0

    def state(self):
        return [SlotState(self.state_name, (self.heads, self.dim, self.vdim), torch.float32)]

    def finalize(self) -> None:
        """One product for q, k, v, the gate and the decays' first projection, padded with rows of zeros to a multiple of
        16 (every product of the framework then serves it)."""
        if self.a1.weight is None:
            return
        self.rank = self.a1.weight.shape[0]
        if self.a2.shape[1] != self.rank:
            raise ValueError(f"gated_linear: the decays' two projections have ranks {self.rank} and {self.a2.shape[1]}")
        self.a1.out = self.rank
        names = ("q", "k", "v", "g", "a1")
        pad = -sum(getattr(self, nm).out for nm in names) % 16
        if pad:
            self.a1.weight = torch.cat((self.a1.weight, self.a1.weight.new_zeros((pad, self.hidden)))).contiguous()
            self.a1.out += pad
        self.inp = Linear.merge(self.build, *(getattr(self, nm) for nm in names))
        for nm in names:
            self.drop(nm)
        self._children["inp"] = self.inp
        self.a2t = self.a2.t().contiguous()       # [rank, channels]: what the decays' kernel streams

    def extra_tensors(self):
        return [self.a2t] if self.a2t is not None else []

    def give_projection(self) -> Linear | None:
        """The product that reads the input, for an owner that merges it with others; `forward` then takes its rows."""
        inp = self.inp
        if inp is not None:
            self.drop("inp")
        return inp

    def forward(self, x: torch.Tensor, step, site, rows: torch.Tensor | None = None, at: int = 0) -> torch.Tensor:
        """`rows`: the input's projections, this mixer's from column `at` on (None: made here from `x`)."""
        k = self.kernels
        if rows is None:
            rows = self.inp(x)
        c, n = self.heads * self.dim, self.heads * self.vdim
        q, kk = rows[:, at: at + c], rows[:, at + c: at + 2 * c]
        v, gate = rows[:, at + 2 * c: at + 2 * c + n], rows[:, at + 2 * c + n: at + 2 * c + 2 * n]
        a = rows[:, at + 2 * c + 2 * n: at + 2 * c + 2 * n + self.rank]
        state = site.slot_state[self.state_name]
        if step.rows.in_order and gla_step_serves(self.dim, self.vdim):       # single tokens: one kernel
            return self.o(k.gla_step(q, kk, v, gate, a, self.scale, self.a2t, self.a2_bias, self.tau, self.norm, self.eps,
                                     state, step.slots, step.starts, self.heads))
        alpha = k.gla_decay(a, self.a2t, self.a2_bias, self.tau)
        o = k.gla_scan(q, kk, v, self.scale, alpha, state, step.slots, step.starts, step.query_start, step.n_rows,
                       self.heads, scan_pieces(step, PIECE, PIECES_FROM))
        return self.o(k.gated_out(o, gate, self.norm, False, self.eps, self.build.dtype))

    __call__ = forward
