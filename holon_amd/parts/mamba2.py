"""The state-space dual form of Mamba-2 as a mixer. One product yields z, x, B, C and a step size a head; x, B and C pass
a short causal filter with a bias and silu (`parts/convs.py`); per head h of group g, with dt = softplus(dt' + dt_bias):

    S <- exp(-exp(A_log_h) dt) S + dt B_g x_h^T,     y_h = S^T C_g + D_h x_h

S [N, V] is float32 and part of the request's slot, as are the filter's last inputs; step sizes, decays, the recurrence
and its read-out are float32. y is multiplied by silu(z), divided by its root mean square in `norm_groups` equal parts
and projected out.

HIP form: `csrc/mamba2.hip`. A step of single tokens runs filter, step size and recurrence as one kernel (`ssd_step`).
Any other step runs the filter and then `ssd_scan`, in which a head's decay is one number a token, so a run of tokens
is matrix products: tokens against each other under a triangle of decays, and each against the state in front of the
run. Rows are cut into pieces of PIECE tokens whose contributions to the state are formed side by side, a walk over a
row's pieces leaves the state in front of each, and the outputs follow, again side by side."""
from __future__ import annotations

import ctypes

import torch

from ..kernels.registry import KernelOp, register_kernel
from ..registry import register_part
from .base import FLOAT32, Build, Part, SlotState
from .convs import CausalConv, causal_conv_plain
from .linear import Linear
from .recurrent import _need, _rows, scan_pieces

_P, _I, _L, _F = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_float
_DT = {torch.float32: 0, torch.bfloat16: 1}
PIECE = 256                   # tokens a piece of a row holds
MAX_STATE = 256               # rows of S that the kernels serve


def ssd_scan_plain(xbc, dt, dt_bias, a_log, d, state, slots, starts, query_start, n_rows, heads, groups, n, vdim, pieces=None):
    """xbc [T, H V + 2 G N] (filtered x, B, C side by side), dt [T, H] (the step sizes' projection; columns of wider rows
    will do); dt_bias, a_log, d [H] float32; state [slots, H, N, V] float32, read unless the row starts at position 0,
    written back. -> y [T, H V] float32. `pieces` (what `scan_pieces` answers) lets a kernel run rows in pieces side by
    side; the result is the same but for the order of the sums."""
    t = xbc.shape[0]
    inner, gn = heads * vdim, groups * n
    x = xbc[:, :inner].float().view(t, heads, vdim)
    B = xbc[:, inner: inner + gn].float().view(t, groups, n).repeat_interleave(heads // groups, dim=1)
    C = xbc[:, inner + gn:].float().view(t, groups, n).repeat_interleave(heads // groups, dim=1)
    step = torch.nn.functional.softplus(dt.float() + dt_bias)
    decay = torch.exp(-torch.exp(a_log) * step)
    y = torch.empty((t, heads, vdim), dtype=torch.float32, device=xbc.device)
    slot_of, start_of, qs = _rows(slots, starts, query_start, n_rows)
    for b in range(n_rows):
        S = state[slot_of[b]].clone() if start_of[b] > 0 else torch.zeros_like(state[slot_of[b]])
        for i in range(qs[b], qs[b + 1]):
            S = decay[i][:, None, None] * S + (step[i][:, None] * B[i])[:, :, None] * x[i][:, None, :]
            y[i] = torch.matmul(S.transpose(1, 2).contiguous(), C[i][:, :, None])[..., 0] + d[:, None] * x[i]
        state[slot_of[b]] = S
    return y.view(t, inner)


def _ssd_scan_hip(launch, xbc, dt, dt_bias, a_log, d, state, slots, starts, query_start, n_rows, heads, groups, n, vdim,
                  pieces=None):
    t = xbc.shape[0]
    _need(xbc.is_cuda and xbc.is_contiguous() and xbc.dtype in _DT and xbc.shape[1] == heads * vdim + 2 * groups * n
          and heads % groups == 0 and dt.dtype == xbc.dtype and dt.shape == (t, heads) and dt.stride(1) == 1
          and all(v.dtype == torch.float32 and v.is_contiguous() and v.shape == (heads,) for v in (dt_bias, a_log, d))
          and state.dtype == torch.float32 and state.is_contiguous() and tuple(state.shape[1:]) == (heads, n, vdim),
          f"ssd_scan: rows {tuple(xbc.shape)}, state {tuple(state.shape)} do not fit {heads} heads in {groups} groups")
    _need(n <= MAX_STATE, f"ssd_scan: {n} state rows (at most {MAX_STATE})")
    _need(pieces is not None and pieces[0] == PIECE, f"ssd_scan: rows come in pieces of {PIECE} tokens")
    f32 = dict(dtype=torch.float32, device=xbc.device)
    y = torch.empty((t, heads * vdim), **f32)
    _, most, base, total = pieces
    sums = torch.empty((3, heads, t), **f32)                 # every token's step size and running log decay in its piece
    sloc, decay = torch.empty((total, heads, n, vdim), **f32), torch.empty((total, heads), **f32)
    launch(xbc.data_ptr(), dt.data_ptr(), dt.stride(0) if t > 1 else heads, dt_bias.data_ptr(), a_log.data_ptr(),
           d.data_ptr(), state.data_ptr(), y.data_ptr(), slots.data_ptr(), starts.data_ptr(), query_start.data_ptr(), n_rows,
           t, heads, groups, n, vdim, state.shape[0], _DT[xbc.dtype], most, base.data_ptr(), sums.data_ptr(),
           sloc.data_ptr(), decay.data_ptr())
    return y


def ssd_step_plain(proj, conv_w, conv_b, held, dt_bias, a_log, d, state, slots, starts, heads, groups, n, vdim):
    """A step of single tokens, row b being token b, from the raw projection [T, >= 2 H V + 2 G N + H]: the filter with
    silu over x, B, C (taps [C, taps], bias [C], the requests' inputs `held` [S, taps, C] as a ring), then the
    recurrence as `ssd_scan`. -> y [T, H V] float32; `held` and `state` are updated in place."""
    t = proj.shape[0]
    inner, channels = heads * vdim, heads * vdim + 2 * groups * n
    order = torch.arange(t + 1, dtype=torch.int32, device=proj.device)
    xbc = causal_conv_plain(proj[:, inner: inner + channels], conv_w, held, slots, starts, order, order[:t], t, False, True,
                            True, conv_b, True)
    return ssd_scan_plain(xbc, proj[:, inner + channels: inner + channels + heads], dt_bias, a_log, d, state, slots, starts,
                          order, t, heads, groups, n, vdim)


def _ssd_step_hip(launch, proj, conv_w, conv_b, held, dt_bias, a_log, d, state, slots, starts, heads, groups, n, vdim):
    t = proj.shape[0]
    channels, taps = heads * vdim + 2 * groups * n, conv_w.shape[1]
    _need(proj.is_cuda and proj.is_contiguous() and proj.dtype in _DT and proj.shape[1] >= heads * vdim + channels + heads
          and conv_w.dtype == proj.dtype and conv_w.is_contiguous() and conv_w.shape[0] == channels and taps <= 16
          and conv_b.dtype == proj.dtype and conv_b.is_contiguous() and conv_b.shape == (channels,)
          and held.dtype == proj.dtype and held.is_contiguous() and tuple(held.shape[1:]) == (taps, channels)
          and all(v.dtype == torch.float32 and v.is_contiguous() and v.shape == (heads,) for v in (dt_bias, a_log, d))
          and state.dtype == torch.float32 and state.is_contiguous() and tuple(state.shape[1:]) == (heads, n, vdim)
          and heads % groups == 0 and slots.shape[0] >= t and starts.shape[0] >= t,
          f"ssd_step: rows {tuple(proj.shape)}, state {tuple(state.shape)} do not fit {heads} heads in {groups} groups")
    _need(n <= MAX_STATE and vdim <= 1024, f"ssd_step: {n} state rows (at most {MAX_STATE}), values of {vdim} (at most 1024)")
    y = torch.empty((t, heads * vdim), dtype=torch.float32, device=proj.device)
    if t:
        launch(proj.data_ptr(), proj.shape[1], conv_w.data_ptr(), conv_b.data_ptr(), held.data_ptr(), dt_bias.data_ptr(),
               a_log.data_ptr(), d.data_ptr(), state.data_ptr(), y.data_ptr(), slots.data_ptr(), starts.data_ptr(), t, heads,
               groups, n, vdim, taps, state.shape[0], _DT[proj.dtype])
    return y


def gated_parts_norm_plain(y, gate, weight, parts, eps, out_dtype):
    """y [T, C] float32, gate [T, C] (columns of wider rows will do), weight [C]: u = y silu(gate); each of `parts` equal
    parts of a row of u is divided by its own root mean square (eps inside the root); times weight. float32 inside, one
    rounding to `out_dtype`."""
    g = gate.float()
    u = (y * (g * torch.sigmoid(g))).view(y.shape[0], parts, -1)
    u = u * torch.rsqrt(u.pow(2).mean(-1, keepdim=True) + eps)
    return (u.view(y.shape) * weight.float()).to(out_dtype)


def _gated_parts_norm_hip(launch, y, gate, weight, parts, eps, out_dtype):
    t, c = y.shape
    _need(y.is_cuda and y.is_contiguous() and y.dtype == torch.float32 and gate.shape == y.shape and gate.dtype in _DT
          and gate.stride(1) == 1 and weight.is_contiguous() and weight.dtype == gate.dtype and weight.shape == (c,)
          and out_dtype == gate.dtype and parts >= 1 and c % parts == 0, "gated_parts_norm: shapes do not fit")
    out = torch.empty((t, c), dtype=out_dtype, device=y.device)
    if t:
        launch(y.data_ptr(), gate.data_ptr(), gate.stride(0) if t > 1 else c, weight.data_ptr(), out.data_ptr(), t, c, parts,
               float(eps), _DT[out_dtype])
    return out


register_kernel(KernelOp("ssd_scan", ssd_scan_plain, "holon_ssd_scan",
                         [_P, _P, _L, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P, _P],
                         _ssd_scan_hip))
register_kernel(KernelOp("ssd_step", ssd_step_plain, "holon_ssd_step",
                         [_P, _I, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I], _ssd_step_hip))
register_kernel(KernelOp("gated_parts_norm", gated_parts_norm_plain, "holon_gated_parts_norm",
                         [_P, _P, _L, _P, _P, _I, _I, _I, _F, _I], _gated_parts_norm_hip))


@register_part("mixer", "mamba2")
class Mamba2(Part):
    """See the module's text. `heads` heads with values of `vdim` and a state of `state_dim` rows each, B and C shared by
    the heads of each of `groups` groups; `taps` of the filter; `norm_groups` and `eps` of the norm behind the gate."""

    graph_safe = True

    def __init__(self, build: Build, *, heads: int, vdim: int, state_dim: int, groups: int, norm_groups: int, taps: int,
                 eps: float, hidden: int, layer: int, name: str = "") -> None:
        super().__init__(build)
        if heads % groups:
            raise ValueError(f"mamba2: {heads} heads are not a multiple of {groups} groups")
        if heads * vdim % norm_groups:
            raise ValueError(f"mamba2: {heads * vdim} values do not form {norm_groups} equal norm groups")
        if state_dim > MAX_STATE:
            raise ValueError(f"mamba2: {state_dim} state rows are above {MAX_STATE}")
        self.heads, self.vdim, self.n, self.groups, self.parts, self.eps = heads, vdim, state_dim, groups, norm_groups, float(eps)
        self.inner, self.channels = heads * vdim, heads * vdim + 2 * groups * state_dim
        self.prefix = f"{name}." if name else ""
        self.attach("in_proj", Linear(build, inp=hidden, out=self.inner + self.channels + heads))
        self.attach("conv", CausalConv(build, channels=self.channels, taps=taps, silu=True, bias=True, ring=True,
                                       name=self.prefix + "conv"))
        self.attach("o", Linear(build, inp=self.inner, out=hidden))
        for nm, init in (("dt_bias", "zero"), ("A_log", "zero"), ("D", "norm")):
            self.declare(nm, (heads,), kind=FLOAT32, init=init)
        self.declare("norm", (self.inner,), init="norm")

    def state(self):
        return self.conv.state() + [SlotState(self.prefix + "S", (self.heads, self.n, self.vdim), torch.float32)]

    def finalize(self) -> None:
        """Rows of zeros pad the first product to a multiple of 16, which the few-row products ask for."""
        pad = -self.in_proj.out % 16
        if pad and self.in_proj.weight is not None:
            self.in_proj.weight = torch.cat((self.in_proj.weight, self.in_proj.weight.new_zeros((pad, self.in_proj.inp))))
            self.in_proj.out += pad
            self.in_proj.finalize()

    def forward(self, x: torch.Tensor, step, site) -> torch.Tensor:
        k = self.kernels
        proj = self.in_proj(x)
        S = site.slot_state[self.prefix + "S"]
        sizes = (self.heads, self.groups, self.n, self.vdim)
        if step.rows.in_order:                    # single tokens
            y = k.ssd_step(proj, self.conv.weight, self.conv.bias, site.slot_state[self.conv.name], self.dt_bias, self.A_log,
                           self.D, S, step.slots, step.starts, *sizes)
        else:
            xbc = self.conv(proj[:, self.inner: self.inner + self.channels], step, site)
            y = k.ssd_scan(xbc, proj[:, self.inner + self.channels: self.inner + self.channels + self.heads], self.dt_bias,
                           self.A_log, self.D, S, step.slots, step.starts, step.query_start, step.n_rows, *sizes,
                           scan_pieces(step, PIECE, 0))
        return self.o(k.gated_parts_norm(y, proj[:, : self.inner], self.norm, self.parts, self.eps, self.build.dtype))

    __call__ = forward
