"""A short causal filter over time on every channel, with the inputs it still needs kept per request.

y_t[c] = act(sum_j w[c, j] * x_(t - taps + 1 + j)[c] (+ x_t[c])), the last column weighing the current token and
zeros standing before a sequence's first token; optionally a bias a channel joins the sum in front of the activation. A
request's last taps - 1 inputs live in its slot
(`SlotState [taps - 1, channels]`, oldest first, in the engine's dtype), so a portion of a prompt or a single decoded
token continues exactly where the step before stopped. With `ring` the slot holds `taps` inputs, that of position p at
place p % taps: a token's own place is then none of those it reads, so the blocks of a kernel that each need some
channel's old inputs need not wait for the one that stores the new input. HIP form: `csrc/recurrent.hip`."""
from __future__ import annotations

import ctypes

import torch

from ..kernels.registry import KernelOp, register_kernel
from .base import Build, Part, SlotState

_P, _I, _L = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64
_DT = {torch.float32: 0, torch.bfloat16: 1}


def causal_conv_plain(x, weight, state, slots, starts, query_start, token_row, n_rows, add_input, silu, in_order=False,
                      bias=None, ring=False):
    """x [T, C] (columns of wider rows will do), weight [C, taps], state [S, taps - 1, C] (`ring`: [S, taps, C], the
    input of position p at p % taps; updated in place), rows as the step lists them
    (slots/starts [B], query_start [B + 1]), bias [C] or None. float32 arithmetic, taps added oldest first, then the
    bias, one rounding. `in_order`:
    every row has one token and token t is row t (a kernel may then do everything in one launch)."""
    taps = weight.shape[1]
    y = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    w = weight.float()
    qs, slot_of, start_of = query_start.tolist(), slots.tolist(), starts.tolist()
    for b in range(n_rows):
        lo, hi = qs[b], qs[b + 1]
        held, start = state[slot_of[b]], start_of[b]
        if ring:                                   # positions start - taps + 1 .. start - 1, zeros before the sequence
            before = range(start - taps + 1, start)
            held = held[[p % taps for p in before]] * torch.tensor([[p >= 0] for p in before], device=x.device).view(-1, 1)
        old = held.float() if start > 0 else torch.zeros_like(held, dtype=torch.float32)
        seq = torch.cat((old, x[lo:hi].float()), dim=0)              # [taps - 1 + n, C]
        acc = torch.zeros((hi - lo, x.shape[1]), dtype=torch.float32, device=x.device)
        for j in range(taps):
            acc = acc + w[:, j] * seq[j: j + hi - lo]
        if bias is not None:
            acc = acc + bias.float()
        if add_input:
            acc = acc + x[lo:hi].float()
        if silu:
            acc = acc * torch.sigmoid(acc)
        y[lo:hi] = acc.to(x.dtype)
        if ring:
            for p in range(max(0, start + hi - lo - taps), start + hi - lo):
                if p >= start - (taps - 1):
                    state[slot_of[b], p % taps] = seq[p - start + taps - 1].to(state.dtype)
        elif taps > 1:
            state[slot_of[b]] = seq[seq.shape[0] - (taps - 1):].to(state.dtype)
    return y


def _causal_conv_hip(launch, x, weight, state, slots, starts, query_start, token_row, n_rows, add_input, silu,
                     in_order=False, bias=None, ring=False):
    t, c = x.shape
    taps = weight.shape[1]
    if not (x.is_cuda and x.stride(1) == 1 and (t <= 1 or x.stride(0) >= c) and x.dtype in _DT and weight.dtype == x.dtype
            and weight.is_contiguous()
            and weight.shape[0] == c and state.dtype == x.dtype and state.is_contiguous()
            and tuple(state.shape[1:]) == (taps if ring else taps - 1, c) and 1 <= taps <= 16
            and (bias is None or (bias.dtype == x.dtype and bias.is_contiguous() and bias.shape == (c,)))):
        raise ValueError(f"causal_conv: rows {tuple(x.shape)}, taps {tuple(weight.shape)}, state {tuple(state.shape)} "
                         "(contiguous, one dtype, 1 to 16 taps)")
    y = torch.empty((t, c), dtype=x.dtype, device=x.device)
    launch(x.data_ptr(), x.stride(0) if t > 1 else c, weight.data_ptr(), None if bias is None else bias.data_ptr(),
           state.data_ptr(), y.data_ptr(), slots.data_ptr(), starts.data_ptr(),
           query_start.data_ptr(), token_row.data_ptr(), t, n_rows, c, taps, state.shape[0], int(add_input), int(silu),
           _DT[x.dtype], int(bool(in_order) and t == n_rows), int(bool(ring)))
    return y


register_kernel(KernelOp("causal_conv", causal_conv_plain, "holon_causal_conv",
                         [_P, _L, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I],
                         _causal_conv_hip))


class CausalConv(Part):
    """The filter as a part: `weight` [channels, taps]; `add_input` adds the input to the filter's output,
    `silu` applies x * sigmoid(x) last; `bias` gives every channel one. `name` is the name of its state among its
    owner's, `ring` its form (see the module's text)."""

    graph_safe = True

    def __init__(self, build: Build, *, channels: int, taps: int, add_input: bool = False, silu: bool = False,
                 name: str = "conv", bias: bool = False, ring: bool = False) -> None:
        super().__init__(build)
        if not 1 <= taps <= 16:
            raise ValueError(f"a causal filter has 1 to 16 taps, got {taps}")
        self.channels, self.taps, self.add_input, self.silu, self.name = channels, int(taps), add_input, silu, name
        self.declare("weight", (channels, taps), init="tap")
        self.bias, self.ring = None, bool(ring)
        if bias:
            self.declare("bias", (channels,), init="zero")

    def state(self):
        return [SlotState(self.name, (self.taps if self.ring else self.taps - 1, self.channels))]

    def forward(self, x: torch.Tensor, step, site) -> torch.Tensor:
        return self.kernels.causal_conv(x, self.weight, site.slot_state[self.name], step.slots, step.starts,
                                        step.query_start, step.token_row, step.n_rows, self.add_input, self.silu,
                                        step.rows.in_order, self.bias, self.ring)

    __call__ = forward
