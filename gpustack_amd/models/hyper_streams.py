"""Parallel residual streams (hyper-connections) and the pieces that sit
between them and a sublayer, for models on the fp32 stream. The gate and the
shift are options of a model.

The residual is S streams x_1 .. x_S instead of one. A sublayer f reads a
learned combination of them and its result goes back to all of them while
the streams mix, everything from the old streams at once:

    u = sum_s a_s x_s;   y = f(norm(u));   x_t <- sum_s M[s, t] x_s + b_t y

* gate: y is multiplied element by element by sigmoid(W h + b), h = norm(u);
* token shift: the mixer reads h + (h' - h) * mu instead of h, h' the same
  row of the sequence's previous token, kept in its state slot between
  steps (engine/kv_cache.py shift_states); several mu give several such rows.

ops.stream_step closes one sublayer and opens the next in one row kernel
(gate, stream update, combination, RMS norm into the GEMM dtype; in a decode
step the token shift as well); the streams, the norm and the gate are fp32.
"""
from __future__ import annotations

import torch
from torch import nn

from .. import ops


class StreamPort(nn.Module):
    """What connects one sublayer to the streams: the weights a (read), M
    (mix, [from, to]) and b (write), the RMS norm on the way in and, with
    `gate`, the gate's bias on the way out; the gate's projection belongs to
    whoever runs its GEMM."""

    def __init__(self, width: int, streams: int, gate: bool = True):
        super().__init__()
        f32 = lambda *shape: nn.Parameter(
            torch.empty(*shape, dtype=torch.float32), requires_grad=False)
        self.read, self.write = f32(streams), f32(streams)
        self.mix = f32(streams, streams)
        self.norm = f32(width)
        self.gate_b = f32(width) if gate else None


class Streams:
    """The streams of one model step: x [T, S, W], and h [T, W], the input
    of the sublayer that is open."""

    def __init__(self, tokens, embed, scale: float, streams: int, eps: float,
                 dtype):
        T, W, dev = tokens.shape[0], embed.shape[1], tokens.device
        self.eps = eps
        self.x = torch.empty(T, streams, W, dtype=torch.float32, device=dev)
        self.h = torch.empty(T, W, dtype=dtype, device=dev)
        self._closing = None                # (port, result, gate logits)
        ops.embed_streams(self.x, tokens, embed, scale)

    def close(self, port: StreamPort, a, gate=None) -> None:
        """The open sublayer's result (and its gate's logits, if it has
        one); written by the next open / finish."""
        self._closing = (port, a, gate)

    def _step(self, read, norm, h, shift=None) -> None:
        port, a, gate = self._closing or (None, None, None)
        self._closing = None
        ops.stream_step(
            self.x, a, gate, port.gate_b if port is not None else None,
            port.mix if port is not None else None,
            port.write if port is not None else None, read, norm, self.eps, h,
            shift=shift)

    def open(self, port: StreamPort):
        self._step(port.read, port.norm, self.h)
        return self.h

    def open_shifted(self, port: StreamPort, mu, state, rg):
        """(h, h shifted towards the previous token's): [T, W] for mu [W],
        one plane [M, T, W] per row of mu [M, W]."""
        hs = torch.empty(*mu.shape[:-1], *self.h.shape, dtype=self.h.dtype,
                         device=self.h.device)
        if rg.single:
            self._step(port.read, port.norm, self.h,
                       (hs, mu, state, rg.row_seq, rg.state_slots, rg.pos32))
        else:
            self._step(port.read, port.norm, self.h)
            ops.token_shift(hs, self.h, mu, state, rg.seq_first, rg.seq_rows,
                            rg.state_slots, rg.row_seq, rg.pos32)
        return self.h, hs

    def finish(self, rows, ones, norm):
        """The streams' sum, normed, at the chosen rows (None: all)."""
        if self._closing is not None:
            self._step(None, None, None)
        if rows is not None:
            self.x = self.x[rows].contiguous()
        y = torch.empty(self.x.shape[0], self.x.shape[2], dtype=self.h.dtype,
                        device=self.x.device)
        ops.stream_step(self.x, None, None, None, None, None, ones, norm,
                        self.eps, y)
        return y
