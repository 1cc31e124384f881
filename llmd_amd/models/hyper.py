"""Hyper-connected residual streams, for stacks whose sublayers read and write several copies of the residual.

There are S streams X_1..X_S, all equal to the embedding at the start. Every sublayer (a mixer or a
feed-forward) has three small learned tensors: ``in`` [S] reads the sublayer's input u = sum_s in[s] X_s,
``mix`` [S, S] (from, to) remixes the streams and ``out`` [S] spreads the sublayer's result over them:

    y = sublayer(norm(u));   X_t <- sum_s mix[s, t] X_s + out[t] y     (all t from the old X)

The stack's output is the norm of sum_s X_s. S = 1 with all three equal to 1 is the plain pre-norm residual.
The norm is a layer norm (weight, no bias) or an RMS norm. Streams, norms and the arithmetic between them
are fp32 in both activation types; ``X`` [S, T, d] is updated in place by one kernel per sublayer that also
produces the next sublayer's normed input.
"""
from __future__ import annotations

import torch

from llmd_amd.ops import seqmix as sm

from .mixers import _param


class HyperConnection(torch.nn.Module):
    """The three tensors of one sublayer's connection to the streams; fp32 copies for the kernels."""

    def __init__(self, S: int, learned: bool, device, dtype):
        super().__init__()
        self.learned = learned
        self.w_in = _param((S,), device, dtype, fill=1.0)
        self.w_out = _param((S,), device, dtype, fill=1.0)
        self.mix = torch.nn.Parameter(torch.eye(S, device=device, dtype=dtype), requires_grad=False)
        self.in32 = self.out32 = self.mix32 = None

    def finalize(self):
        self.in32, self.out32 = self.w_in.data.float(), self.w_out.data.float()
        self.mix32 = self.mix.data.float().contiguous()


def stream_stack(ids, table, ones, subs, final_norm, eps: float, dtype, rms: bool = False, layer_out=None):
    """Run a stack over its streams. ``subs``: (connection, norm weight, sublayer(h), ends a layer) of every
    sublayer in order; ``ones`` [S] fp32 reads the plain sum for the final norm. Returns that norm's
    output; ``layer_out``: optional list that receives the sum of the streams after every layer."""
    X = torch.empty(ones.numel(), ids.shape[0], table.shape[1], dtype=torch.float32, device=ids.device)
    sm.hyper_embed(ids, table, X)
    first_in, first_w = (subs[0][0].in32, subs[0][1]) if subs else (ones, final_norm)
    h = sm.hyper_norm(X, first_in, first_w, eps, dtype, rms)
    for i, (hc, _, fn, ends_layer) in enumerate(subs):
        nxt_in, nxt_w = (subs[i + 1][0].in32, subs[i + 1][1]) if i + 1 < len(subs) else (ones, final_norm)
        h = sm.hyper_update_norm(X, fn(h), hc.mix32, hc.out32, nxt_in, nxt_w, eps, dtype, rms)
        if ends_layer and layer_out is not None:
            layer_out.append(X.sum(0))
    return h
