"""Real-gated linear recurrent unit (De et al., "Griffin: Mixing Gated Linear
Recurrences with Local Attention for Efficient Language Models"): a diagonal
recurrence with one fp32 state per channel and input-dependent decays, for
ragged batches.

* ``rglru_gates``: the channels are split into equal blocks; each has two
  square matrices of its own. With ``r = sigmoid(R_b u_b + rb)`` and
  ``i = sigmoid(I_b u_b + ib)``:

      log a = -c * r * softplus(lam)          a = exp(log a)
      b     = sqrt(1 - a^2) * i * u

  ``1 - a^2`` is evaluated as ``-expm1(2 log a)`` (exact where a is near 1).
* ``diagonal_scan``: ``S <- a * S + b`` per channel from the slot's state (zero
  at a sequence's start), read out as ``S * act(gate)``.
* ``rglru_mix``: the recurrent block between its input and output projections
  (short convolution, gates, scan, gated read-out); one kernel where every
  sequence brings a single token.

Everything is fp32 whatever the storage type of u, the matrices and the gate
rows (products of 16-bit operands accumulate in fp32 and stay fp32).
"""

import torch
import torch.nn.functional as F

from .causal_conv import conv_silu_ragged

RGLRU_C = 8.0


def _sk():
    from . import serving_kernels
    return serving_kernels


def rglru_gates(u, w_r, b_r, w_i, b_i, lam, c=RGLRU_C):
    """u [T, blocks*n]; w_r, w_i [blocks, n, n] ([out, in] per block, u's
    dtype); b_r, b_i, lam [blocks*n] fp32. Returns fp32 a, b [T, blocks*n]."""
    T, W = u.shape
    blocks, n, _ = w_r.shape
    assert blocks * n == W and w_i.shape == w_r.shape
    assert w_r.dtype == w_i.dtype == u.dtype
    if u.is_cuda and _sk().enabled():
        return _sk().rglru_gates(u, w_r, b_r, w_i, b_i, lam, c)
    ub = u.float().view(T, blocks, n)

    def gate(w, bias):
        z = torch.stack([F.linear(ub[:, j], w[j].float())
                         for j in range(blocks)], 1).reshape(T, W)
        return torch.sigmoid(z + bias.float())

    log_a = -c * gate(w_r, b_r) * F.softplus(lam.float())
    b = torch.sqrt(-torch.expm1(2 * log_a)) * gate(w_i, b_i) * u.float()
    return torch.exp(log_a), b


def diagonal_scan(a, b, state, batch, gate=None, act="gelu_tanh",
                  out_dtype=torch.float32):
    """a, b [T, W] fp32; state [slots, W] fp32, updated in place; gate [T, W]
    pre-activation (may be a column slice) or None. Returns S (times
    ``act(gate)``, "gelu_tanh" or "silu") as [T, W] ``out_dtype``."""
    T, W = a.shape
    assert b.shape == (T, W) and state.shape[1:] == (W,)
    assert a.dtype == b.dtype == state.dtype == torch.float32
    if act not in ("gelu_tanh", "silu"):
        raise ValueError(f"unknown gate activation {act!r}")
    if a.is_cuda and _sk().enabled():
        return _sk().diagonal_scan(a, b, state, batch, gate, act, out_dtype)
    out = torch.empty(T, W, dtype=torch.float32, device=a.device)
    at = 0
    for slot, count in zip(batch.slots, batch.counts):
        S = state[slot]
        for t in range(at, at + count):
            S = a[t] * S + b[t]
            out[t] = S
        state[slot] = S
        at += count
    if gate is not None:
        g = gate.float()
        out = out * (F.gelu(g, approximate="tanh") if act == "gelu_tanh"
                     else F.silu(g))
    return out.to(out_dtype)


def rglru_mix(proj, conv_w, conv_b, conv_state, w_r, b_r, w_i, b_i, lam,
              state, batch, c=RGLRU_C):
    """proj [T, 2W] = y | x: ``scan(gates(conv(x))) * gelu_tanh(y)`` as [T, W]
    in proj's dtype. conv_state [slots, taps-1, W] and state [slots, W] (fp32)
    are advanced in place."""
    W = proj.shape[1] // 2
    if proj.is_cuda and _sk().enabled() and \
            _sk().rglru_step_ok(proj, batch, w_r.shape[1]):
        return _sk().rglru_step(proj, conv_w, conv_b, conv_state, w_r, b_r,
                                w_i, b_i, lam, state, batch, c)
    u = conv_silu_ragged(proj[:, W:], conv_w, conv_state, batch, conv_b,
                         proj.dtype, act=None)
    a, b = rglru_gates(u, w_r, b_r, w_i, b_i, lam, c)
    return diagonal_scan(a, b, state, batch, proj[:, :W], "gelu_tanh",
                         proj.dtype)
