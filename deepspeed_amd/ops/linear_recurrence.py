"""Linear recurrences with a matrix state per head, for ragged batches.

A head carries ``S`` ([dim, vdim], fp32, one per request slot). Per token, in
this order:

    S <- decay * S                  decay: one number per head, or one per key
                                    channel (it then scales the rows of S)
    u  = v                          plain form ("gla")
    u  = beta * (v - S^T k)         delta-rule form (beta given)
    S <- S + k u^T
    o  = S^T q                      (sees this token's write)

so a step that brings only a portion of a sequence continues from the slot's
state exactly where the previous step stopped, and a result cannot depend on
where a sequence was cut. Everything is fp32; q/k/v may arrive in the compute
dtype (they are projections) and are widened on load.

Around the scan:

* ``delta_prep``: the gated delta rule's inputs from its fused projection
  (short convolution + SiLU on q, k, v with carried tails; q and k scaled to
  unit length per head; ``beta = sigmoid(b)``;
  ``decay = exp(-exp(A_log) * softplus(a + dt_bias))``).
* ``ssd_prep``: the scalar-decay state-space form's inputs from its fused
  projection ``z | x | B | C | dt`` (short convolution with bias + SiLU on
  x|B|C with carried tails; ``dt = softplus(dt + dt_bias)``;
  ``decay = exp(-exp(A_log) * dt)``; the scan's ``v`` is ``dt * x``, its keys
  are B and its queries C, shared by the heads of a group).
* ``gate_group_norm``: the read-out plus the skip ``D * x``, times
  ``silu(gate)``, then an RMS norm over equal parts of the row, times a weight.
* ``sigmoid_pow``: ``sigmoid(z + bias) ** (1 / tau)`` for per-channel decays.
* ``softplus_decay``: ``exp(-exp(A_log_h) * softplus(z + bias))`` per head and
  key channel (the delta rule with a decay of its own for every row of S).
* ``head_norm_gate``: per-head RMS norm of the read-out times a weight shared
  by the heads (or none), times ``silu(gate)`` or ``sigmoid(gate)``.
* ``retention_prep``: queries and keys of a retention layer (the plain form
  with one fixed decay per head): partial rotary positions, keys scaled.
* ``retention_mix``: a retention layer between its input and output
  projections (prologue, recurrence, normed and gated read-out); one kernel
  where every sequence brings a single token.
"""

import torch
import torch.nn.functional as F

from .causal_conv import conv_silu_ragged
from .rope import rope_half_, rope_interleaved_

UNIT_EPS = 1e-6


def _sk():
    from . import serving_kernels
    return serving_kernels


def unit_heads(x, scale=1.0):
    """x [T, n, d] fp32 -> x / sqrt(sum(x^2) + 1e-6) * scale per head."""
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + UNIT_EPS) * scale


def delta_prep(proj, batch, conv_w, conv_state, a_log, dt_bias, kv_heads,
               heads, dim, vdim, beta_col=None, a_col=None):
    """proj [T, ...] starts with q | k | v; by default the row goes on
    ``| gate | b | a`` (the gate columns are left for ``head_norm_gate``).
    ``beta_col`` / ``a_col`` name the first of the ``heads`` columns of b and
    of a in other layouts; ``a_col=-1`` makes no per-head decay here (the
    caller has one per key channel, see ``softplus_decay``) and returns None
    for it. conv_w [2*kv_heads*dim + heads*vdim, taps] and
    conv_state [slots, taps-1, same] cover the q|k|v columns.
    Returns fp32 q [T, kv_heads, dim] (unit length times dim^-1/2),
    k [T, kv_heads, dim] (unit length), v [T, heads, vdim], beta [T, heads],
    decay [T, heads]."""
    T = proj.shape[0]
    nqk, nv = kv_heads * dim, heads * vdim
    C = 2 * nqk + nv
    if beta_col is None:
        assert proj.shape[1] == C + nv + 2 * heads
        beta_col = C + nv
    if a_col is None:
        a_col = beta_col + heads
    assert conv_w.shape[0] == C
    if proj.is_cuda and _sk().enabled():
        return _sk().delta_prep(proj, batch, conv_w, conv_state, a_log,
                                dt_bias, kv_heads, heads, dim, vdim,
                                beta_col, a_col)
    y = conv_silu_ragged(proj[:, :C], conv_w, conv_state, batch)
    q = unit_heads(y[:, :nqk].reshape(T, kv_heads, dim), dim ** -0.5)
    k = unit_heads(y[:, nqk:2 * nqk].reshape(T, kv_heads, dim))
    v = y[:, 2 * nqk:].reshape(T, heads, vdim)
    beta = torch.sigmoid(proj[:, beta_col:beta_col + heads].float())
    decay = None
    if a_col >= 0:
        dt = F.softplus(proj[:, a_col:a_col + heads].float()
                        + dt_bias.float())
        decay = torch.exp(-torch.exp(a_log.float()) * dt)
    return q.contiguous(), k.contiguous(), v.contiguous(), beta, decay


def softplus_decay(z, bias, a_log, heads):
    """Per head and key channel: ``exp(-exp(a_log_h) * softplus(z + bias))``
    in fp32. z [T, heads*dim] (a projection, may be a column slice),
    bias [heads*dim], a_log [heads]. Returns [T, heads, dim]."""
    if z.is_cuda and _sk().enabled():
        return _sk().softplus_decay(z, bias, a_log, heads)
    T, C = z.shape
    dt = F.softplus(z.float() + bias.float()).view(T, heads, C // heads)
    return torch.exp(-torch.exp(a_log.float())[None, :, None] * dt)


def sigmoid_pow(z, bias, inv_tau):
    """``sigmoid(z + bias) ** inv_tau`` in fp32, evaluated as
    ``exp(inv_tau * log_sigmoid(.))``."""
    if z.is_cuda and _sk().enabled():
        return _sk().sigmoid_pow(z, bias, inv_tau)
    return torch.exp(inv_tau * F.logsigmoid(z.float() + bias.float()))


def linear_scan(q, k, v, decay, beta, state, batch, q_scale=1.0):
    """q, k [T, G, dim]; v [T, H, vdim] (head h reads q/k head h // (H/G));
    decay fp32: [T, H] or [T, H, dim], or [H] (one fixed number per head);
    beta [T, H] fp32 or None;
    state [slots, H, dim, vdim] fp32, updated in place. q, k, v may be
    strided views (last axis contiguous); q and k share a dtype, v may have
    another. Returns o [T, H, vdim] fp32."""
    T, G, dim = q.shape
    H, vdim = v.shape[1], v.shape[2]
    assert H % G == 0 and state.dtype == torch.float32
    assert state.shape[1:] == (H, dim, vdim)
    assert decay.shape in ((H,), (T, H), (T, H, dim))
    if q.is_cuda and _sk().enabled():
        return _sk().linear_scan(q, k, v, decay, beta, state, batch, q_scale)
    rep = H // G
    qf = (q.float() * q_scale).repeat_interleave(rep, 1)
    kf = k.float().repeat_interleave(rep, 1)
    vf = v.float()
    dec = decay.float()
    if dec.dim() == 1:
        dec = dec.expand(T, H)
    dec = dec[:, :, None, None] if dec.dim() == 2 else dec[:, :, :, None]
    out = torch.empty(T, H, vdim, dtype=torch.float32, device=q.device)
    at = 0
    for slot, count in zip(batch.slots, batch.counts):
        S = state[slot]
        for t in range(at, at + count):
            S = dec[t] * S
            u = vf[t]
            if beta is not None:
                u = beta[t, :, None] * (u - torch.einsum("hdv,hd->hv", S,
                                                         kf[t]))
            S = S + kf[t][:, :, None] * u[:, None, :]
            out[t] = torch.einsum("hdv,hd->hv", S, qf[t])
        state[slot] = S
        at += count
    return out


def head_norm_gate(o, weight, gate, eps, out_dtype, act="silu",
                   out_scale=1.0, out=None):
    """o [T, H, vdim] fp32; weight [vdim] or None (no weight); gate
    [T, H*vdim] pre-activation (may be a column slice). Returns
    ``o / sqrt(mean_v(o^2) + eps) * weight * act(gate) * out_scale`` as
    [T, H*vdim] ``out_dtype``; ``act`` is "silu" or "sigmoid"; ``out`` (a view
    with contiguous rows) receives the result when given."""
    T, H, vdim = o.shape
    if out is None:
        out = torch.empty(T, H * vdim, dtype=out_dtype, device=o.device)
    assert out.shape == (T, H * vdim) and out.stride(1) == 1 \
        and out.dtype == out_dtype
    if act not in ("silu", "sigmoid"):
        raise ValueError(f"unknown gate activation {act!r}")
    if o.is_cuda and _sk().enabled():
        return _sk().head_norm_gate(o, weight, gate, eps, act, out_scale, out)
    y = o * torch.rsqrt(o.pow(2).mean(-1, keepdim=True) + eps)
    if weight is not None:
        y = y * weight.float()
    g = F.silu(gate.float()) if act == "silu" else torch.sigmoid(gate.float())
    out.copy_(y.reshape(T, H * vdim) * g * out_scale)
    return out


def ssd_prep(proj, batch, conv_w, conv_b, conv_state, a_log, dt_bias, heads,
             groups, state, vdim):
    """proj [T, 2*heads*vdim + 2*groups*state + heads] =
    z | x | B | C | dt (the z columns are left for ``gate_group_norm``).
    conv_w [heads*vdim + 2*groups*state, taps], conv_b and conv_state
    [slots, taps-1, same] cover the x|B|C columns.
    Returns fp32 C [T, groups, state], B [T, groups, state],
    v = dt * x [T, heads, vdim], x [T, heads, vdim], decay [T, heads]."""
    T = proj.shape[0]
    inner, gn = heads * vdim, groups * state
    C = inner + 2 * gn
    assert proj.shape[1] == 2 * inner + 2 * gn + heads and conv_w.shape[0] == C
    if proj.is_cuda and _sk().enabled():
        return _sk().ssd_prep(proj, batch, conv_w, conv_b, conv_state, a_log,
                              dt_bias, heads, groups, state, vdim)
    y = conv_silu_ragged(proj[:, inner:inner + C], conv_w, conv_state, batch,
                         conv_b)
    x = y[:, :inner].reshape(T, heads, vdim)
    Bk = y[:, inner:inner + gn].reshape(T, groups, state)
    Cq = y[:, inner + gn:].reshape(T, groups, state)
    dt = F.softplus(proj[:, inner + C:].float() + dt_bias.float())
    decay = torch.exp(-torch.exp(a_log.float()) * dt)
    v = dt[:, :, None] * x
    return Cq.contiguous(), Bk.contiguous(), v, x.contiguous(), decay


def gate_group_norm(o, x, skip, gate, weight, parts, eps, out_dtype):
    """o, x [T, H, vdim] fp32; skip [H]; gate [T, H*vdim] pre-activation (may
    be a column slice); weight [H*vdim]. With ``y = (o + skip_h * x) *
    silu(gate)``, returns ``y / sqrt(mean_part(y^2) + eps) * weight`` where
    the mean runs over each of ``parts`` equal pieces of the row, as
    [T, H*vdim] ``out_dtype``."""
    T, H, vdim = o.shape
    n = H * vdim
    assert n % parts == 0 and weight.numel() == n
    if o.is_cuda and _sk().enabled():
        return _sk().gate_group_norm(o, x, skip, gate, weight, parts, eps,
                                     out_dtype)
    y = (o + skip.float()[None, :, None] * x).reshape(T, n) \
        * F.silu(gate.float())
    y = y.reshape(T, parts, n // parts)
    y = y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + eps)
    return (y.reshape(T, n) * weight.float()).to(out_dtype)


def retention_prep(proj, batch, heads, dim, rot_dims, cos, sin, k_scale,
                   layout="half"):
    """proj [T, 2*heads*dim] = q | k (may be a column slice). Rotates the first
    ``rot_dims`` coordinates of every head ("half" pairs i with
    i + rot_dims/2, "interleaved" 2i with 2i+1) and then multiplies the keys
    by ``k_scale``. Returns fp32 q, k [T, heads, dim]."""
    T, n = proj.shape[0], heads * dim
    assert proj.shape[1] == 2 * n and layout in ("half", "interleaved")
    if proj.is_cuda and _sk().enabled():
        return _sk().retention_prep(proj, batch, heads, dim, rot_dims, cos,
                                    sin, k_scale, layout)
    rotate = rope_interleaved_ if layout == "interleaved" else rope_half_
    q = proj[:, :n].float().reshape(T, heads, dim).clone()
    k = proj[:, n:].float().reshape(T, heads, dim).clone()
    if rot_dims:
        rotate(q, batch.tok_pos, cos, sin, rot_dims)
        rotate(k, batch.tok_pos, cos, sin, rot_dims)
    return q, k * k_scale


def retention_mix(qk, v, gate, decay, state, batch, heads, dim, vdim,
                  rot_dims, cos, sin, eps, out_scale=1.0, out=None):
    """qk [T, 2*heads*dim] = q | k, v and gate [T, heads*vdim] (column slices
    are fine); decay [heads] fp32; state [slots, heads, dim, vdim] fp32,
    advanced in place. Rotate-half positions on q and k, keys then times
    ``dim ** -0.5``; ``S <- decay S + k v^T``, ``o = S^T q``; every head's o
    divided by its root mean square, times ``silu(gate) * out_scale``.
    Returns [T, heads*vdim] in qk's dtype, written into ``out`` when given."""
    T = qk.shape[0]
    if out is None:
        out = torch.empty(T, heads * vdim, dtype=qk.dtype, device=qk.device)
    if qk.is_cuda and _sk().enabled() and \
            _sk().retention_step_ok(batch, dim, vdim):
        return _sk().retention_step(qk, v, gate, decay, state, batch, heads,
                                    dim, vdim, rot_dims, cos, sin,
                                    dim ** -0.5, eps, out_scale, out)
    q, k = retention_prep(qk, batch, heads, dim, rot_dims, cos, sin,
                          dim ** -0.5)
    o = linear_scan(q, k, v.view(T, heads, vdim), decay, None, state, batch)
    return head_norm_gate(o, None, gate, eps, qk.dtype, "silu", out_scale,
                          out)
