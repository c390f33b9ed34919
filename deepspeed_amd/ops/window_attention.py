"""Multi-head attention over paged K/V rows with a sliding window that also
keeps a sequence's first tokens, for ragged batches.

Every token caches ONE row per stream: ``[k (G x dim) ; v (G x vdim)]`` for the
G key/value heads; query head h reads key/value head ``h // (H / G)``. Position
i of a sequence sees position j when ``j <= i`` and (``i - j < window`` or
``j < keep_first``); kept tokens stay where they are (their rows were rotated
at their true positions). ``window <= 0`` means no window (plain causal).
Scores, softmax and the weighted sum are fp32.

Two more masks and a score transform share the kernels: ``chunk > 0`` lets
position i see j only when ``i // chunk == j // chunk`` (chunks counted from a
sequence's position 0, wherever a prompt was cut); ``softcap > 0`` replaces a
scaled score s by ``softcap * tanh(s / softcap)`` before the softmax.

``sink`` (one fp32 score per query head) joins the softmax's denominator as
``exp(sink_h)``: it has no key and no value and is not scaled, so the weights of
a row sum to less than one. Zeros give the softmax with one added to its
denominator. ``gate`` ([T, heads] pre-activations) scales every head's result
by ``sigmoid(gate)``.

``attn_prep`` finishes a step's fused q|k|v projection: an RMS norm of queries
and keys (``norm="whole"``: over the WHOLE query projection, all heads at
once, one weight per coordinate, and over the whole key projection;
``norm="head"``: per head over ``dim`` with one weight of size ``dim`` shared
by the heads; ``norm="after"``: per head AFTER the rotation, without weight;
``None``: no norm), rotation of the first ``rot_dims``
coordinates of every head (``layout="interleaved"`` pairs 2i with 2i+1,
``"half"`` pairs i with i + rot_dims/2), optionally each value head divided by
its root mean square (``v_unit_eps``), and the write of the new rows into the
pool. A layer that borrows another layer's rows passes ``own_kv=False``: its
projection holds queries only and nothing is written.

Further steps of the same prologue: ``conv`` = (weights [C, taps], tails
[slots, taps-1, C]) first runs a short causal convolution over every projected
channel (ops/causal_conv.py); ``v_from_k`` takes the keys as projected (before
norm and rotation) as values, so the projection is q | k alone and vdim is dim;
``q_factor`` is a per-position table of factors on the finished queries
(``temperature_table``); ``side`` = (z, out, act) evaluates a plain activation
of another column slice of the same projection in the same launch.
"""

import torch

from .activations import act_rows
from .causal_conv import conv_silu_ragged
from .rope import rope_half_, rope_interleaved_


def _sk():
    from . import serving_kernels
    return serving_kernels


def _rms_all(x, w, eps):
    xf = x.float()
    return xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps) * w.float()


def _qk_norm(x, w, eps, norm, n_heads, dim):
    T = x.shape[0]
    if norm == "whole":
        return _rms_all(x, w, eps).reshape(T, n_heads, dim)
    xf = x.float().reshape(T, n_heads, dim)
    if norm == "head":
        return _rms_all(xf, w, eps)
    return xf.clone()           # rotated in place: never the caller's rows


def attn_prep(proj, batch, pool, q_norm_w, k_norm_w, eps, heads, kv_heads,
              dim, vdim, rot_dims, cos, sin, own_kv=True, norm="whole",
              layout="interleaved", v_unit_eps=None, conv=None,
              v_from_k=False, q_factor=None, side=None):
    """proj [T, heads*dim (+ kv_heads*dim + kv_heads*vdim)] = q | k | v (may
    be a column slice of a wider projection). Returns q [T, heads, dim] in
    proj's dtype; with ``own_kv`` the rows [k ; v] of this step's tokens are
    written into ``pool`` ([blocks, block_size, kv_heads*(dim+vdim)])."""
    T = proj.shape[0]
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    assert proj.shape[1] == nq + (nk + (0 if v_from_k else nv) if own_kv
                                  else 0)
    assert norm in ("whole", "head", "after", None)
    assert layout in ("interleaved", "half")
    assert not v_from_k or (own_kv and vdim == dim and conv is None)
    if proj.is_cuda and _sk().enabled():
        return _sk().attn_prep(proj, batch, pool, q_norm_w, k_norm_w, eps,
                               heads, kv_heads, dim, vdim, rot_dims, cos, sin,
                               own_kv, norm, layout, v_unit_eps, conv,
                               v_from_k, q_factor, side)
    if side is not None:
        act_rows(side[0], side[2], out=side[1])
    if conv is not None:
        proj = conv_silu_ragged(proj, conv[0], conv[1], batch, None,
                                proj.dtype, act=None)
    rotate = rope_interleaved_ if layout == "interleaved" else rope_half_

    def finish(x, w, n):
        x = _qk_norm(x, w, eps, None if norm == "after" else norm, n, dim)
        if rot_dims:
            rotate(x, batch.tok_pos, cos, sin, rot_dims)
        if norm == "after":
            x = x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)
        return x

    q = finish(proj[:, :nq], q_norm_w, heads)
    if q_factor is not None:
        q = q * q_factor[batch.tok_pos.long()].view(T, 1, 1)
    if own_kv:
        k = finish(proj[:, nq:nq + nk], k_norm_w, kv_heads)
        v = proj[:, nq:] if v_from_k else proj[:, nq + nk:]
        if v_unit_eps is not None:
            vf = v.float().reshape(T, kv_heads, vdim)
            v = (vf * torch.rsqrt(vf.pow(2).mean(-1, keepdim=True)
                                  + v_unit_eps)).reshape(T, nv)
        rows = torch.cat([k.reshape(T, nk).to(pool.dtype),
                          v.to(pool.dtype)], -1)
        pool.view(-1, nk + nv)[batch.tok_row.long()] = rows
    return q.to(proj.dtype)


def window_mask(qpos, kpos, window, keep_first, chunk=0):
    """[len(qpos), len(kpos)] bool: which keys each query sees."""
    d = qpos[:, None] - kpos[None, :]
    near = d >= 0
    if window > 0:
        near = near & ((d < window) | (kpos[None, :] < keep_first))
    if chunk > 0:
        near = near & ((qpos[:, None] // chunk == kpos[None, :] // chunk)
                       | (kpos[None, :] < keep_first))
    return near


def window_attention(q, pool, batch, kv_heads, dim, vdim, scale, window=0,
                     keep_first=0, path=None, chunk=0, softcap=0.0,
                     out_scale=1.0, out=None, sink=None, gate=None):
    """q [T, heads, dim]; pool holds every sequence's rows INCLUDING this
    step's. Returns [T, heads*vdim] in q's dtype, times ``out_scale``;
    ``out`` (a [T, heads*vdim] view whose rows are contiguous, e.g. a column
    slice of a wider buffer) receives the result when given. ``sink`` [heads]
    fp32 or None, ``gate`` [T, heads] in q's dtype (a column slice is fine) or
    None."""
    T, H, _ = q.shape
    assert H % kv_heads == 0 and pool.shape[-1] == kv_heads * (dim + vdim)
    assert not (window > 0 and chunk > 0), "one mask per layer"
    if out is None:
        out = torch.empty(T, H * vdim, dtype=q.dtype, device=q.device)
    assert out.shape == (T, H * vdim) and out.stride(1) == 1
    if q.is_cuda and _sk().enabled():
        return _sk().window_attention(q, pool, batch, kv_heads, dim, vdim,
                                      scale, window, keep_first, path, chunk,
                                      softcap, out_scale, out, sink, gate)
    bs = batch.block_size
    rows = pool.view(-1, pool.shape[-1])
    rep = H // kv_heads
    at = 0
    for i, (st, cnt) in enumerate(zip(batch.starts, batch.counts)):
        L = st + cnt
        pos = torch.arange(L, device=q.device)
        ctx = rows[batch.block_table[i].long()[pos // bs] * bs + pos % bs]
        ctx = ctx.float()
        k = ctx[:, :kv_heads * dim].reshape(L, kv_heads, dim) \
            .repeat_interleave(rep, 1)
        v = ctx[:, kv_heads * dim:].reshape(L, kv_heads, vdim) \
            .repeat_interleave(rep, 1)
        s = torch.einsum("thd,lhd->htl", q[at:at + cnt].float(), k) * scale
        if softcap > 0:
            s = softcap * torch.tanh(s / softcap)
        see = window_mask(st + torch.arange(cnt, device=q.device), pos,
                          window, keep_first, chunk)
        s = s.masked_fill(~see[None], float("-inf"))
        if sink is not None:
            rest = sink.float().view(-1, 1, 1).expand(-1, cnt, 1)
            p = torch.softmax(torch.cat([s, rest], -1), -1)[..., :-1]
        else:
            p = torch.softmax(s, -1)
        o = torch.einsum("htl,lhv->thv", p, v) * out_scale
        if gate is not None:
            o = o * torch.sigmoid(gate[at:at + cnt].float())[:, :, None]
        out[at:at + cnt] = o.reshape(cnt, H * vdim).to(q.dtype)
        at += cnt
    return out
