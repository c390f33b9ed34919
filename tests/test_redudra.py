"""Redudra through the serving path (registry -> ContinuousBatcher ->
PagedStateCache -> ops) against the plain oracle in redudra_oracle.py.

Every test makes its own small configuration and random tensors under the
checkpoint's names; the same tensors feed the oracle (float64) and
``load_named_tensors``. The device is the GPU when there is one (tests marked
``gpu`` then run the HIP kernels), the CPU otherwise.
"""

import json
import math
import os

import pytest
import torch

from tests import redudra_oracle as O
from deepspeed_amd.inference.ragged import ContinuousBatcher, Request
from deepspeed_amd.inference.state_cache import PagedStateCache
from deepspeed_amd.models import build_model, load_pretrained

DEV = "cuda" if torch.cuda.is_available() else "cpu"


# ------------------------------------------------------- configurations
def rg(width=12, blocks=3, conv=3):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks,
                                       "conv": conv}}


def par(heads=4, kv=2, dim=10, vdim=6, scale=0.4, size=9, keep=2, base=100.0,
        dims=8, factor=3.0, original=24, fast=4.0, slow=1.0, rheads=3, rdim=8,
        rvdim=5, rbase=50.0, rdims=6, decay=None, ls=0.8, rs=1.3):
    decay = decay or [1 - 0.5 ** (1 + 2 * i) for i in range(rheads)]
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                 "scale": scale, "mask": {"size": size, "keep_first": keep},
                 "rot": {"base": base, "dims": dims,
                         "scaling": {"factor": factor, "original": original,
                                     "fast": fast, "slow": slow}}},
        "right": {"heads": rheads, "dim": rdim, "vdim": rvdim,
                  "rot": {"base": rbase, "dims": rdims}, "decay": decay},
        "left_scale": ls, "right_scale": rs}}


def dense(ff=20):
    return {"kind": "dense", "ff": ff}


def config(layers, width=24, vocab=41, eps=1e-5, loop=None, mult=0.7,
           cap=6.0):
    """layers: (mixer entry, mlp or None) pairs."""
    cfg = {"architecture": "Redudra", "vocab": vocab, "width": width,
           "norm": {"eps": eps}, "residual_mult": mult, "logit_softcap": cap,
           "layers": [{**mix, "mlp": mlp} for mix, mlp in layers]}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def tensors(cfg, seed=0):
    """Random tensors of a useful scale under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rn(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(o, i, s=1.0):
        return rn(o, i, s=s * i ** -0.5)

    t = {"embed": rn(cfg["vocab"], W), "final.norm": 1 + rn(W, s=0.1),
         "final.norm.b": rn(W, s=0.2), "head": lin(cfg["vocab"], W, 2.0)}
    if cfg.get("loop"):
        t["loop.step"] = rn(cfg["loop"]["times"], W, s=0.7)
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        q = p + "mix."
        t[p + "norm1"], t[p + "norm1.b"] = 1 + rn(W, s=0.1), rn(W, s=0.2)
        t[p + "shift"] = 0.5 + rn(W, s=0.3)
        if spec["type"] == "rglru":
            C, nb = m["width"], m["blocks"]
            n = C // nb
            for name in ("y", "x"):
                t[q + name], t[q + name + ".b"] = lin(C, W), rn(C, s=0.3)
            t[q + "conv"], t[q + "conv.b"] = rn(C, m["conv"], s=0.6), \
                rn(C, s=0.3)
            for name in ("ra", "ri"):
                t[q + name] = rn(nb, n, n, s=2 * n ** -0.5)
                t[q + name + ".b"] = rn(nb, n, s=0.5)
            t[q + "lam"] = rn(C) - 2.0
            t[q + "o"] = lin(W, C)
        else:
            a, r = m["left"], m["right"]
            for name, rows in (("q", a["heads"] * a["dim"]),
                               ("k", a["kv_heads"] * a["dim"]),
                               ("v", a["kv_heads"] * a["vdim"])):
                t[q + "left." + name] = lin(rows, W)
            t[q + "left.o"] = lin(W, a["heads"] * a["vdim"])
            nq, nv = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            for name, rows in (("q", nq), ("k", nq), ("v", nv), ("g", nv)):
                t[q + "right." + name] = lin(rows, W)
            t[q + "right.o"] = lin(W, nv)
        if not spec["mlp"]:
            continue
        ff = spec["mlp"]["ff"]
        t[p + "norm2"], t[p + "norm2.b"] = 1 + rn(W, s=0.1), rn(W, s=0.2)
        f = p + "mlp."
        for name, o, i_ in (("gate", ff, W), ("up", ff, W), ("down", W, ff)):
            t[f + name], t[f + name + ".b"] = lin(o, i_), rn(o, s=0.3)
    return t


BASE = config([(rg(), dense(40)),
               (par(), dense(16)),
               (rg(width=10, blocks=2, conv=4), None),
               (par(heads=2, kv=1, dim=6, vdim=8, dims=6, rheads=2, rdim=4,
                    rvdim=7, rdims=4, size=5, keep=1), dense(9)),
               (rg(width=8, blocks=1, conv=2), dense(24))],
              loop=(1, 3, 2))


class Served:
    """A configuration loaded into the framework plus its oracle weights."""

    def __init__(self, cfg, seed=0, dtype=torch.float32, slots=4,
                 max_tokens=512, block=16, t=None):
        self.cfg = cfg
        self.t = t or tensors(cfg, seed)
        if dtype == torch.bfloat16:
            # the oracle gets the weights as 16-bit serving holds them
            self.t = {k: v.bfloat16().float() for k, v in self.t.items()}
        self.w64 = {k: v.double() for k, v in self.t.items()}
        self.model = build_model(self.cfg, dtype, self.t) \
            .load_named_tensors(self.t).to(DEV).eval()
        build = self.model.build_cache
        self.model.build_cache = \
            lambda *a, **k: build(*a, **{**k, "block_size": block})
        self.batcher = ContinuousBatcher(self.model, max_slots=slots,
                                         dtype=dtype, device=torch.device(DEV),
                                         max_tokens=max_tokens)
        self.n = 0

    def oracle(self, tokens, streams=None):
        return O.forward(list(tokens), self.w64, self.cfg, streams=streams)

    def run(self, tokens, cuts):
        """One request fed in portions ``cuts``; logits of every position."""
        self.n += 1
        req = self.batcher.open("q%d" % self.n)
        out, at = [], 0
        for c in cuts:
            out.append(self.batcher.feed([(req, tokens[at:at + c])]).double()
                       .cpu())
            at += c
        assert at == len(tokens)
        self.batcher.close(req)
        return torch.cat(out)


def toks(n, vocab=41, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def close(got, want, tol=2e-4):
    scale = want.std().item()
    err = (got - want).abs().max().item() / scale
    assert err < tol, "relative error %.3g" % err


def close_rms(got, want, tol):
    """16-bit runs: root-mean-square error per position, against the spread.
    A retention head of a few columns whose read-out nearly cancels is scaled
    up by its norm, rounding included, so single positions get more room."""
    err = ((got - want) ** 2).mean(-1).sqrt() / want.std().item()
    assert err.median().item() < tol, "median %.3g" % err.median().item()
    assert err.max().item() < 6 * tol, "worst %.3g" % err.max().item()


def begun(states, held, counts, row_dims=(), block=8, tokens=1 << 14,
          dtype=torch.float32):
    """A cache whose slots already hold ``held`` tokens, with a step of
    ``counts`` new ones begun."""
    cache = PagedStateCache(list(row_dims), states, len(held), tokens,
                            block_size=block, device=DEV, dtype=dtype)
    for slot, n in enumerate(held):
        cache.reset_slot(slot)
        cache.lens[slot] = n
    return cache, cache.begin_ragged(list(range(len(held))), counts)


# ------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("dims,base,factor,original,fast,slow", [
    (8, 100.0, 3.0, 24, 4.0, 1.0), (16, 10000.0, 4.0, 4096, 32.0, 1.0),
    (6, 50.0, 1.0, 64, 8.0, 2.0), (64, 500000.0, 8.0, 8192, 32.0, 1.0),
    (4, 10.0, 2.0, 7, 30.0, 20.0)])          # both ramp ends clamp
def test_yarn_tables(dims, base, factor, original, fast, slow):
    from deepspeed_amd.models.savovik import rot_tables
    rot = {"dims": dims, "base": base, "scaling": {
        "factor": factor, "original": original, "fast": fast, "slow": slow}}
    cos, sin = rot_tables(rot, 300, DEV)
    f, mag = O.frequencies(rot)
    ang = torch.arange(300).double()[:, None] * torch.tensor(f, dtype=torch.float64)[None]
    assert (cos.cpu() - mag * ang.cos()).abs().max() < 1e-6
    assert (sin.cpu() - mag * ang.sin()).abs().max() < 1e-6
    plain, _ = rot_tables({"dims": dims, "base": base}, 300, DEV)
    if factor != 1.0:       # something is really scaled
        assert (plain - cos).abs().max() > 0.05


def _shift_oracle(x, y, mult, extra, w, b, mu, eps):
    new = x.double() + (0 if y is None else mult * y.double()) \
        + (0 if extra is None else extra.double())
    h = O.layer_norm(new, w.double(), b.double(), eps)
    return new, (h if mu is None else O.token_shift(h, mu.double())), h


@pytest.mark.parametrize("C", [24, 13])
@pytest.mark.parametrize("with_y,with_extra", [(True, False), (True, True),
                                               (False, True), (False, False)])
def test_residual_norm_and_shift_over_portions(C, with_y, with_extra):
    """Two sequences cut differently; the row before a portion comes from the
    slot, the row before a sequence is zero, a reused slot starts anew."""
    from deepspeed_amd.ops.norms import residual_norm
    L = {0: 11, 2: 6}
    x = {s: rnd(n, C, seed=s) for s, n in L.items()}
    y = {s: rnd(n, C, seed=9 + s) for s, n in L.items()}
    w, b, mu, e = 1 + 0.1 * rnd(C, seed=3), rnd(C, seed=4), rnd(C, seed=5), \
        rnd(C, seed=6)
    cache = PagedStateCache([], {"h": ((C,), torch.float32)}, 3, 256,
                            block_size=8, device=DEV)
    for _ in range(2):                       # the second time in used slots
        for s in L:
            cache.reset_slot(s)
        at, news, outs = {0: 0, 2: 0}, {0: [], 2: []}, {0: [], 2: []}
        for step in [{0: 4, 2: 1}, {2: 2}, {0: 1, 2: 3}, {0: 6}]:
            bt = cache.begin_ragged(list(step), list(step.values()))

            def part(v):
                return torch.cat([v[s][at[s]:at[s] + n]
                                  for s, n in step.items()]).to(DEV)

            nx, h = residual_norm(
                part(x), part(y) if with_y else None, 0.3, w.to(DEV),
                b.to(DEV), 1e-4, None, e.to(DEV) if with_extra else None,
                mu.to(DEV), cache.states["h"], bt)
            cache.end_step()
            o = 0
            for s, n in step.items():
                news[s].append(nx[o:o + n].cpu())
                outs[s].append(h[o:o + n].cpu())
                o += n
                at[s] += n
        for s in L:
            new, want, plain = _shift_oracle(
                x[s], y[s] if with_y else None, 0.3, e if with_extra else None,
                w, b, mu, 1e-4)
            close(torch.cat(news[s]).double(), new, 1e-5)
            close(torch.cat(outs[s]).double(), want, 1e-4)
            close(cache.states["h"][s].cpu().double(), plain[-1], 1e-4)


def test_residual_norm_without_shift_and_of_chosen_rows():
    from deepspeed_amd.ops.norms import residual_norm
    x, y = rnd(9, 24), rnd(9, 24, seed=1)
    w, b = 1 + 0.1 * rnd(24, seed=2), rnd(24, seed=3)
    new, want, _ = _shift_oracle(x, y, -0.6, None, w, b, None, 1e-5)
    stream = x.to(DEV)
    rows = torch.tensor([7, 0, 7]).to(DEV)
    same, h = residual_norm(stream, y.to(DEV), -0.6, w.to(DEV), b.to(DEV),
                            1e-5, index=rows)
    close(h.cpu().double(), want[[7, 0, 7]], 1e-4)
    assert torch.equal(stream.cpu(), x)          # picked rows only read it
    got, h = residual_norm(stream, y.to(DEV), -0.6, w.to(DEV), b.to(DEV),
                           1e-5)
    close(h.cpu().double(), want, 1e-4)
    assert got.data_ptr() == stream.data_ptr()   # added in place
    close(stream.cpu().double(), new, 1e-5)


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_convolution_without_activation(taps):
    from deepspeed_amd.ops.causal_conv import conv_silu_ragged
    C, L = 16, 12
    x, w, b = rnd(L, C), rnd(C, taps, seed=1), rnd(C, seed=2)
    want = O.causal_conv(x.double(), w.double(), b.double())
    for cuts in ([12], [1] * 12, [2, 7, 1, 2]):
        cache, out, at = None, [], 0
        cache = PagedStateCache([], {"conv": (taps - 1, C)}, 1, 64,
                                block_size=8, device=DEV)
        for c in cuts:
            bt = cache.begin_ragged([0], [c])
            out.append(conv_silu_ragged(x[at:at + c].to(DEV), w.to(DEV),
                                        cache.states["conv"], bt, b.to(DEV),
                                        act=None))
            cache.end_step()
            at += c
        close(torch.cat(out).cpu().double(), want, 1e-5)


def test_gates_and_scan_of_the_diagonal_recurrence():
    from deepspeed_amd.ops.gated_recurrence import diagonal_scan, rglru_gates
    T, nb, n = 21, 3, 7
    W = nb * n
    u, z = rnd(T, W), rnd(T, W, seed=1)
    wr, wi = rnd(nb, n, n, seed=2), rnd(nb, n, n, seed=3)
    br, bi, lam = rnd(nb, n, seed=4), rnd(nb, n, seed=5), 3 * rnd(W, seed=6)
    d = lambda v: v.double()
    r = O.sigmoid(O.block_linear(d(wr), d(br), d(u)))
    i = O.sigmoid(O.block_linear(d(wi), d(bi), d(u)))
    want = O.rglru_scan(d(u), r, i, d(lam)) * O.gelu_tanh(d(z))
    g = lambda v: v.reshape(-1).to(DEV)
    a, b = rglru_gates(u.to(DEV), wr.to(DEV), g(br), wi.to(DEV), g(bi),
                       g(lam))
    for cuts in ([21], [1] * 21, [2, 10, 1, 8]):
        cache = PagedStateCache([], {"rec": ((W,), torch.float32)}, 1, 64,
                                block_size=8, device=DEV)
        out, at = [], 0
        for c in cuts:
            bt = cache.begin_ragged([0], [c])
            out.append(diagonal_scan(
                a[at:at + c].contiguous(), b[at:at + c].contiguous(),
                cache.states["rec"], bt, z[at:at + c].to(DEV)))
            cache.end_step()
            at += c
        close(torch.cat(out).cpu().double(), want, 1e-4)


def test_step_factor_keeps_its_digits_when_the_decay_is_near_one():
    """1 - a^2 from a rounded a would have no correct digit left here."""
    from deepspeed_amd.ops.gated_recurrence import rglru_gates
    W = 8
    lam = torch.full((W,), -14.0)
    u, w = rnd(3, W), torch.zeros(1, W, W)
    zero = torch.zeros(W)
    _, b = rglru_gates(u.to(DEV), w.to(DEV), zero.to(DEV), w.to(DEV),
                       zero.to(DEV), lam.to(DEV))
    la = -8 * 0.5 * math.log1p(math.exp(-14.0))
    want = math.sqrt(-math.expm1(2 * la)) * 0.5 * u.double()
    close(b.cpu().double(), want, 1e-5)


def test_diagonal_state_carries_a_far_token():
    """Decays next to one: after 400 tokens without input the first token's
    contribution is still what the recurrence says, prompts and decoding."""
    from deepspeed_amd.ops.gated_recurrence import diagonal_scan
    W, L = 24, 400
    a = torch.full((L, W), 0.9995)
    b = torch.zeros(L, W)
    b[0] = rnd(W) * 100
    want = b[0].double() * 0.9995 ** torch.arange(L).double()[:, None]
    for cuts in ([400], [130, 2, 268], [399, 1], [1] * 20 + [380]):
        cache = PagedStateCache([], {"rec": ((W,), torch.float32)}, 1, 512,
                                block_size=8, device=DEV)
        out, at = [], 0
        for c in cuts:
            bt = cache.begin_ragged([0], [c])
            out.append(diagonal_scan(a[at:at + c].to(DEV).contiguous(),
                                     b[at:at + c].to(DEV).contiguous(),
                                     cache.states["rec"], bt))
            cache.end_step()
            at += c
        close(torch.cat(out).cpu().double(), want, 1e-4)


@pytest.mark.parametrize("dims", [0, 4, 8])
def test_retention_prologue_rotates_then_scales_keys(dims):
    from deepspeed_amd.ops.linear_recurrence import retention_prep
    from deepspeed_amd.ops.rope import rope_tables
    H, d, start, T = 3, 8, 37, 6
    cache, bt = begun({}, [start], [T])
    cos, sin = rope_tables(dims, 64, 30.0, device=DEV) if dims \
        else (None, None)
    x = rnd(T, 2 * H * d)
    q, k = retention_prep(x.to(DEV), bt, H, d, dims, cos, sin, 0.25)
    full = torch.zeros(start + T, 2 * H, d, dtype=torch.float64)
    full[start:] = x.double().view(T, 2 * H, d)
    want = O.rotate(full, {"dims": dims, "base": 30.0})[start:] if dims \
        else full[start:]
    close(q.cpu().double(), want[:, :H], 1e-5)
    close(k.cpu().double(), want[:, H:] * 0.25, 1e-5)


def test_softcap_is_returned_in_32_bit():
    from deepspeed_amd.ops.activations import softcap_rows
    z = (rnd(5, 24) * 20).bfloat16()
    got = softcap_rows(z.to(DEV), 7.0)
    assert got.dtype == torch.float32
    close(got.cpu().double(), 7.0 * torch.tanh(z.double() / 7.0), 1e-5)


def test_head_norm_without_weight_scaled_into_a_wider_row():
    from deepspeed_amd.ops.linear_recurrence import head_norm_gate
    for vdim in (5, 16):
        o, g = rnd(4, 3, vdim), rnd(4, 3 * vdim, seed=1)
        wide = torch.full((4, 3 * vdim + 8), 9.0).to(DEV)
        head_norm_gate(o.to(DEV), None, g.to(DEV), 1e-3, torch.float32,
                       out_scale=0.4, out=wide[:, 8:])
        od = o.double()
        want = od / torch.sqrt((od * od).mean(-1, keepdim=True) + 1e-3)
        want = want.reshape(4, -1) * O.silu(g.double()) * 0.4
        close(wide[:, 8:].cpu().double(), want, 1e-5)
        assert (wide[:, :8] == 9.0).all()


# -------------------------------------------------------- mixers over cuts
def _run_mixer(cfg, t, h, cuts, block=8, dtype=torch.float32):
    """The mixer of a one-layer model over one sequence in portions."""
    model = build_model(cfg, dtype, t).load_named_tensors(t).to(DEV).eval()
    cache = model.build_cache(2, 1024, dtype=dtype, device=DEV,
                              block_size=block)
    cache.reset_slot(1)
    out, at = [], 0
    for c in cuts:
        cache.begin_ragged([1], [c])
        st = {k: cache.states[f"{k}0"] for k in ("conv", "rec")
              if f"{k}0" in cache.states}
        out.append(model.layers[0].mixer(h[at:at + c].to(DEV, dtype), cache,
                                         model.stream_of.get(0), st)
                   .double().cpu())
        cache.end_step()
        at += c
    assert at == h.shape[0]
    return torch.cat(out)


CUTS = [[19], [1] * 19, [2, 1, 9, 2, 5], [2] * 9 + [1]]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("width,blocks,conv", [(12, 3, 3), (10, 1, 1),
                                               (16, 16, 4), (24, 2, 7)])
def test_rglru_matches_oracle_over_cuts(cuts, width, blocks, conv):
    cfg = config([(rg(width, blocks, conv), None)])
    t = tensors(cfg, 5)
    w = {k: v.double() for k, v in t.items()}
    h = rnd(19, 24, seed=1)
    want = O.rglru(h.double(), w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)
    close(_run_mixer(cfg, t, h, cuts), want)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("kw", [
    dict(), dict(kv=4, keep=0, dims=10), dict(kv=1, size=1, keep=0, dims=2),
    dict(size=40, keep=5, rdims=8, rheads=1), dict(size=3, keep=19),
    dict(ls=0.0), dict(rs=0.0)])
def test_attention_beside_retention_matches_oracle_over_cuts(cuts, kw):
    cfg = config([(par(**kw), None)])
    t = tensors(cfg, 6)
    w = {k: v.double() for k, v in t.items()}
    h = rnd(19, 24, seed=2)
    want = O.parallel(h.double(), w, "l0.mix.", cfg["layers"][0]["mixer"],
                      1e-5)
    close(_run_mixer(cfg, t, h, cuts), want)


# ---- one key stands out: who sees it shows in the result
SIZE, KEEP = 91, 3


def _loud(target, L, seed=0):
    """A one-layer model and inputs in which token ``target``'s key is far
    above the others in an unrotated coordinate, for every query alike; its
    value is unlike the others'."""
    cfg = config([(par(size=SIZE, keep=KEEP, dims=8, dim=10, heads=2, kv=1,
                       rheads=1, rs=0.0, scale=0.5), None)])
    t = tensors(cfg, seed)
    h = rnd(L, 24, seed=seed + 1) * 0.5
    h[:, 0], h[:, 1] = 0.0, 1.0
    if 0 <= target < L:
        h[target, 0] = 1.0
    q, k = t["l0.mix.left.q"], t["l0.mix.left.k"]
    q[8], q[18], k[8] = 0.0, 0.0, 0.0    # coordinate 8 of both query heads
    q[8, 1] = q[18, 1] = 6.0
    k[8, 0] = 8.0
    t["l0.mix.left.v"][:, 0] = 5.0
    return cfg, t, h


@pytest.mark.parametrize("target", [0, KEEP - 1, KEEP, 63, 64, 100])
@pytest.mark.parametrize("cuts", ["prompt", "portions", "decode"])
def test_keys_just_inside_and_outside_window_and_kept_tokens(target, cuts):
    """The target passes out of the window within the run (unless kept): the
    positions on both sides of that edge are in the compared range, as one
    prompt, in portions cut around the edge, and decoded alone."""
    edge = target + SIZE                 # first position that does not see it
    L = edge + 6
    cfg, t, h = _loud(target, L)
    w = {k: v.double() for k, v in t.items()}
    m = cfg["layers"][0]["mixer"]
    want = O.parallel(h.double(), w, "l0.mix.", m, 1e-5)
    c = {"prompt": [L], "portions": [edge - 3, 2, 3, 4],
         "decode": [edge - 4] + [1] * 10}[cuts]
    got = _run_mixer(cfg, t, h, c, block=64)
    close(got, want, 5e-4)
    # the crafted key is what decides: losing it changes the row visibly
    step = (want[edge] - want[edge - 1]).norm() / want[edge - 1].norm()
    if target >= KEEP:
        assert step > 0.5
    else:
        quiet = O.parallel(_loud(-1, L)[2].double(), w, "l0.mix.", m, 1e-5)
        assert (want[edge + 5] - quiet[edge + 5]).norm() > \
            0.5 * want[edge + 5].norm()


def test_a_far_key_in_the_retention_state():
    """One loud key 300 tokens back under a decay near one, matched by every
    query: portions, decoding and the whole prompt agree with the oracle."""
    cfg = config([(par(rheads=2, rdim=6, rdims=4, decay=[0.999, 0.5], ls=0.0,
                       rs=1.0), None)])
    t = tensors(cfg, 3)
    L = 320
    h = rnd(L, 24, seed=4) * 0.5
    h[:, 0], h[:, 1] = 0.0, 1.0
    h[7, 0] = 1.0
    q, k = t["l0.mix.right.q"], t["l0.mix.right.k"]
    for r in (5, 11):                     # unrotated coordinate of each head
        q[r], k[r] = 0.0, 0.0
        q[r, 1], k[r, 0] = 5.0, 50.0
    w = {n: v.double() for n, v in t.items()}
    want = O.parallel(h.double(), w, "l0.mix.", cfg["layers"][0]["mixer"],
                      1e-5)
    for cuts in ([320], [63, 2, 200, 55], [312] + [1] * 8):
        close(_run_mixer(cfg, t, h, cuts, block=64), want, 1e-3)
    # the far key dominates what the slow head reads at the end
    h2 = h.clone()
    h2[7, 0] = 0.0
    other = O.parallel(h2.double(), w, "l0.mix.", cfg["layers"][0]["mixer"],
                       1e-5)
    assert (other[-1] - want[-1]).norm() > 0.3 * want[-1].norm()


# ----------------------------------------------- the model, step by step
@pytest.fixture(scope="module")
def base():
    return Served(BASE)


def test_first_tokens(base):
    for n in (1, 2, 3, 4):
        t = toks(n, seed=n)
        close(base.run(t, [n]), base.oracle(t))


def test_prefill_equals_token_by_token(base):
    t = toks(26, seed=2)
    want = base.oracle(t)
    close(base.run(t, [26]), want)
    close(base.run(t, [1] * 26), want)


@pytest.mark.parametrize("cuts", [[2] * 13, [15, 1, 1, 9], [3, 5, 2, 16],
                                  [16, 10], [7, 2, 2, 2, 13]])
def test_portions_cut_anywhere(base, cuts):
    t = toks(26, seed=3)
    close(base.run(t, cuts), base.oracle(t))


def test_layer_streams_match_oracle(base):
    t = toks(14, seed=4)
    want = []
    base.oracle(t, want)
    b = base.batcher
    r = b.open("streams")
    b.cache.begin_ragged([r.slot], [len(t)])
    taps = []
    base.model(torch.tensor(t, device=DEV), kv_cache=b.cache, taps=taps)
    b.cache.end_step()
    b.close(r)
    assert len(taps) == len(want) == 7          # layers 1 and 2 run twice
    for got, ref in zip(taps, want):
        close(got.cpu().double(), ref)


def test_every_pass_of_the_loop_has_its_own_cache_and_state(base):
    cache = base.batcher.cache
    # runs: 0 rg | 1 par, 2 rg | 3 par, 4 rg | 5 par, 6 rg
    assert len(cache.pools) == 3
    want = {f"shift{r}" for r in range(7)} | {f"rec{r}" for r in range(7)} \
        | {f"conv{r}" for r in (0, 2, 4, 6)}
    assert set(cache.states) == want
    assert len(base.model.layers) == 5          # weights are stored once
    assert [a for _, a in base.model.runs] == \
        [None, 0, None, 1, None, None, None]


def test_unequal_batch_equals_each_alone(base):
    seqs = [toks(n, seed=20 + n) for n in (1, 9, 17, 30)]
    b = base.batcher
    reqs = [b.open("u%d" % i) for i in range(4)]
    first = b.feed([(r, s[:max(1, len(s) // 2)]) for r, s in zip(reqs, seqs)]) \
        .double().cpu()
    rest = [(r, s[max(1, len(s) // 2):]) for r, s in zip(reqs, seqs)
            if len(s) > 1]
    second = b.feed(rest).double().cpu()
    for r in reqs:
        b.close(r)
    a1 = a2 = 0
    for s in seqs:
        n1 = max(1, len(s) // 2)
        got = first[a1:a1 + n1]
        a1 += n1
        if len(s) > 1:
            got = torch.cat([got, second[a2:a2 + len(s) - n1]])
            a2 += len(s) - n1
        close(got, base.oracle(s))


def test_a_request_left_out_of_steps_goes_on_later(base):
    a, c = toks(20, seed=31), toks(12, seed=32)
    b = base.batcher
    ra, rc = b.open("left"), b.open("busy")
    got = [b.feed([(ra, a[:6]), (rc, c[:3])]).cpu()[:6]]
    b.feed([(rc, c[3:8])])
    b.feed([(rc, c[8:])])
    got.append(b.feed([(ra, a[6:])]).cpu())
    b.close(ra)
    b.close(rc)
    close(torch.cat(got).double(), base.oracle(a))


def test_blocks_and_slots_are_used_again():
    """A pool of 4 blocks of 16 and 2 slots serves 6 requests in turn, each
    leaving rows, states, convolution tails and a last row behind."""
    s = Served(BASE, slots=2, max_tokens=64, block=16)
    for k in range(6):
        t = toks(20 + k, seed=40 + k)
        other = toks(9, seed=80 + k)
        b = s.batcher
        r1, r2 = b.open("a%d" % k), b.open("b%d" % k)
        got = b.feed([(r1, t[:11]), (r2, other)]).cpu()[:11]
        got = torch.cat([got, b.feed([(r1, t[11:])]).cpu()])
        b.close(r1)
        b.close(r2)
        close(got.double(), s.oracle(t))
    assert s.batcher.cache.blocks_free() == 4


def test_chosen_rows_are_the_rows_of_the_whole_step(base):
    t = toks(12, seed=33)
    b = base.batcher
    r = b.open("rows")
    got = b.feed([(r, t)], rows=[11, 0, 5]).cpu().double()
    b.close(r)
    assert got.shape[0] == 3
    close(got, base.oracle(t)[[11, 0, 5]])


def test_long_decode_past_windows_and_block_borders(base):
    t = toks(120, seed=9)
    close(base.run(t, [5] + [1] * 115), base.oracle(t), 5e-4)


VARIANTS = {
    # sizes that the base makes equal or 1 are unequal or larger here
    "no_loop_full_rotation": config(
        [(par(heads=3, kv=3, dim=4, vdim=7, dims=4, size=1, keep=0,
              factor=1.0, rheads=4, rdim=6, rvdim=9, rdims=2), dense(7)),
         (rg(width=15, blocks=5, conv=1), None)], width=16, mult=1.0,
        cap=1.5),
    "loop_over_the_last_layers_three_times": config(
        [(rg(width=20, blocks=4, conv=2), dense(33)),
         (par(heads=6, kv=2, dim=8, vdim=4, dims=6, size=300, keep=0,
              rheads=1, rdim=10, rvdim=2, rdims=10, decay=[0.95]),
          dense(11)),
         (rg(width=6, blocks=6, conv=6), dense(5))],
        width=20, vocab=29, loop=(1, 3, 3), eps=1e-3, mult=0.25),
    "whole_model_looped_once": config(
        [(par(size=4, keep=30), None), (par(ls=-0.5, rs=2.0), None)],
        width=12, vocab=53, loop=(0, 2, 1), cap=50.0),
    "layers_around_the_loop": config(
        [(par(rheads=2, decay=[1.0, 0.25]), dense(8)),
         (rg(width=32, blocks=2, conv=4), dense(8)),
         (rg(width=8, blocks=4, conv=3), None),
         (par(heads=8, kv=4, dim=2, vdim=2, dims=2), dense(64))],
        width=10, vocab=17, loop=(1, 2, 4), mult=1.5),
}


@pytest.mark.parametrize("name", sorted(VARIANTS))
def test_other_sizes_and_orders(name):
    cfg = VARIANTS[name]
    s = Served(cfg, seed=3)
    t = toks(23, vocab=cfg["vocab"], seed=4)
    want = s.oracle(t)
    close(s.run(t, [23]), want, 5e-4)
    close(s.run(t, [4, 1, 1, 11, 2, 4]), want, 5e-4)


def test_bfloat16_stays_near_the_oracle():
    s = Served(BASE, dtype=torch.bfloat16)
    t = toks(30, seed=6)
    want = s.oracle(t)
    close_rms(s.run(t, [30]), want, 0.025)
    close_rms(s.run(t, [7, 1, 20, 1, 1]), want, 0.025)


def test_states_stay_32_bit_in_16_bit_serving():
    s = Served(BASE, dtype=torch.bfloat16)
    st = s.batcher.cache.states
    assert {st[k].dtype for k in st if k[:3] in ("rec", "shi")} == \
        {torch.float32}
    assert st["conv0"].dtype == torch.bfloat16
    assert s.batcher.cache.pools[0].dtype == torch.bfloat16
    m = s.model.layers[0]
    assert {m.shift.dtype, m.norm1.weight.dtype, m.mixer.lam.dtype,
            m.mixer.b_r.dtype, s.model.loop_step.dtype} == {torch.float32}
    assert s.run(toks(3), [3]).shape == (3, 41)


# ------------------------------- mid size, default 64-token blocks
def _mid_config():
    return config(
        [(rg(width=96, blocks=3, conv=4), dense(150)),
         (par(heads=6, kv=2, dim=24, vdim=16, dims=16, size=48, keep=5,
              scale=0.2, base=3000.0, original=64, fast=8.0, rheads=3,
              rdim=32, rvdim=24, rdims=32, rbase=9000.0,
              decay=[0.9, 0.99, 0.999]), dense(80)),
         (par(heads=2, kv=1, dim=64, vdim=32, dims=64, size=70, keep=1,
              scale=0.12, base=500.0, original=32, rheads=2, rdim=16,
              rvdim=40, rdims=8), None),
         (rg(width=160, blocks=4, conv=3), dense(64))],
        width=96, vocab=131, eps=1e-6, loop=(0, 3, 2), mult=0.6, cap=10.0)


def _mixed_schedule(dtype):
    """Three requests of 150, 70 and 5 tokens share steps: portions that end
    inside, on and one past a block border beside single tokens; the short
    one ends early and its slot serves a fourth request."""
    s = Served(_mid_config(), seed=5, dtype=dtype, slots=3, max_tokens=64 * 6,
               block=64)
    seqs = {"a": toks(150, 131, 1), "b": toks(70, 131, 2),
            "c": toks(5, 131, 3), "d": toks(40, 131, 4)}
    plan = [{"a": 63, "b": 1, "c": 5}, {"a": 1, "b": 64, "d": 2},
            {"a": 1, "b": 1, "d": 30}, {"a": 64, "b": 1, "d": 1},
            {"a": 1, "b": 1, "d": 7}, {"a": 20, "b": 2}]
    b = s.batcher
    live, at, got = {}, {k: 0 for k in seqs}, {k: [] for k in seqs}
    for step in plan:
        entries = []
        for k, n in step.items():
            if k not in live:
                live[k] = b.open(k)
            entries.append((live[k], seqs[k][at[k]:at[k] + n]))
        out = b.feed(entries).double().cpu()
        o = 0
        for k, n in step.items():
            got[k].append(out[o:o + n])
            o += n
            at[k] += n
            if at[k] == len(seqs[k]):
                b.close(live.pop(k))
    assert at == {k: len(v) for k, v in seqs.items()}
    return s, seqs, got


def test_mid_size_mixed_schedule_over_block_borders():
    s, seqs, got = _mixed_schedule(torch.float32)
    for k, t in seqs.items():
        close(torch.cat(got[k]), s.oracle(t), 5e-4)


# -------------------------------------------- the framework's entry points
def test_greedy_generation_through_the_scheduler(base):
    prompts = [toks(n, seed=60 + n) for n in (3, 12, 18)]
    b = base.batcher
    b.token_budget, b.prefill_chunk = 16, 7      # prompts enter in portions
    for i, p in enumerate(prompts):
        b.put(Request(uid=100 + i, prompt=torch.tensor(p), max_new_tokens=6))
    done = {r.uid: r.generated for r in b.run_to_completion()}
    b.token_budget, b.prefill_chunk = 2048, 0
    for i, p in enumerate(prompts):
        seq = list(p)
        for _ in range(6):
            seq.append(int(base.oracle(seq)[-1].argmax()))
        assert done[100 + i] == seq[len(p):]


def _save(folder, cfg, t):
    from safetensors.torch import save_file
    folder.mkdir(exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16().contiguous() for k, v in t.items()},
              str(folder / "model.safetensors"))


def test_registry_loads_a_checkpoint_folder(tmp_path):
    cfg = VARIANTS["loop_over_the_last_layers_three_times"]
    t = {k: v.bfloat16().float() for k, v in tensors(cfg, seed=8).items()}
    _save(tmp_path, cfg, t)
    model = load_pretrained(str(tmp_path), dtype=torch.float32, device=DEV)
    assert model.architecture == "Redudra"
    assert model.cfg.to_dict() == cfg
    b = ContinuousBatcher(model, max_slots=1, dtype=torch.float32,
                          device=torch.device(DEV), max_tokens=64)
    r = b.open("x")
    seq = toks(10, vocab=cfg["vocab"])
    got = b.feed([(r, seq)], rows=[9]).cpu().double()
    want = O.forward(seq, {k: v.double() for k, v in t.items()}, cfg)
    close(got, want[9:])
    # the parameters go back out under the checkpoint's names
    back = model.named_tensors()
    assert set(back) == set(t)
    for k, v in t.items():
        assert torch.equal(back[k].float().cpu(), v), k


def test_config_rejects_what_the_design_does_not_have():
    for layers, loop in (
            ([({"type": "conv", "mixer": {}}, None)], None),
            ([(rg(), None)], (0, 2, 2)),                    # past the end
            ([(rg(width=10, blocks=3), None)], None),
            ([(par(dims=3), None)], None),                  # odd rotation
            ([(par(heads=3, kv=2), None)], None),
            ([(par(rheads=3, decay=[0.5, 0.6]), None)], None),
            ([(rg(), {"kind": "moe", "ff": 8})], None)):
        with pytest.raises(ValueError):
            build_model(config(layers, loop=loop))
    t = tensors(BASE)
    t["l0.shift"] = t["l0.shift"][:-1]
    with pytest.raises(ValueError):
        build_model(BASE, torch.float32, t).load_named_tensors(t)


def test_schedule_replay_runner(tmp_path):
    """bin/trace_run end to end: two requests, portions beside single tokens,
    a slot used again; logits files against the oracle."""
    import subprocess
    import sys
    import numpy as np
    cfg = BASE
    t = {k: v.bfloat16().float() for k, v in tensors(cfg, seed=11).items()}
    mdir, out = tmp_path / "m", tmp_path / "o"
    _save(mdir, cfg, t)
    a, b, c = toks(9, seed=1), toks(5, seed=2), toks(4, seed=3)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [0, 5]},
                                {"id": "b", "tokens": b[:2], "want": []}],
         "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [2]}],
         "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[6:7], "want": []}],
         "end": []},
        {"step": 3, "entries": [{"id": "a", "tokens": a[7:], "want": [0, 1]},
                                {"id": "c", "tokens": c, "want": [3]}],
         "end": ["a", "c"]},
    ]
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run(
        [sys.executable, os.path.join(repo, "bin", "trace_run"), "--model",
         str(mdir), "--dtype", "float32", "--out", str(out), "--max-tokens",
         "128", "--slots", "2"],
        input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
        capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l.startswith("done")] == \
        ["done %d" % i for i in range(4)]
    w = {k: v.double() for k, v in t.items()}
    la, lb, lc = (O.forward(s, w, cfg) for s in (a, b, c))
    want = {0: la[[0, 5]], 1: lb[[4]], 3: torch.cat([la[[7, 8]], lc[[3]]])}
    assert not (out / "2.f32").exists()
    for n, ref in want.items():
        got = np.fromfile(out / ("%d.f32" % n), dtype="<f4").reshape(
            ref.shape)
        close(torch.from_numpy(got).double(), ref)


def test_generate_command_line(tmp_path):
    """bin/ds_generate: registry -> init_inference -> generate, greedy."""
    import subprocess
    import sys
    cfg = VARIANTS["whole_model_looped_once"]
    t = {k: v.bfloat16().float() for k, v in tensors(cfg, seed=14).items()}
    _save(tmp_path, cfg, t)
    a, b = toks(6, 53, seed=70), toks(6, 53, seed=71)
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run(
        [sys.executable, os.path.join(repo, "bin", "ds_generate"),
         "--model-dir", str(tmp_path), "--dtype", "float32", "--max-new-tokens",
         "3", "--tokens", ",".join(map(str, a)), "--tokens",
         ",".join(map(str, b))], text=True, capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    lines = [json.loads(l) for l in p.stdout.split("\n")
             if l.startswith("{")]
    w = {k: v.double() for k, v in t.items()}
    for prompt, line in zip((a, b), lines):
        seq = list(prompt)
        for _ in range(3):
            seq.append(int(O.forward(seq, w, cfg)[-1].argmax()))
        assert line["generated"] == seq[len(prompt):]


def test_http_server_generates_the_oracles_tokens():
    """The FastAPI front end over the same scheduler: concurrent requests,
    greedy tokens as the oracle's."""
    from concurrent.futures import ThreadPoolExecutor
    from fastapi.testclient import TestClient
    from deepspeed_amd.inference.server import InferenceServer, build_app
    s = Served(BASE, seed=21)
    prompts = [toks(n, seed=90 + n) for n in (5, 9, 3)]
    server = InferenceServer(s.model, max_slots=2).start()
    try:
        client = TestClient(build_app(server))

        def call(p):
            r = client.post("/generate", json={"token_ids": p,
                                               "max_new_tokens": 4})
            assert r.status_code == 200
            return r.json()["generated"]

        with ThreadPoolExecutor(3) as ex:
            got = list(ex.map(call, prompts))
    finally:
        server.stop()
    for p, g in zip(prompts, got):
        seq = list(p)
        for _ in range(4):
            seq.append(int(s.oracle(seq)[-1].argmax()))
        assert g == seq[len(p):]


# ------------------------------------------- HIP kernels against eager ops
@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_kernels_match_eager_on_the_same_device(dtype, monkeypatch):
    from deepspeed_amd.ops import serving_kernels as sk
    t = toks(40, seed=12)
    s = Served(BASE, dtype=dtype)
    kern = s.run(t, [17, 1, 1, 21])
    monkeypatch.setenv("DS_AMD_SERVING_EAGER", "1")
    assert not sk.enabled()
    eager = s.run(t, [17, 1, 1, 21])
    if dtype == torch.float32:
        close(kern, eager, 1e-4)
    else:
        close_rms(kern, eager, 0.025)


@pytest.mark.gpu
def test_kernel_libraries_are_loaded():
    from deepspeed_amd.ops import serving_kernels as sk
    Served(BASE).run(toks(5), [5])
    assert {"seq", "rows", "recur"} <= set(sk._libs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mid_size_mixed_schedule_on_the_kernels(dtype):
    s, seqs, got = _mixed_schedule(dtype)
    for k, t in seqs.items():
        if dtype == torch.float32:
            close(torch.cat(got[k]), s.oracle(t), 5e-4)
        else:
            close_rms(torch.cat(got[k]), s.oracle(t), 0.025)


def _both(monkeypatch, fn):
    """fn() on the kernels, then on the eager formulations."""
    got = fn()
    monkeypatch.setenv("DS_AMD_SERVING_EAGER", "1")
    want = fn()
    monkeypatch.delenv("DS_AMD_SERVING_EAGER")
    return got, want


def near(got, want, dtype):
    got, want = got.double(), want.double()
    tol = 2e-5 if dtype == torch.float32 else 1.2e-2
    err = (got - want).abs().max() / want.abs().max()
    assert err < tol, "relative error %.3g" % err


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C", [24, 13, 512, 1000, 2056, 4096, 8192, 9000])
def test_residual_norm_kernel_against_eager(C, dtype, monkeypatch):
    from deepspeed_amd.ops.norms import residual_norm
    for held, counts in (([0], [1]), ([5, 0, 9, 0], [1, 7, 1, 3]),
                         ([0, 3, 1, 0, 2], [1, 1200, 2, 1021, 6])):
        if C > 4096 and sum(counts) > 2000:
            continue
        T = sum(counts)
        x0, y = rnd(T, C).to(DEV), rnd(T, C, seed=1).to(DEV, dtype)
        w, b, mu, e = (rnd(C, seed=k).to(DEV) for k in (2, 3, 4, 5))
        st0 = rnd(len(held), C, seed=6).to(DEV)

        def run(shift, extra, with_y=True):
            cache, bt = begun({}, held, counts)
            st, x = st0.clone(), x0.clone()
            nx, h = residual_norm(
                x, y if with_y else None, 0.4, w, b, 1e-5, dtype,
                e if extra else None, mu if shift else None,
                st if shift else None, bt if shift else None)
            return nx, h, st

        for args in ((True, False), (True, True), (False, False),
                     (True, True, False), (True, False, False)):
            got, want = _both(monkeypatch, lambda: run(*args))
            near(got[0], want[0], torch.float32)
            near(got[1], want[1], dtype)
            near(got[2], want[2], torch.float32)
        rows = torch.tensor([T - 1, 0]).to(DEV)
        got, want = _both(monkeypatch, lambda: residual_norm(
            x0, y, 0.4, w, b, 1e-5, dtype, index=rows)[1])
        near(got, want, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C,taps", [(24, 4), (24, 3), (16, 2), (13, 4),
                                    (520, 4), (40, 1), (40, 6)])
def test_convolution_kernel_without_activation(C, taps, dtype, monkeypatch):
    from deepspeed_amd.ops.causal_conv import conv_silu_ragged
    for held, counts in (([4, 0, 1], [1, 1, 1]), ([0, 6, 2], [9, 1, 30])):
        wide = rnd(sum(counts), C + 16).to(DEV, dtype)
        w, b = rnd(C, taps, seed=1).to(DEV, dtype), rnd(C, seed=2).to(DEV)
        st0 = rnd(len(held), taps - 1, C, seed=3).to(DEV, dtype)

        def run():
            _, bt = begun({}, held, counts)
            st = st0.clone()
            for i, n in enumerate(held):      # nothing before position 0
                st[i, :max(0, taps - 1 - n)] = 0
            return conv_silu_ragged(wide[:, 16:], w, st, bt, b, dtype,
                                    None), st

        got, want = _both(monkeypatch, run)
        near(got[0], want[0], dtype)
        if taps > 1:
            assert torch.equal(got[1], want[1])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("blocks,n", [(3, 5), (2, 72), (1, 20), (4, 64),
                                      (2, 256), (1, 200)])
def test_gate_kernels_against_eager(blocks, n, dtype, monkeypatch):
    from deepspeed_amd.ops import serving_kernels as sk
    from deepspeed_amd.ops.gated_recurrence import rglru_gates
    W = blocks * n
    wr, wi = ((rnd(blocks, n, n, seed=k) * n ** -0.5).to(DEV, dtype)
              for k in (1, 2))
    br, bi, lam = (rnd(W, seed=k).to(DEV) for k in (3, 4, 5))
    lam = lam * 4                       # decays from almost one to almost zero
    for T in (1, 3, 17, 70, 600):
        u = rnd(T, W, seed=T).to(DEV, dtype)
        got, want = _both(monkeypatch, lambda: rglru_gates(u, wr, br, wi, bi,
                                                           lam))
        # 16-bit operands: the products still accumulate and stay in 32 bit
        for g, e in zip(got, want):
            assert g.dtype == torch.float32
            near(g, e, torch.float32)
        if dtype == torch.bfloat16:
            for g, e in zip(sk.rglru_gates(u, wr, br, wi, bi, lam, 8.0,
                                           "split"), want):
                near(g, e, torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [12, 64, 100, 4096])
def test_diagonal_scan_kernels_against_eager(W, dtype, monkeypatch):
    from deepspeed_amd.ops.gated_recurrence import diagonal_scan
    for counts in ([1, 1, 1], [3, 8, 1], [40, 1, 9], [1, 300, 257, 2],
                   [128, 129, 127, 256]):
        if W > 1000 and max(counts) > 100:
            continue
        T, n = sum(counts), len(counts)
        a = torch.sigmoid(3 + 3 * rnd(T, W)).to(DEV)
        b = rnd(T, W, seed=1).to(DEV)
        z = rnd(T, W + 8, seed=2).to(DEV, dtype)[:, 8:]
        st0 = rnd(n, W, seed=3).to(DEV)
        for act, gate in (("gelu_tanh", z), ("silu", z), ("silu", None)):
            def run():
                _, bt = begun({}, [2] * n, counts)
                st = st0.clone()
                return diagonal_scan(a, b, st, bt, gate, act, dtype), st

            got, want = _both(monkeypatch, run)
            near(got[0], want[0], dtype)
            near(got[1], want[1], torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,dims", [(3, 8, 6), (2, 64, 64), (5, 32, 16),
                                      (2, 24, 8), (3, 5, 2), (1, 128, 0)])
def test_retention_prologue_kernel_against_eager(H, d, dims, dtype,
                                                 monkeypatch):
    from deepspeed_amd.ops.linear_recurrence import retention_prep
    from deepspeed_amd.ops.rope import rope_tables
    cos, sin = rope_tables(dims, 2048, 500.0, device=DEV) if dims \
        else (None, None)
    _, bt = begun({}, [0, 1100], [9, 4])
    x = rnd(13, 2 * H * d + 8).to(DEV, dtype)[:, 8:]
    for layout in ("half", "interleaved"):
        got, want = _both(monkeypatch, lambda: retention_prep(
            x, bt, H, d, dims, cos, sin, 0.3, layout))
        near(got[0], want[0], torch.float32)
        near(got[1], want[1], torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("vdt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,dv", [(3, 8, 5), (2, 64, 64), (2, 128, 48),
                                    (1, 200, 32)])
def test_scan_with_a_fixed_decay_against_eager(H, d, dv, vdt, monkeypatch):
    from deepspeed_amd.ops.linear_recurrence import linear_scan
    counts = [1, 70, 20]
    T = sum(counts)
    q, k = rnd(T, H, d).to(DEV), (rnd(T, H, d, seed=1) * d ** -0.5).to(DEV)
    v = rnd(T, H * dv + 8, seed=2).to(DEV, vdt)[:, :H * dv].view(T, H, dv)
    dec = (1 - 0.5 ** (1 + 2 * torch.arange(H).float())).to(DEV)
    st0 = rnd(3, H, d, dv, seed=3).to(DEV)

    def run():
        _, bt = begun({}, [2, 0, 5], counts)
        st = st0.clone()
        st[1] = 0
        return linear_scan(q, k, v, dec, None, st, bt), st

    got, want = _both(monkeypatch, run)
    near(got[0], want[0], torch.float32)
    near(got[1], want[1], torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("blocks,n,taps,N", [
    (3, 5, 4, 3), (2, 72, 3, 1), (1, 20, 1, 5), (4, 64, 2, 17), (2, 256, 4, 40),
    (1, 200, 7, 2), (1, 328, 4, 5)])
def test_single_token_recurrence_step_against_its_parts(blocks, n, taps, N,
                                                        monkeypatch):
    """One fused kernel against convolution, gates and scan one by one, over
    several steps, from the first token on; slots in no order."""
    from deepspeed_amd.ops import serving_kernels as sk
    from deepspeed_amd.ops.gated_recurrence import rglru_mix
    W, bf = blocks * n, torch.bfloat16
    wr, wi = ((rnd(blocks, n, n, seed=k) * n ** -0.5).to(DEV, bf)
              for k in (1, 2))
    br, bi, lam, cb = (rnd(W, seed=k).to(DEV) for k in (3, 4, 5, 6))
    cw = rnd(W, taps, seed=7).to(DEV, bf)
    slots = torch.randperm(N + 2, generator=torch.Generator()
                           .manual_seed(N)).tolist()[:N]

    def run(fused):
        cache = PagedStateCache([], {"conv": ((taps - 1, W), bf),
                                     "rec": ((W,), torch.float32)}, N + 2,
                                64 * N, block_size=8, device=DEV, dtype=bf)
        for s in slots[1::2]:            # half of them go on from somewhere
            cache.states["conv"][s] = rnd(taps - 1, W, seed=s).to(DEV, bf)
            cache.states["rec"][s] = rnd(W, seed=50 + s).to(DEV)
            cache.lens[s] = 9
        outs = []
        for k in range(taps + 2):
            bt = cache.begin_ragged(slots, [1] * N)
            proj = rnd(N, 2 * W + 8, seed=90 + k).to(DEV, bf)[:, 8:]
            args = (proj, cw, cb, cache.states["conv"], wr, br, wi, bi, lam,
                    cache.states["rec"], bt)
            if fused:
                assert sk.rglru_step_ok(proj, bt, n)
            outs.append(rglru_mix(*args))
            cache.end_step()
        return torch.stack(outs), cache.states["conv"], cache.states["rec"]

    got = run(True)
    monkeypatch.setattr(sk, "STEP_MAX", 0)
    want = run(False)
    monkeypatch.setenv("DS_AMD_SERVING_EAGER", "1")
    eager = run(False)
    for ref in (want, eager):
        near(got[0], ref[0], bf)
        assert torch.equal(got[1], ref[1])
        # a convolution's sum can round to the neighbouring 16-bit value
        near(got[2], ref[2], bf)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,dv,dims,N", [
    (3, 8, 5, 6, 2), (2, 64, 64, 64, 1), (2, 128, 256, 32, 9),
    (1, 36, 300, 0, 3), (4, 16, 128, 16, 33)])
def test_single_token_retention_step_against_its_parts(H, d, dv, dims, N,
                                                       dtype, monkeypatch):
    from deepspeed_amd.ops.linear_recurrence import retention_mix
    from deepspeed_amd.ops.rope import rope_tables
    cos, sin = rope_tables(dims, 2048, 500.0, device=DEV) if dims \
        else (None, None)
    dec = torch.tensor([0.99, 1.0, 0.0, 0.3][:H]).to(DEV)
    x = rnd(N, 8 + 2 * H * (d + dv)).to(DEV, dtype)
    st0 = rnd(N, H, d, dv, seed=3).to(DEV)
    nq, nv = 8 + 2 * H * d, H * dv

    def run():
        _, bt = begun({}, [7 * i for i in range(N)], [1] * N)
        st, wide = st0.clone(), torch.zeros(N, nv + 8, device=DEV,
                                            dtype=dtype)
        retention_mix(x[:, 8:nq], x[:, nq:nq + nv], x[:, nq + nv:], dec, st,
                      bt, H, d, dv, dims, cos, sin, 1e-5, 0.7, wide[:, 8:])
        return wide, st

    got, want = _both(monkeypatch, run)
    near(got[0], want[0], dtype)
    near(got[1], want[1], torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("counts", [[1, 70, 20], [64, 63, 65], [2, 200, 128],
                                    [16]])
@pytest.mark.parametrize("H,G,d,dv", [(3, 3, 8, 4), (2, 2, 64, 64),
                                      (4, 2, 128, 48), (1, 1, 100, 260),
                                      (2, 1, 36, 128)])
def test_chunked_scan_against_the_token_by_token_scan(H, G, d, dv, counts,
                                                      monkeypatch):
    """Portions at, around and far from a chunk's length, decays from one that
    forgets at once to one that never does, states that hold something."""
    from deepspeed_amd.ops import serving_kernels as sk
    from deepspeed_amd.ops.linear_recurrence import linear_scan
    T, n = sum(counts), len(counts)
    q, k = rnd(T, G, d).to(DEV), (rnd(T, G, d, seed=1) * d ** -0.5).to(DEV)
    v = rnd(T, H * dv + 8, seed=2).to(DEV, torch.bfloat16)[:, 4:4 + H * dv] \
        .view(T, H, dv)
    dec = torch.tensor([0.99, 1.0, 0.0, 0.3][:H]).to(DEV)
    st0 = rnd(n, H, d, dv, seed=3).to(DEV)

    def run(path):
        _, bt = begun({}, [3] * n, counts)
        st = st0.clone()
        return sk.linear_scan(q, k, v, dec, None, st, bt, 0.7, path), st

    got, want = run("chunk"), run("scan")
    for g, e in zip(got, want):
        err = (g - e).abs().max() / e.abs().max()
        assert err < 5e-5, "relative error %.3g" % err
    monkeypatch.setenv("DS_AMD_SERVING_EAGER", "1")
    _, bt = begun({}, [3] * n, counts)
    st = st0.clone()
    near(want[0], linear_scan(q, k, v, dec, None, st, bt, 0.7),
         torch.float32)
    near(want[1], st, torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,v,weight,act", [
    (3, 5, True, "silu"), (4, 64, False, "silu"), (3, 128, True, "sigmoid"),
    (2, 256, False, "sigmoid"), (1, 520, True, "silu"), (5, 24, False,
                                                         "silu")])
def test_head_norm_kernel_against_eager(H, v, weight, act, dtype,
                                        monkeypatch):
    from deepspeed_amd.ops.linear_recurrence import head_norm_gate
    o = rnd(37, H, v).to(DEV)
    g = rnd(37, H * v + 8, seed=1).to(DEV, dtype)[:, 8:]
    w = rnd(v, seed=2).to(DEV) if weight else None

    def run():
        wide = torch.zeros(37, H * v + 16, device=DEV, dtype=dtype)
        head_norm_gate(o, w, g, 1e-5, dtype, act, 0.7, wide[:, 16:])
        return wide

    got, want = _both(monkeypatch, run)
    near(got, want, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_softcap_kernel_against_eager(dtype, monkeypatch):
    from deepspeed_amd.ops.activations import softcap_rows
    for shape in ((3, 41), (5, 4096)):
        z = (rnd(*shape) * 40).to(DEV, dtype)
        got, want = _both(monkeypatch, lambda: softcap_rows(z, 30.0))
        near(got, want, torch.float32)
