"""Fubolix through the serving path (registry -> ContinuousBatcher ->
PagedStateCache -> ops) against the plain oracle in fubolix_oracle.py.

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

from tests import fubolix_oracle as O
from deepspeed_amd.inference.ragged import ContinuousBatcher, Request
from deepspeed_amd.inference.state_cache import PagedStateCache
from deepspeed_amd.models import build_model, load_pretrained

DEV = "cuda" if torch.cuda.is_available() else "cpu"


# ------------------------------------------------------- configurations
def _rot(base, dims, factor=3.0, original=24, fast=4.0, slow=1.0):
    return {"base": base, "dims": dims,
            "scaling": {"factor": factor, "original": original, "fast": fast,
                        "slow": slow}}


def win(heads=4, kv=2, dim=10, scale=0.4, size=9, keep=2, base=100.0, dims=8,
        **yarn):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim,
        "scale": scale, "mask": {"size": size, "keep_first": keep},
        "rot": _rot(base, dims, **yarn)}}


def temp(heads=3, kv=1, dim=8, vdim=6, scale=0.5, coef=0.7, every=5):
    return {"type": "attention_2", "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
        "scale": scale, "q_temp": {"coef": coef, "every": every}}}


def conv(heads=2, kv=2, dim=12, vdim=6, scale=0.3, taps=3, base=50.0, dims=6,
         **yarn):
    return {"type": "attention_3", "mixer": {
        "heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
        "scale": scale, "conv": taps, "rot": _rot(base, dims, **yarn)}}


def dense(ff=20):
    return {"kind": "dense", "ff": ff}


def config(layers, width=24, vocab=41, eps=1e-5, scale=1.7):
    """layers: (mixer entry, mlp or None) pairs."""
    return {"architecture": "Fubolix", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": [{**mix, "mlp": mlp} for mix, mlp in layers]}


def tensors(cfg, seed=0):
    """Random tensors of a useful scale under the checkpoint's names."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rn(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(o, i, s=1.0):
        return rn(o, i, s=s * i ** -0.5)

    t = {"embed": rn(cfg["vocab"], W), "head": lin(cfg["vocab"], W, 2.0)}

    def norm(name):
        t[name], t[name + ".b"] = 1 + rn(W, s=0.2), rn(W, s=0.3)
        t[name + ".alpha"] = 0.6 + rn(1, s=0.1).reshape(())

    norm("final.norm")
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        q = p + "mix."
        norm(p + "norm1")
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        parts = [("q", H * d), ("k", G * d)]
        if spec["type"] != "attention":
            parts.append(("v", G * dv))
        for name, rows in parts:
            t[q + name] = lin(rows, W, 1.5)
            if spec["type"] == "attention_3":
                t[q + name + ".conv"] = rn(rows, m["conv"], s=0.7)
        if spec["type"] == "attention":
            t[q + "g"] = lin(H, W, 1.5)
        elif spec["type"] == "attention_2":
            t[q + "q.norm"], t[q + "k.norm"] = 1 + rn(d, s=0.3), \
                1 + rn(d, s=0.3)
        else:
            t[q + "sink"] = rn(H)
        t[q + "o"] = lin(W, H * dv)
        if spec["mlp"]:
            ff = spec["mlp"]["ff"]
            t[p + "mlp.up"], t[p + "mlp.down"] = lin(ff, W), lin(W, ff)
    return t


BASE = config([(win(), dense(40)), (conv(), dense(16)), (temp(), None),
               (win(heads=3, kv=3, dim=6, dims=6, size=5, keep=1), dense(9)),
               (conv(heads=4, kv=1, dim=6, vdim=8, taps=2, dims=4),
                dense(24))])


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
        return O.forward(self.cfg, self.w64, list(tokens), streams)

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


def differs(got, want, by):
    """The two are visibly apart (what a planted mistake must achieve)."""
    assert (got - want).abs().max().item() / want.std().item() > by


def close_rms(got, want, tol):
    """16-bit runs: root-mean-square error per position, against the spread."""
    err = ((got - want) ** 2).mean(-1).sqrt() / want.std().item()
    assert err.median().item() < tol, "median %.3g" % err.median().item()
    assert err.max().item() < 4 * tol, "worst %.3g" % err.max().item()


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
@pytest.mark.parametrize("C", [24, 13])
def test_dynamic_tanh_with_residual(C):
    from deepspeed_amd.ops.norms import residual_tanh
    x, y = 3 * rnd(7, C), rnd(7, C, seed=1)
    w, b = 1 + 0.3 * rnd(C, seed=2), rnd(C, seed=3)
    al = torch.tensor([0.45])
    args = (al.to(DEV), w.to(DEV), b.to(DEV))

    def want(v):
        return O.dynamic_tanh(v.double(), al, w, b)

    stream = x.clone().to(DEV)
    close(residual_tanh(stream, None, *args).cpu().double(), want(x), 1e-5)
    assert torch.equal(stream.cpu(), x)
    rows = torch.tensor([6, 0, 6]).to(DEV)
    h = residual_tanh(stream, y.to(DEV), *args, index=rows)
    close(h.cpu().double(), want(x + y)[[6, 0, 6]], 1e-5)
    assert torch.equal(stream.cpu(), x)          # picked rows only read it
    h = residual_tanh(stream, y.to(DEV), *args)
    close(h.cpu().double(), want(x + y), 1e-5)
    close(stream.cpu().double(), (x + y).double(), 1e-5)
    differs(h.cpu().double(), want(x), 0.3)


@pytest.mark.parametrize("coef,every", [(0.5, 4), (0.1, 1), (1.3, 7),
                                        (0.7, 300)])
def test_temperature_table(coef, every):
    from deepspeed_amd.ops.rope import temperature_table
    got = temperature_table(700, coef, every, DEV).cpu()
    for p in range(700):
        assert abs(got[p].item() - O.query_temperature(p, coef, every)) < 1e-5
    # the step falls between positions every - 2 and every - 1
    if every > 1:
        assert got[every - 2] == 1.0 and got[every - 1] > 1.0


def test_relu_squared_into_a_column_slice():
    from deepspeed_amd.ops.activations import act_rows
    z = rnd(5, 40)
    wide = torch.full((5, 32), 7.0).to(DEV)
    got = act_rows(z.to(DEV)[:, 8:32], "relu2", out=wide[:, 4:28])
    want = torch.where(z > 0, z * z, 0 * z)[:, 8:32]
    close(got.cpu(), want, 1e-6)
    assert torch.equal(wide[:, 4:28].cpu(), got.cpu())
    assert (wide[:, :4] == 7).all() and (wide[:, 28:] == 7).all()


@pytest.mark.parametrize("layout,pairing", [("interleaved", "neighbours"),
                                            ("half", "halves")])
@pytest.mark.parametrize("dims", [2, 8, 10])
def test_prologue_rotation_then_unit_rms_keys_as_values(layout, pairing,
                                                        dims):
    from deepspeed_amd.models.savovik import rot_tables
    from deepspeed_amd.ops.window_attention import attn_prep
    H, G, d, L = 3, 2, 10, 30
    rot = _rot(100.0, dims)
    cos, sin = rot_tables(rot, 512, DEV)
    proj = rnd(L, (H + G) * d)
    cache, bt = begun({}, [0], [L], row_dims=[2 * G * d])
    q = attn_prep(proj.to(DEV), bt, cache.pools[0], None, None, 0.05, H, G, d,
                  d, dims, cos, sin, norm="after", layout=layout,
                  v_from_k=True)
    pd = proj.double()
    want = O.unit_rms(O.rotate(pd[:, :H * d].view(L, H, d), rot, pairing),
                      0.05)
    close(q.cpu().double(), want, 1e-5)
    rows = cache.pools[0].view(-1, 2 * G * d)[bt.tok_row.long()].cpu().double()
    k = pd[:, H * d:].view(L, G, d)
    close(rows[:, :G * d].view(L, G, d),
          O.unit_rms(O.rotate(k, rot, pairing), 0.05), 1e-5)
    assert torch.equal(rows[:, G * d:].float(), proj[:, H * d:])
    # the norm does not commute with the rotation's factor on some coordinates
    early = O.rotate(O.unit_rms(pd[:, :H * d].view(L, H, d), 0.05), rot,
                     pairing)
    differs(q.cpu().double(), early, 0.05)


def test_prologue_head_norms_and_temperature_at_scattered_positions():
    from deepspeed_amd.ops.rope import temperature_table
    from deepspeed_amd.ops.window_attention import attn_prep
    H, G, d, dv = 4, 2, 6, 5
    held, counts = [0, 13, 300], [3, 2, 1]
    cache, bt = begun({}, held, counts, row_dims=[G * (d + dv)])
    proj = rnd(6, H * d + G * (d + dv))
    wq, wk = 1 + 0.3 * rnd(d, seed=1), 1 + 0.3 * rnd(d, seed=2)
    tab = temperature_table(cache.max_seq, 0.9, 7, DEV)
    q = attn_prep(proj.to(DEV), bt, cache.pools[0], wq.to(DEV), wk.to(DEV),
                  1e-3, H, G, d, dv, 0, None, None, norm="head",
                  q_factor=tab)
    pos = [0, 1, 2, 13, 14, 300]
    want = O.unit_rms(proj[:, :H * d].double().view(6, H, d), 1e-3) * wq
    fac = torch.tensor([O.query_temperature(p, 0.9, 7) for p in pos])
    close(q.cpu().double(), want * fac[:, None, None], 1e-5)
    rows = cache.pools[0].view(-1, G * (d + dv))[bt.tok_row.long()].cpu()
    k = O.unit_rms(proj[:, H * d:(H + G) * d].double().view(6, G, d), 1e-3)
    close(rows[:, :G * d].double().view(6, G, d), k * wk, 1e-5)


@pytest.mark.parametrize("taps", [1, 2, 3, 5])
def test_prologue_convolution_over_portions_and_reused_slots(taps):
    from deepspeed_amd.models.savovik import rot_tables
    from deepspeed_amd.ops.window_attention import attn_prep
    H, G, d, dv, L = 2, 1, 8, 16, 23
    C = H * d + G * (d + dv)
    rot = _rot(50.0, 4)
    cos, sin = rot_tables(rot, 512, DEV)
    w = rnd(C, taps, seed=9)
    cache = PagedStateCache([G * (d + dv)], {"conv": (taps - 1, C)}, 2, 128,
                            block_size=8, device=DEV)
    for n, cuts in enumerate(([23], [1] * 23, [2, 3, 1, 1, 2, 14],
                              [9, 1, 2, 11])):
        x = rnd(L, C, seed=n)
        cache.reset_slot(1)
        out, rows, at = [], [], 0
        for c in cuts:
            bt = cache.begin_ragged([1], [c])
            out.append(attn_prep(
                x[at:at + c].to(DEV), bt, cache.pools[0], None, None, 1e-5, H,
                G, d, dv, 4, cos, sin, norm=None, layout="half",
                conv=(w.to(DEV), cache.states["conv"])).cpu())
            rows.append(cache.pools[0].view(-1, G * (d + dv))
                        [bt.tok_row.long()].cpu())
            cache.end_step()
            at += c
        y = O.short_conv(x.double(), w.double())
        close(torch.cat(out).double(),
              O.rotate(y[:, :H * d].view(L, H, d), rot, "halves"), 1e-5)
        rows = torch.cat(rows).double()
        close(rows[:, :G * d].view(L, G, d), O.rotate(
            y[:, H * d:(H + G) * d].view(L, G, d), rot, "halves"), 1e-5)
        close(rows[:, G * d:], y[:, (H + G) * d:], 1e-5)
        if taps > 1:
            close(cache.states["conv"][1].cpu(), x[-(taps - 1):], 1e-6)


@pytest.mark.parametrize("sink", [None, 0.0, 2.5, -60.0, 200.0])
@pytest.mark.parametrize("gated", [False, True])
def test_attention_sink_and_gate(sink, gated):
    from deepspeed_amd.ops.window_attention import window_attention
    H, G, d, dv, L = 4, 2, 6, 5, 21
    q, k, v = rnd(L, H, d), rnd(L, G, d, seed=1), rnd(L, G, dv, seed=2)
    gate = rnd(L, H + 3, seed=3)
    rest = None if sink is None else torch.full((H,), sink) \
        + 0.3 * (sink != 0) * torch.arange(H)
    cache, bt = begun({}, [0], [L], row_dims=[G * (d + dv)])
    cache.pools[0].view(-1, G * (d + dv))[bt.tok_row.long()] = torch.cat(
        [k.reshape(L, -1), v.reshape(L, -1)], 1).to(DEV)
    wide = torch.zeros(L, H * dv + 4).to(DEV)
    for mask, kw in ((None, {}), ({"size": 6, "keep_first": 2},
                                  {"window": 6, "keep_first": 2})):
        got = window_attention(
            q.to(DEV), cache.pools[0], bt, G, d, dv, 0.8, out=wide[:, 4:],
            sink=None if rest is None else rest.to(DEV),
            gate=gate.to(DEV)[:, 3:] if gated else None, **kw)
        o = O.attend(q.double(), k.double(), v.double(), 0.8, mask,
                     torch.full((H,), -1e4) if rest is None else rest)
        if gated:
            o = o * torch.sigmoid(gate[:, 3:].double())[:, :, None]
        if sink == 200.0:               # nothing is left beside it
            assert got.abs().max() < 1e-30 and o.abs().max() < 1e-30
        else:
            close(got.cpu().double(), o.reshape(L, -1), 1e-4)
        assert (wide[:, :4] == 0).all()


def test_one_in_the_denominator_is_a_share_of_the_first_token():
    """A sequence's first token sees itself alone: its weight is e^s / (1 +
    e^s), not one."""
    from deepspeed_amd.ops.window_attention import window_attention
    q, v = torch.tensor([[[2.0]]]), torch.tensor([[3.0]])
    cache, bt = begun({}, [0], [1], row_dims=[2])
    cache.pools[0].view(-1, 2)[bt.tok_row.long()] = \
        torch.tensor([[0.25, 3.0]]).to(DEV)
    got = window_attention(q.to(DEV), cache.pools[0], bt, 1, 1, 1, 1.0,
                           sink=torch.zeros(1).to(DEV))
    e = math.exp(0.5)
    assert abs(got.item() - 3.0 * e / (1 + e)) < 1e-6


# --------------------------------------------------- one mixer at a time
def _run_mixer(cfg, t, h, cuts, block=8, dtype=torch.float32):
    """The only layer's mixer on rows ``h`` in portions ``cuts``."""
    model = build_model(cfg, dtype, t).load_named_tensors(t).to(DEV)
    cache = model.build_cache(1, h.shape[0] + block, dtype=dtype, device=DEV,
                              block_size=block)
    cache.reset_slot(0)
    out, at = [], 0
    for c in cuts:
        cache.begin_ragged([0], [c])
        out.append(model.layers[0](h[at:at + c].to(DEV, dtype), cache, 0,
                                   {"conv": cache.states.get("conv0")}))
        cache.end_step()
        at += c
    assert at == h.shape[0]
    return torch.cat(out).cpu().double()


def _mixer_oracle(cfg, t, h):
    spec = cfg["layers"][0]
    return O.MIXERS[spec["type"]](h.double(),
                                  {k: v.double() for k, v in t.items()},
                                  "l0.mix.", spec["mixer"],
                                  cfg["norm"]["eps"])


@pytest.mark.parametrize("mix", [
    win(), win(heads=2, kv=2, dim=4, dims=4, size=1, keep=0),
    win(heads=6, kv=2, dim=16, dims=2, size=4, keep=7, factor=1.0),
    win(heads=1, kv=1, dim=8, dims=8, size=100, keep=3, original=5),
    temp(), temp(heads=2, kv=2, dim=5, vdim=9, coef=2.0, every=1),
    temp(heads=4, kv=1, dim=8, vdim=8, every=200),
    conv(), conv(heads=3, kv=1, dim=8, vdim=8, taps=1, dims=8),
    conv(heads=4, kv=2, dim=6, vdim=5, taps=5, dims=2, factor=1.0),
    conv(heads=2, kv=1, dim=16, vdim=24, taps=4, dims=16)])
def test_each_mixer_alone(mix):
    cfg = config([(mix, None)])
    t = tensors(cfg, 1)
    h = rnd(26, 24, seed=2)
    want = _mixer_oracle(cfg, t, h)
    for cuts in ([26], [1] * 26, [7, 2, 2, 15], [17, 9]):
        close(_run_mixer(cfg, t, h, cuts), want)


# ------------------------- crafted keys: borders, windows, far away, sinks
SIZE, KEEP = 70, 3


def _loud(target, L, mix):
    """Layer input whose column 0 is raised at ``target`` only and column 1
    everywhere: every query asks along the last coordinate of each head (never
    rotated) and only the target's key answers."""
    cfg = config([(mix, None)])
    t = tensors(cfg, 3)
    h = rnd(L, 24, seed=4) * 0.5
    h[:, 0], h[:, 1] = 0.0, 1.0
    if target >= 0:
        h[target, 0] = 1.0
    q, k = t["l0.mix.q"], t["l0.mix.k"]
    d = mix["mixer"]["dim"]
    for r in range(d - 1, q.shape[0], d):
        q[r], q[r, 1] = 0.0, 12.0
    for r in range(d - 1, k.shape[0], d):
        k[r], k[r, 0] = 0.0, 12.0
    for name in "qk":                     # the current token alone
        if "l0.mix." + name + ".conv" in t:
            c = t["l0.mix." + name + ".conv"]
            c[d - 1::d], c[d - 1::d, -1] = 0.0, 1.0
    return cfg, t, h


@pytest.mark.parametrize("target", [0, KEEP - 1, KEEP, 63, 64, 100])
@pytest.mark.parametrize("cuts", ["prompt", "portions", "decode"])
def test_keys_just_inside_and_outside_window_and_kept_tokens(target, cuts):
    """The target passes out of the window within the run (unless kept): the
    positions on both sides of that edge are in the compared range, as one
    prompt, in portions cut around the edge, and decoded alone."""
    edge = target + SIZE                 # first position that does not see it
    L = edge + 6
    cfg, t, h = _loud(target, L, win(size=SIZE, keep=KEEP, scale=2.0))
    want = _mixer_oracle(cfg, t, h)
    c = {"prompt": [L], "portions": [edge - 3, 2, 3, 4],
         "decode": [edge - 4] + [1] * 10}[cuts]
    close(_run_mixer(cfg, t, h, c, block=64), want, 5e-4)
    # the crafted key is what decides: losing it changes the row visibly
    step = (want[edge] - want[edge - 1]).norm() / want[edge - 1].norm()
    if target >= KEEP:
        assert step > 0.5
    else:
        quiet = _mixer_oracle(cfg, t, _loud(-1, L, win())[2])
        assert (want[edge + 5] - quiet[edge + 5]).norm() > \
            0.5 * want[edge + 5].norm()


@pytest.mark.parametrize("mix", [temp(scale=1.0, every=40),
                                 conv(scale=0.1, dims=6, taps=3)],
                         ids=["temperature", "convolution"])
@pytest.mark.parametrize("target", [0, 1, 63, 64, 127, 128])
def test_a_far_key_among_hundreds(mix, target):
    L = 260
    cfg, t, h = _loud(target, L, mix)
    want = _mixer_oracle(cfg, t, h)
    for cuts in ([260], [64, 64, 2, 130], [250] + [1] * 10):
        close(_run_mixer(cfg, t, h, cuts, block=64), want, 1e-3)
    quiet = _mixer_oracle(cfg, t, _loud(-1, L, mix)[2])
    assert (want[-1] - quiet[-1]).norm() > 0.3 * want[-1].norm()


@pytest.mark.parametrize("mix", [win(), temp(), conv()],
                         ids=["window", "temperature", "convolution"])
def test_the_sink_shows_where_scores_are_low(mix, monkeypatch):
    """Small queries give scores near zero: the first tokens then lose a large
    share to the sink, and an oracle without it is far off."""
    cfg = config([(mix, None)])
    t = tensors(cfg, 5)
    t["l0.mix.q"] *= 0.05
    h = rnd(12, 24, seed=6)
    want = _mixer_oracle(cfg, t, h)
    got = _run_mixer(cfg, t, h, [5, 1, 1, 5])
    close(got, want)
    monkeypatch.setattr(O, "softmax_rest",
                        lambda s, rest: torch.softmax(s, 0))
    differs(got, _mixer_oracle(cfg, t, h), 0.5)


def test_temperature_steps_between_the_right_positions(monkeypatch):
    cfg = config([(temp(coef=3.0, every=8, scale=1.0), None)])
    t = tensors(cfg, 7)
    h = rnd(20, 24, seed=8)
    got = _run_mixer(cfg, t, h, [6, 1, 1, 1, 11])
    close(got, _mixer_oracle(cfg, t, h))
    real = O.query_temperature
    monkeypatch.setattr(O, "query_temperature",
                        lambda p, c, e: real(p - 1, c, e))    # one off
    off = _mixer_oracle(cfg, t, h)
    close(got[:7], off[:7])
    differs(got[7:8], off[7:8], 0.05)


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
    assert len(taps) == len(want) == 5
    for got, ref in zip(taps, want):
        close(got.cpu().double(), ref)


def test_cache_streams_and_states(base):
    cache = base.batcher.cache
    assert [p.shape[-1] for p in cache.pools] == \
        [2 * 2 * 10, 2 * 18, 14, 2 * 3 * 6, 14]
    assert {k: tuple(s.shape[1:]) for k, s in cache.states.items()} == \
        {"conv1": (2, 24 + 24 + 12), "conv4": (1, 24 + 6 + 8)}


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
    leaving rows and convolution tails behind; the first has one token, so
    its tail holds less than the convolution is long."""
    s = Served(BASE, slots=2, max_tokens=64, block=16)
    for k in range(6):
        t = toks(20 + k if k else 12, seed=40 + k)
        other = toks(9, seed=80 + k)
        b = s.batcher
        r1, r2 = b.open("a%d" % k), b.open("b%d" % k)
        n = 11 if k else 1
        got = b.feed([(r1, t[:n]), (r2, other)]).cpu()[:n]
        got = torch.cat([got, b.feed([(r1, t[n:])]).cpu()])
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
    "wide_heads": config(
        [(win(heads=2, kv=1, dim=20, dims=12, size=4, keep=0, factor=1.0,
              scale=1.1), dense(7)),
         (temp(heads=6, kv=3, dim=4, vdim=11, every=1, coef=0.2), dense(50))],
        width=16, scale=0.5),
    "convolutions_of_every_length": config(
        [(conv(heads=3, kv=3, dim=8, vdim=8, taps=1, dims=8), None),
         (conv(heads=2, kv=1, dim=16, vdim=8, taps=4, dims=16), dense(11)),
         (conv(heads=5, kv=5, dim=4, vdim=7, taps=6, dims=2), dense(8))],
        width=20, vocab=29, eps=1e-3),
    "windows_of_one_and_of_all": config(
        [(win(heads=4, kv=4, dim=8, dims=8, size=1, keep=4), None),
         (win(heads=8, kv=2, dim=6, dims=2, size=400, keep=0,
              original=300), dense(33)), (win(size=2, keep=40), dense(5))],
        width=12, vocab=53, scale=5.0),
    "one_layer": config([(temp(heads=1, kv=1, dim=3, vdim=3, coef=0.0,
                               every=64), dense(3))], width=9, vocab=7),
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
    close_rms(s.run(t, [30]), want, 0.02)
    close_rms(s.run(t, [7, 1, 20, 1, 1]), want, 0.02)


def test_what_stays_32_bit_in_16_bit_serving():
    s = Served(BASE, dtype=torch.bfloat16)
    m = s.model.layers
    assert {m[0].norm1.alpha.dtype, m[0].norm1.weight.dtype,
            m[0].norm1.bias.dtype, m[1].att.sink.dtype, m[2].att.q_norm.dtype,
            m[0].att.sink.dtype} == {torch.float32}
    assert s.batcher.cache.states["conv1"].dtype == torch.bfloat16
    assert s.batcher.cache.pools[0].dtype == torch.bfloat16
    taps = []
    b = s.batcher
    r = b.open("x")
    b.cache.begin_ragged([r.slot], [3])
    s.model(torch.tensor(toks(3), device=DEV), kv_cache=b.cache, taps=taps)
    b.cache.end_step()
    b.close(r)
    assert {x.dtype for x in taps} == {torch.float32}


# ------------------------------- mid size, default 64-token blocks
def _mid_config():
    return config(
        [(conv(heads=6, kv=2, dim=24, vdim=16, taps=4, dims=16, scale=0.2,
               base=3000.0, original=64, fast=8.0), dense(152)),
         (win(heads=4, kv=1, dim=32, dims=24, size=48, keep=5, scale=0.3,
              base=3000.0, original=64, fast=8.0), dense(80)),
         (temp(heads=2, kv=2, dim=64, vdim=40, scale=0.12, every=33), None),
         (win(heads=2, kv=2, dim=64, dims=64, size=70, keep=1, scale=0.12,
              base=500.0, original=32), dense(64)),
         (conv(heads=4, kv=2, dim=40, vdim=136, taps=3, dims=32, scale=0.15),
          dense(96))], width=96, vocab=131, eps=1e-6)


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
    cfg = VARIANTS["convolutions_of_every_length"]
    t = {k: v.bfloat16().float() for k, v in tensors(cfg, seed=8).items()}
    _save(tmp_path, cfg, t)
    model = load_pretrained(str(tmp_path), dtype=torch.float32, device=DEV)
    assert model.architecture == "Fubolix"
    assert model.cfg.to_dict() == cfg
    b = ContinuousBatcher(model, max_slots=1, dtype=torch.float32,
                          device=torch.device(DEV), max_tokens=64)
    r = b.open("x")
    seq = toks(10, vocab=cfg["vocab"])
    got = b.feed([(r, seq)], rows=[9]).cpu().double()
    want = O.forward(cfg, {k: v.double() for k, v in t.items()}, seq)
    close(got, want[9:])
    # the parameters go back out under the checkpoint's names
    back = model.named_tensors()
    assert set(back) == set(t)
    for k, v in t.items():
        assert torch.equal(back[k].float().cpu(), v), k


def test_every_tensor_of_a_checkpoint_is_read():
    for cfg in [BASE, _mid_config()] + list(VARIANTS.values()):
        model = build_model(cfg, torch.float32)
        assert {n for n, _ in model._named_parts()} == set(tensors(cfg))


def test_config_rejects_what_the_design_does_not_have():
    def with_key(mix, key, value):
        return {**mix, "mixer": {**mix["mixer"], key: value}}

    for layers in (
            [({"type": "conv", "mixer": {}}, None)],
            [(win(dims=3), None)],                          # odd rotation
            [(win(dims=12), None)],                         # wider than a head
            [(win(heads=3, kv=2), None)],
            [(with_key(win(), "vdim", 6), None)],           # values are keys
            [(with_key(temp(), "rot", _rot(10.0, 4)), None)],
            [(with_key(conv(), "mask", {"size": 4}), None)],
            [(temp(every=0), None)], [(conv(taps=0), None)],
            [(temp(), {"kind": "moe", "ff": 8})]):
        with pytest.raises(ValueError):
            build_model(config(layers))
    t = tensors(BASE)
    t["l0.norm1.b"] = t["l0.norm1.b"][:-1]
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
    la, lb, lc = (O.forward(cfg, w, s) for s in (a, b, c))
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
    cfg = VARIANTS["windows_of_one_and_of_all"]
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
    assert len(lines) == 2
    w = {k: v.double() for k, v in t.items()}
    for prompt, line in zip((a, b), lines):
        seq = list(prompt)
        for _ in range(3):
            seq.append(int(O.forward(cfg, w, seq)[-1].argmax()))
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


def test_declared_kernel_arguments_match_the_sources():
    """Entry points whose argument kinds Python declares: as the C source
    has them."""
    import re
    from deepspeed_amd.ops import serving_kernels as sk
    for lib, table in sk._SIGNATURES.items():
        with open(sk.LIBRARIES[lib][0]) as f:
            src = f.read()
        for name, kinds in table.items():
            args = re.search(r"int %s\((.*?)\)\s*\{" % name, src, re.S)
            got = ""
            for a in args.group(1).split(","):
                a = a.strip()
                got += "p" if "*" in a or "hipStream_t" in a else \
                    "l" if "int64_t" in a else "f" if "float" in a else "i"
            assert got == kinds, name


# ------------------------------------------- HIP kernels against eager ops
@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("which", ["base", "mid"])
def test_kernels_match_eager_on_the_same_device(which, dtype, monkeypatch):
    from deepspeed_amd.ops import serving_kernels as sk
    cfg = BASE if which == "base" else _mid_config()
    t = toks(40, cfg["vocab"], seed=12)
    s = Served(cfg, dtype=dtype)
    kern = s.run(t, [17, 1, 1, 21])
    monkeypatch.setenv("DS_AMD_SERVING_EAGER", "1")
    assert not sk.enabled()
    eager = s.run(t, [17, 1, 1, 21])
    if dtype == torch.float32:
        close(kern, eager, 1e-4)
    else:
        close_rms(kern, eager, 0.02)


@pytest.mark.gpu
def test_kernel_libraries_are_loaded():
    from deepspeed_amd.ops import serving_kernels as sk
    Served(BASE).run(toks(5), [5])
    assert {"seq", "rows"} <= set(sk._libs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mid_size_mixed_schedule_on_the_kernels(dtype):
    s, seqs, got = _mixed_schedule(dtype)
    for k, t in seqs.items():
        if dtype == torch.float32:
            close(torch.cat(got[k]), s.oracle(t), 5e-4)
        else:
            close_rms(torch.cat(got[k]), s.oracle(t), 0.02)


@pytest.mark.gpu
@pytest.mark.parametrize("mix,target,L", [
    (win(size=SIZE, keep=KEEP, scale=2.0), KEEP, KEEP + SIZE + 6),
    (win(size=SIZE, keep=KEEP, scale=2.0), KEEP - 1, KEEP + SIZE + 6),
    (win(size=SIZE, keep=KEEP, scale=2.0, dim=16), 64, 64 + SIZE + 6),
    (temp(scale=1.0, every=40), 63, 260), (conv(scale=0.1), 64, 260),
    (conv(scale=0.1, dim=16, vdim=8, dims=0), 0, 200)])
def test_crafted_keys_on_the_kernels(mix, target, L):
    cfg, t, h = _loud(target, L, mix)
    want = _mixer_oracle(cfg, t, h)
    for cuts in ([L], [L - 9, 2, 3, 4], [L - 10] + [1] * 10):
        close(_run_mixer(cfg, t, h, cuts, block=64), want, 1e-3)


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
@pytest.mark.parametrize("C", [1, 13, 24, 200, 520, 1000, 4096, 4099, 8192])
def test_dynamic_tanh_kernel_against_eager(C, dtype, monkeypatch):
    from deepspeed_amd.ops.norms import residual_tanh
    al = torch.tensor([0.4]).to(DEV)
    w, b = rnd(C, seed=1).to(DEV), rnd(C, seed=2).to(DEV)
    for T in (1, 3, 70, 1030):
        x0, y = 4 * rnd(T, C).to(DEV), rnd(T, C, seed=3).to(DEV, dtype)
        rows = torch.tensor([T - 1, 0, T // 2]).to(DEV)
        for yy, idx in ((y, None), (None, None), (y, rows), (None, rows)):
            def run():
                x = x0.clone()
                return residual_tanh(x, yy, al, w, b, dtype, idx), x

            got, want = _both(monkeypatch, run)
            near(got[0], want[0], dtype)
            assert torch.equal(got[1], want[1])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_relu_squared_kernel_against_eager(dtype, monkeypatch):
    from deepspeed_amd.ops.activations import act_rows
    for T, F, pad in ((3, 40, 8), (5, 13, 3), (600, 1024, 16), (7, 24, 5)):
        z = rnd(T, F + pad).to(DEV, dtype)[:, pad:]

        def run():
            wide = torch.zeros(T, F + 2 * pad, device=DEV, dtype=dtype)
            act_rows(z, "relu2", out=wide[:, pad:pad + F])
            return wide

        got, want = _both(monkeypatch, run)
        assert torch.equal(got, want)


PREPS = [  # heads, kv, dim, vdim, rotated, layout, norm, taps, keys as values
    (6, 2, 64, 64, 32, "interleaved", "after", 0, True),
    (4, 2, 10, 10, 8, "interleaved", "after", 0, True),
    (8, 1, 128, 128, 128, "half", "after", 0, True),
    (3, 3, 24, 24, 6, "interleaved", "after", 0, True),
    (6, 2, 80, 88, 48, "half", None, 3, False),
    (4, 2, 96, 40, 32, "half", None, 4, False),
    (2, 2, 16, 24, 16, "half", None, 2, False),
    (2, 1, 256, 128, 64, "half", "head", 4, False),
    (2, 1, 320, 512, 64, "interleaved", "after", 2, False),
    (2, 1, 8, 8, 0, "half", "head", 3, False),
    (3, 1, 24, 16, 8, "half", None, 3, False),      # pairs inside a group
    (2, 2, 12, 6, 6, "half", None, 3, False),
    (2, 2, 16, 16, 16, "half", None, 6, False),
    (2, 2, 16, 16, 16, "half", None, 1, False),
    (4, 2, 64, 48, 0, "half", "head", 0, False),
    (5, 1, 9, 7, 0, "half", "head", 0, False)]


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,dims,layout,norm,taps,vk", PREPS)
def test_prologue_kernel_against_eager(H, G, d, dv, dims, layout, norm, taps,
                                       vk, dtype, monkeypatch):
    """Queries, pool rows, convolution tails and the side activation, over
    single-token steps, portions beside single tokens, and a long step whose
    workgroups take several tokens across sequence borders."""
    from deepspeed_amd.ops.rope import rope_tables, temperature_table
    from deepspeed_amd.ops.window_attention import attn_prep
    n_in = H * d + G * (d + (0 if vk else dv))
    ff = 72
    wq, wk = (1 + 0.2 * rnd(d, seed=k).to(DEV) for k in (1, 2))
    cw = rnd(n_in, taps, seed=3).to(DEV, dtype) if taps else None
    cos, sin = rope_tables(dims, 2048, 500.0, device=DEV) if dims \
        else (None, None)
    tab = temperature_table(2048, 0.6, 3, DEV)
    cases = [([0, 7, 1, 30], [1, 1, 1, 1]), ([0, 5, 1], [9, 1, 2]),
             ([3, 0, 2, 0], [301, 2, 1, 250])]
    ld = (n_in + ff + 7) // 8 * 8
    for held, counts in cases:
        T = sum(counts)
        wide = rnd(T, ld, seed=T).to(DEV, dtype)
        st0 = rnd(len(held), max(taps - 1, 0), n_in, seed=5).to(DEV, dtype)
        for i, n in enumerate(held):      # nothing before position 0
            st0[i, :max(0, taps - 1 - n)] = 0

        def run():
            cache, bt = begun({}, held, counts, [G * (d + dv)], dtype=dtype)
            st = st0.clone()
            both = torch.zeros(T, 16 + ff, device=DEV, dtype=dtype)
            q = attn_prep(wide[:, :n_in], bt, cache.pools[0],
                          wq if norm == "head" else None,
                          wk if norm == "head" else None, 1e-4, H, G, d, dv,
                          dims, cos, sin, norm=norm, layout=layout,
                          conv=(cw, st) if taps else None, v_from_k=vk,
                          q_factor=tab,
                          side=(wide[:, n_in:n_in + ff], both[:, 16:],
                                "relu2"))
            return q, cache.pools[0], both, st

        got, want = _both(monkeypatch, run)
        near(got[0], want[0], dtype)
        near(got[1], want[1], dtype)
        assert torch.equal(got[2], want[2])
        assert torch.equal(got[3], want[3])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,window,keep", [
    (6, 2, 64, 64, 70, 3), (4, 1, 80, 96, 0, 0), (8, 2, 128, 128, 0, 0),
    (3, 3, 20, 12, 9, 2), (6, 1, 200, 130, 0, 0), (2, 1, 16, 24, 300, 40)])
def test_attention_kernels_with_sink_and_gate(H, G, d, dv, window, keep,
                                              dtype, monkeypatch):
    """Both kernels (tiles in 16 bits; exact), whole and split keys."""
    from deepspeed_amd.ops import serving_kernels as sk
    from deepspeed_amd.ops import window_attention as wa
    sink = (3 * rnd(H, seed=4)).to(DEV)
    for held, counts in (([0], [1]), ([900, 3, 64], [1, 1, 1]),
                         ([0, 63, 200], [130, 2, 1]), ([500], [40])):
        T = sum(counts)
        cache, bt = begun({}, held, counts, [G * (d + dv)], block=64,
                          dtype=dtype)
        cache.pools[0].copy_(rnd(*cache.pools[0].shape, seed=1))
        q = rnd(T, H, d, seed=2).to(DEV, dtype)
        gate = rnd(T, H + 5, seed=3).to(DEV, dtype)[:, 5:]
        for s, g in ((sink, gate), (sink, None), (None, gate),
                     (torch.zeros_like(sink), None)):
            args = (q, cache.pools[0], bt, G, d, dv, d ** -0.5, window, keep)
            got, want = _both(monkeypatch, lambda: wa.window_attention(
                *args, sink=s, gate=g))
            near(got, want, dtype)
            if dtype == torch.bfloat16:
                near(sk.window_attention(*args, path="exact", sink=s, gate=g),
                     want, dtype)
