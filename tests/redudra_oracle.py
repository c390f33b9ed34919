"""A plain, slow formulation of the Redudra design's mechanisms, one function
per mechanism, written from its equations for whole sequences (no cache, no
batching, no steps). float64 throughout; it shares no code with the serving
path and is what the tests compare against.

Weights arrive as a dict of tensors under their checkpoint names
('l<i>.mix.left.q', 'l<i>.mlp.up', ...), linear weights stored [out, in].
"""

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    inner = math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)
    return 0.5 * z * (1.0 + torch.tanh(inner))


def softplus(z):
    return torch.where(z > 30, z,
                       torch.log1p(torch.exp(torch.clamp(z, max=30))))


def lin(w, x, b=None):
    y = x @ w.to(F64).t()
    return y if b is None else y + b.to(F64)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    var = (d * d).mean(-1, keepdim=True)
    return d / torch.sqrt(var + eps) * w.to(F64) + b.to(F64)


# ----------------------------------------------------------- token shift
def token_shift(h, mu):
    """Row t moves towards row t-1 by mu per column; the row before the first
    is zero."""
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        prev = h[t - 1] if t > 0 else torch.zeros_like(h[0])
        out[t] = h[t] + (prev - h[t]) * mu.to(F64)
    return out


# -------------------------------------------------------------- rotation
def frequencies(rot):
    """(frequency per pair, factor on cos and sin)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])

    def turn_dim(turns):
        return dims * math.log(orig / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(turn_dim(float(sc["fast"]))), 0)
    hi = min(math.ceil(turn_dim(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = (i - lo) / max(hi - lo, 0.001)
        ramp = min(max(ramp, 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, rot):
    """x [L, heads, d]; coordinate i pairs with i + dims/2 among the first
    ``dims``."""
    dims = int(rot["dims"])
    half = dims // 2
    f, mag = frequencies(rot)
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(half):
            c, s = mag * math.cos(p * f[i]), mag * math.sin(p * f[i])
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * c - v * s
            out[p, :, i + half] = v * c + u * s
    return out


# ---------------------------------------------------------------- mixers
def sees(i, j, size, keep_first):
    return j <= i and (i - j < size or j < keep_first)


def window_attention(h, w, pre, m):
    L = h.shape[0]
    H, G = int(m["heads"]), int(m["kv_heads"])
    d, dv = int(m["dim"]), int(m["vdim"])
    q = rotate(lin(w[pre + "q"], h).view(L, H, d), m["rot"])
    k = rotate(lin(w[pre + "k"], h).view(L, G, d), m["rot"])
    v = lin(w[pre + "v"], h).view(L, G, dv)
    size, keep = int(m["mask"]["size"]), int(m["mask"]["keep_first"])
    out = torch.zeros(L, H, dv, dtype=F64)
    for i in range(L):
        js = [j for j in range(i + 1) if sees(i, j, size, keep)]
        for hh in range(H):
            g = hh // (H // G)
            s = (k[js, g] @ q[i, hh]) * float(m["scale"])
            p = torch.exp(s - s.max())
            out[i, hh] = (p[:, None] * v[js, g]).sum(0) / p.sum()
    return lin(w[pre + "o"], out.reshape(L, H * dv))


def retention(h, w, pre, m, eps):
    L = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = rotate(lin(w[pre + "q"], h).view(L, H, d), m["rot"])
    k = rotate(lin(w[pre + "k"], h).view(L, H, d), m["rot"]) * d ** -0.5
    v = lin(w[pre + "v"], h).view(L, H, dv)
    o = torch.zeros(L, H, dv, dtype=F64)
    for hh in range(H):
        S = torch.zeros(d, dv, dtype=F64)
        for t in range(L):
            S = float(m["decay"][hh]) * S + torch.outer(k[t, hh], v[t, hh])
            o[t, hh] = S.t() @ q[t, hh]
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return lin(w[pre + "o"], o.reshape(L, H * dv) * silu(lin(w[pre + "g"], h)))


def parallel(h, w, pre, m, eps):
    return float(m["left_scale"]) * window_attention(
        h, w, pre + "left.", m["left"]) + float(m["right_scale"]) * retention(
            h, w, pre + "right.", m["right"], eps)


def causal_conv(x, w, b):
    """x [L, C]; w [C, taps], the last column multiplies the current input;
    zeros before the start."""
    L, taps = x.shape[0], w.shape[1]
    w = w.to(F64)
    out = b.to(F64).repeat(L, 1)
    for t in range(L):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


def block_linear(w, b, x):
    """w [blocks, n, n] ([out, in] each), b [blocks, n]; x [L, blocks*n]."""
    n = w.shape[1]
    return torch.cat([lin(w[j], x[:, j * n:(j + 1) * n], b[j])
                      for j in range(w.shape[0])], -1)


def rglru_scan(u, r, i, lam):
    """Gated diagonal recurrence from a zero state."""
    L, C = u.shape
    S = torch.zeros(C, dtype=F64)
    out = torch.zeros(L, C, dtype=F64)
    rate = softplus(lam.to(F64))
    for t in range(L):
        log_a = -8.0 * r[t] * rate
        a = torch.exp(log_a)
        S = a * S + torch.sqrt(1.0 - a * a) * i[t] * u[t]
        out[t] = S
    return out


def rglru(h, w, pre, m, eps):
    y = gelu_tanh(lin(w[pre + "y"], h, w[pre + "y.b"]))
    u = causal_conv(lin(w[pre + "x"], h, w[pre + "x.b"]), w[pre + "conv"],
                    w[pre + "conv.b"])
    r = sigmoid(block_linear(w[pre + "ra"], w[pre + "ra.b"], u))
    i = sigmoid(block_linear(w[pre + "ri"], w[pre + "ri.b"], u))
    return lin(w[pre + "o"], rglru_scan(u, r, i, w[pre + "lam"]) * y)


# ---------------------------------------------------------- feed-forward
def dense_ff(h, w, pre):
    g = lin(w[pre + "gate"], h, w[pre + "gate.b"])
    u = lin(w[pre + "up"], h, w[pre + "up.b"])
    return lin(w[pre + "down"], silu(g) * u, w[pre + "down.b"])


# ----------------------------------------------------------------- model
MIXERS = {"rglru": rglru, "parallel": parallel}


def layer(x, w, cfg, i):
    spec, eps, pre = cfg["layers"][i], float(cfg["norm"]["eps"]), f"l{i}."
    mult = float(cfg["residual_mult"])
    h = layer_norm(x, w[pre + "norm1"], w[pre + "norm1.b"], eps)
    h = token_shift(h, w[pre + "shift"])
    x = x + mult * MIXERS[spec["type"]](h, w, pre + "mix.", spec["mixer"],
                                        eps)
    if spec.get("mlp"):
        h = layer_norm(x, w[pre + "norm2"], w[pre + "norm2.b"], eps)
        x = x + mult * dense_ff(h, w, pre + "mlp.")
    return x


def layer_order(cfg):
    """[(layer, row of 'loop.step' added before it or None)]."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    order = [(i, None) for i in range(a)]
    for t in range(int(loop["times"])):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def forward(tokens, w, cfg, streams=None):
    """Logits [L, vocab] of one whole sequence. ``streams`` (a list) receives
    the residual stream after every layer run."""
    x = w["embed"].to(F64)[torch.tensor(list(tokens), dtype=torch.long)]
    for i, step in layer_order(cfg):
        if step is not None:
            x = x + w["loop.step"][step].to(F64)
        x = layer(x, w, cfg, i)
        if streams is not None:
            streams.append(x.clone())
    x = layer_norm(x, w["final.norm"], w["final.norm.b"],
                   float(cfg["norm"]["eps"]))
    cap = float(cfg["logit_softcap"])
    return cap * torch.tanh(lin(w["head"], x) / cap)
