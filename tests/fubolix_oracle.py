"""A plain, slow formulation of the Fubolix design's mechanisms, one function
per mechanism, written from its equations for whole sequences (no cache, no
batching, no steps). float64 throughout; it shares no code with the serving
path and is what the tests compare against.

Weights arrive as a dict of tensors under their checkpoint names
('l<i>.mix.q', 'l<i>.mlp.up', ...), linear weights stored [out, in].
"""

import math

import torch

F64 = torch.float64


def lin(w, x):
    return x @ w.to(F64).t()


# ----------------------------------------------------------------- norms
def dynamic_tanh(x, alpha, w, b):
    """No statistic of the row: every coordinate alone."""
    a = float(alpha.to(F64))
    return torch.tanh(a * x) * w.to(F64) + b.to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


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
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, rot, pairing):
    """x [L, heads, d]. ``pairing``: "neighbours" (2i with 2i+1) or "halves"
    (i with i + dims/2), among the first ``dims`` coordinates."""
    dims = int(rot["dims"])
    f, mag = frequencies(rot)
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(dims // 2):
            a, b = (2 * i, 2 * i + 1) if pairing == "neighbours" \
                else (i, i + dims // 2)
            c, s = mag * math.cos(p * f[i]), mag * math.sin(p * f[i])
            u, v = x[p, :, a], x[p, :, b]
            out[p, :, a] = u * c - v * s
            out[p, :, b] = v * c + u * s
    return out


# ------------------------------------------------------- short convolution
def short_conv(u, w):
    """u [L, C]; the last column of w weighs the current token."""
    L, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(L):
        for j in range(taps):
            src = t - taps + 1 + j
            if src >= 0:
                y[t] += w[:, j].to(F64) * u[src]
    return y


# ------------------------------------------------------- query temperature
def query_temperature(p, coef, every):
    return 1.0 + coef * math.log(math.floor((p + 1) / every) + 1)


# -------------------------------------------------------------- attention
def sees(i, j, mask):
    if j > i:
        return False
    if mask is None:
        return True
    return i - j < int(mask["size"]) or j < int(mask.get("keep_first", 0))


def softmax_rest(s, rest):
    """exp(s_j) / (exp(rest) + sum exp(s_j)): ``rest`` is a score without a
    key and a value."""
    m = max(float(s.max()), float(rest))
    e = torch.exp(s - m)
    return e / (math.exp(float(rest) - m) + e.sum())


def attend(q, k, v, scale, mask, sink):
    """q [L, H, d], k [L, G, d], v [L, G, dv]; sink [H]."""
    L, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(L, H, v.shape[2], dtype=F64)
    for i in range(L):
        js = [j for j in range(i + 1) if sees(i, j, mask)]
        for h in range(H):
            g = h // (H // G)
            p = softmax_rest((k[js, g] @ q[i, h]) * scale, sink[h])
            out[i, h] = (p[:, None] * v[js, g]).sum(0)
    return out


# ----------------------------------------------------------------- mixers
def _sizes(m):
    return (int(m["heads"]), int(m["kv_heads"]), int(m["dim"]),
            int(m["vdim"]))


def mixer_attention(h, w, pre, m, eps):
    """Values are the keys as projected; unit-RMS queries and keys after the
    rotation; window with kept first tokens; one gate per head."""
    L = h.shape[0]
    H, G, d, dv = _sizes(m)
    q = lin(w[pre + "q"], h).view(L, H, d)
    k = lin(w[pre + "k"], h).view(L, G, d)
    v = k.clone()
    q = unit_rms(rotate(q, m["rot"], "neighbours"), eps)
    k = unit_rms(rotate(k, m["rot"], "neighbours"), eps)
    o = attend(q, k, v, float(m["scale"]), m["mask"], torch.zeros(H))
    gate = 1.0 / (1.0 + torch.exp(-lin(w[pre + "g"], h)))       # [L, H]
    o = o * gate[:, :, None]
    return lin(w[pre + "o"], o.reshape(L, H * dv))


def mixer_attention_2(h, w, pre, m, eps):
    """No rotation; weighted per-head norms; queries grow with position."""
    L = h.shape[0]
    H, G, d, dv = _sizes(m)
    q = unit_rms(lin(w[pre + "q"], h).view(L, H, d), eps) \
        * w[pre + "q.norm"].to(F64)
    k = unit_rms(lin(w[pre + "k"], h).view(L, G, d), eps) \
        * w[pre + "k.norm"].to(F64)
    v = lin(w[pre + "v"], h).view(L, G, dv)
    t = m["q_temp"]
    for p in range(L):
        q[p] *= query_temperature(p, float(t["coef"]), t["every"])
    o = attend(q, k, v, float(m["scale"]), None, torch.zeros(H))
    return lin(w[pre + "o"], o.reshape(L, H * dv))


def mixer_attention_3(h, w, pre, m, eps):
    """Short convolutions on q, k and v, then the rotation; a learned sink."""
    L = h.shape[0]
    H, G, d, dv = _sizes(m)
    q, k, v = (short_conv(lin(w[pre + n], h), w[pre + n + ".conv"])
               for n in "qkv")
    q = rotate(q.view(L, H, d), m["rot"], "halves")
    k = rotate(k.view(L, G, d), m["rot"], "halves")
    o = attend(q, k, v.view(L, G, dv), float(m["scale"]), None,
               w[pre + "sink"].to(F64))
    return lin(w[pre + "o"], o.reshape(L, H * dv))


MIXERS = {"attention": mixer_attention, "attention_2": mixer_attention_2,
          "attention_3": mixer_attention_3}


# ------------------------------------------------------------ feed-forward
def feed_forward(h, w, pre):
    z = lin(w[pre + "up"], h)
    z = torch.where(z > 0, z * z, torch.zeros_like(z))
    return lin(w[pre + "down"], z)


# ------------------------------------------------------------- whole model
def embed(ids, w, scale):
    return w["embed"].to(F64)[torch.as_tensor(ids)] * scale


def layer(x, w, i, spec, eps):
    pre = f"l{i}."
    h = dynamic_tanh(x, w[pre + "norm1.alpha"], w[pre + "norm1"],
                     w[pre + "norm1.b"])
    y = MIXERS[spec["type"]](h, w, pre + "mix.", spec["mixer"], eps)
    if spec.get("mlp"):
        y = y + feed_forward(h, w, pre + "mlp.")
    return x + y


def forward(cfg, w, ids, layers_out=None):
    """Logits [len(ids), vocab] of one sequence; ``layers_out`` receives the
    stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embed(ids, w, float(cfg["embedding"]["scale"]))
    for i, spec in enumerate(cfg["layers"]):
        x = layer(x, w, i, spec, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    h = dynamic_tanh(x, w["final.norm.alpha"], w["final.norm"],
                     w["final.norm.b"])
    return lin(w["head"], h)
