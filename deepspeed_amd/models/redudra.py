"""Redudra: a decoder-only serving model that alternates gated diagonal
recurrences with layers in which windowed attention and retention run side by
side, assembled from the framework's ragged-batch mechanisms.

* a layer is pre-norm (layer norm with weight and bias) on an fp32 stream and
  adds each sublayer's result times one constant:
  ``x += m * mixer(shift(norm1(x)))``, ``x += m * ff(norm2(x))``;
* the mixer's input is mixed with the previous token's normed row, per column
  ("token shift"); that row is carried per request slot. The residual add of
  one sublayer, the norm and the shift of the next are one pass
  (ops/norms.py ``residual_norm``);
* mixer ``rglru``: two projected branches; one passes a short causal
  convolution and a real-gated linear recurrent unit with block-diagonal gates
  (ops/gated_recurrence.py), the other gates the read-out through a tanh GELU;
* mixer ``parallel``: grouped-query attention with a sliding window that keeps
  the first tokens and YaRN-scaled rotate-half positions
  (ops/window_attention.py), beside retention: the plain matrix-state
  recurrence with one fixed decay per head, rotated queries and keys and an
  unweighted per-head RMS norm under a SiLU gate (ops/linear_recurrence.py).
  Both read ONE fused input projection and feed ONE fused output projection;
* feed-forward: dense, SiLU-gated, with biases;
* a block of layers may run several times with the same weights; every layer
  RUN has its own cache stream and slot states, and a learned row per pass is
  added to the stream before the pass's first layer;
* logits are capped by ``cap * tanh(z / cap)`` and returned in fp32.

The model runs only through a ``PagedStateCache`` step: ``forward`` takes the
flat token list of a ragged batch. Every size and constant comes from the
config.
"""

from dataclasses import dataclass
from typing import List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..inference.state_cache import PagedStateCache
from ..ops.activations import softcap_rows
from ..ops.gated_recurrence import rglru_mix
from ..ops.linear_recurrence import retention_mix
from ..ops.norms import embed_rows, residual_norm
from .lolulorn import GatedMLP, PostNorm
from .savovik import GroupedAttention, rot_tables

MIXERS = ("rglru", "parallel")


@dataclass
class RedudraConfig:
    vocab_size: int
    width: int
    layers: List[dict]
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    logit_softcap: float = 0.0        # 0: logits pass unchanged
    loop: Optional[dict] = None       # {start, stop, times}
    max_seq_len: int = 1 << 16

    @classmethod
    def from_dict(cls, d: dict) -> "RedudraConfig":
        cfg = cls(vocab_size=int(d["vocab"]), width=int(d["width"]),
                  layers=list(d["layers"]), norm_eps=float(d["norm"]["eps"]),
                  residual_mult=float(d.get("residual_mult", 1.0)),
                  logit_softcap=float(d.get("logit_softcap") or 0.0),
                  loop=d.get("loop"))
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        d = {"architecture": "Redudra", "vocab": self.vocab_size,
             "width": self.width, "layers": self.layers,
             "norm": {"eps": self.norm_eps},
             "residual_mult": self.residual_mult,
             "logit_softcap": self.logit_softcap}
        if self.loop:
            d["loop"] = self.loop
        return d

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def validate(self):
        for i, spec in enumerate(self.layers):
            if spec["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {spec['type']!r}")
            mlp = spec.get("mlp")
            if mlp and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown mlp kind "
                                 f"{mlp['kind']!r}")
        if self.loop:
            a, b, t = (int(self.loop[k]) for k in ("start", "stop", "times"))
            if not (0 <= a <= b <= len(self.layers)) or t < 0:
                raise ValueError("loop: need 0 <= start <= stop <= layers "
                                 "and times >= 0")

    def layer_runs(self):
        """[(layer, pass it opens or None)] in execution order; the index in
        this list names the run's cache stream and slot states."""
        n = len(self.layers)
        if not self.loop:
            return [(i, None) for i in range(n)]
        a, b, times = (int(self.loop[k]) for k in ("start", "stop", "times"))
        runs = [(i, None) for i in range(a)]
        for t in range(times):
            runs += [(i, t if i == a else None) for i in range(a, b)]
        return runs + [(i, None) for i in range(b, n)]


def _w(*shape, dtype):
    return nn.Parameter(torch.empty(*shape, dtype=dtype), requires_grad=False)


class RGLRUMixer(nn.Module):
    """Mixer 'rglru': fused biased projection y | x."""

    def __init__(self, width, m: dict, eps, dtype):
        super().__init__()
        self.inner, self.blocks = int(m["width"]), int(m["blocks"])
        self.taps = int(m.get("conv", 1))
        if self.inner % self.blocks or self.taps < 1:
            raise ValueError("rglru: width must be a multiple of blocks")
        C, n = self.inner, self.inner // self.blocks
        self.w_in = _w(2 * C, width, dtype=dtype)
        self.b_in = _w(2 * C, dtype=dtype)
        self.conv = _w(C, self.taps, dtype=dtype)
        self.conv_b = _w(C, dtype=torch.float32)
        self.w_r = _w(self.blocks, n, n, dtype=dtype)
        self.w_i = _w(self.blocks, n, n, dtype=dtype)
        self.b_r = _w(C, dtype=torch.float32)
        self.b_i = _w(C, dtype=torch.float32)
        self.lam = _w(C, dtype=torch.float32)
        self.w_o = _w(width, C, dtype=dtype)

    row_dim = 0          # nothing cached per token: the state is per slot

    def state_shapes(self, dtype):
        return {"conv": ((self.taps - 1, self.inner), dtype),
                "rec": ((self.inner,), torch.float32)}

    def forward(self, h, cache: PagedStateCache, stream, states):
        b = cache.batch
        y = rglru_mix(F.linear(h, self.w_in, self.b_in), self.conv,
                      self.conv_b, states["conv"], self.w_r, self.b_r,
                      self.w_i, self.b_i, self.lam, states["rec"], b)
        return F.linear(y, self.w_o)


class WindowRetentionMixer(nn.Module):
    """Mixer 'parallel': windowed attention beside retention. ONE input
    projection ``q | k | v`` (attention) ``| q | k | v | g`` (retention) and
    ONE output projection over ``[left_scale * attention ; right_scale *
    retention]`` (the scales are applied in fp32 where the two are made)."""

    def __init__(self, width, m: dict, eps, dtype):
        super().__init__()
        self.att = GroupedAttention(m["left"], eps, dtype, bias=False,
                                    qk_norm=False, layout="half",
                                    v_unit=False, mask="window")
        r = m["right"]
        self.heads, self.dim, self.vdim = int(r["heads"]), int(r["dim"]), \
            int(r["vdim"])
        self.rot = r.get("rot") or {"dims": 0}
        self.rot_dims = int(self.rot.get("dims", 0))
        self.decay = [float(x) for x in r["decay"]]
        if len(self.decay) != self.heads or self.rot_dims % 2 or \
                self.rot_dims > self.dim:
            raise ValueError("retention: one decay per head, and rot.dims "
                             "even and at most dim")
        self.left_scale = float(m.get("left_scale", 1.0))
        self.right_scale = float(m.get("right_scale", 1.0))
        self.eps = eps
        self.n_qk, self.n_v = self.heads * self.dim, self.heads * self.vdim
        self.w_in = _w(self.att.n_in + 2 * self.n_qk + 2 * self.n_v, width,
                       dtype=dtype)
        self.w_o = _w(width, self.att.n_out + self.n_v, dtype=dtype)
        self.register_buffer("head_decay", torch.tensor(
            self.decay, dtype=torch.float32), persistent=False)

    @property
    def row_dim(self):
        return self.att.row_dim

    def state_shapes(self, dtype):
        return {"rec": ((self.heads, self.dim, self.vdim), torch.float32)}

    def forward(self, h, cache: PagedStateCache, stream, states):
        b = cache.batch
        n0, n_l, nq, nv = self.att.n_in, self.att.n_out, self.n_qk, self.n_v
        proj = F.linear(h, self.w_in)
        both = torch.empty(h.shape[0], n_l + nv, dtype=h.dtype, device=h.device)
        self.att.run(proj[:, :n0], cache, stream, out=both[:, :n_l],
                     out_scale=self.left_scale)
        cos, sin = rot_tables(self.rot, cache.max_seq, h.device) \
            if self.rot_dims else (None, None)
        retention_mix(proj[:, n0:n0 + 2 * nq],
                      proj[:, n0 + 2 * nq:n0 + 2 * nq + nv],
                      proj[:, n0 + 2 * nq + nv:], self.head_decay,
                      states["rec"], b, self.heads, self.dim, self.vdim,
                      self.rot_dims, cos, sin, self.eps, self.right_scale,
                      both[:, n_l:])
        return F.linear(both, self.w_o)


class RedudraLayer(nn.Module):
    def __init__(self, cfg: RedudraConfig, spec: dict, dtype):
        super().__init__()
        W, eps, m = cfg.width, cfg.norm_eps, spec["mixer"]
        self.kind = spec["type"]
        self.mult = cfg.residual_mult
        if self.kind == "rglru":
            self.mixer = RGLRUMixer(W, m, eps, dtype)
        elif self.kind == "parallel":
            self.mixer = WindowRetentionMixer(W, m, eps, dtype)
        else:
            raise ValueError(f"unknown mixer type {self.kind!r}")
        self.norm1 = PostNorm(W, eps)
        self.shift = _w(W, dtype=torch.float32)
        mlp = spec.get("mlp")
        self.mlp = self.norm2 = None
        if mlp:
            self.norm2 = PostNorm(W, eps)
            self.mlp = GatedMLP(W, int(mlp["ff"]), "silu", dtype, bias=True)

    def forward(self, x, pending, extra, cache, stream, states, dtype):
        """x: fp32 stream; ``pending``: the result of the sublayer before (not
        yet added) or None; ``extra``: a row added to every token before this
        layer or None. Returns the stream and this layer's own pending
        result."""
        n1, n2 = self.norm1, self.norm2
        x, h = residual_norm(x, pending, self.mult, n1.weight, n1.bias,
                             n1.eps, dtype, extra, self.shift,
                             states["shift"], cache.batch)
        y = self.mixer(h, cache, stream, states)
        if self.mlp is not None:
            x, h = residual_norm(x, y, self.mult, n2.weight, n2.bias, n2.eps,
                                 dtype)
            y = self.mlp(h)
        return x, y


class RedudraForCausalLM(nn.Module):
    architecture = "Redudra"

    def __init__(self, cfg: RedudraConfig, dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        self.dtype = dtype
        W = cfg.width
        self.embed = _w(cfg.vocab_size, W, dtype=dtype)
        self.layers = nn.ModuleList([RedudraLayer(cfg, s, dtype)
                                     for s in cfg.layers])
        self.runs = cfg.layer_runs()
        # cache stream of every layer run that caches rows
        self.stream_of, n = {}, 0
        for r, (i, _) in enumerate(self.runs):
            if self.layers[i].mixer.row_dim:
                self.stream_of[r] = n
                n += 1
        self.loop_step = _w(int(cfg.loop["times"]), W, dtype=torch.float32) \
            if cfg.loop else None
        self.final_norm = PostNorm(W, cfg.norm_eps)
        self.head = _w(cfg.vocab_size, W, dtype=dtype)

    # ------------------------------------------------------------ weights
    def init_random(self, seed=0):
        """Random weights of a useful scale for tests and benchmarks."""
        g = torch.Generator().manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            rnd = torch.randn(p.shape, generator=g)
            if leaf == "weight":
                p.data.copy_(1 + 0.1 * rnd)
            elif leaf == "shift":
                p.data.copy_(0.5 + 0.2 * rnd)
            elif leaf in ("bias", "b_in", "b_gu", "b_down", "conv_b", "b_r",
                          "b_i", "lam", "loop_step"):
                p.data.copy_(0.3 * rnd)
            elif leaf == "conv":
                p.data.copy_(0.4 * rnd)
            elif name == "embed":
                p.data.copy_(0.7 * rnd)
            else:
                p.data.copy_(p.shape[-1] ** -0.5 * rnd)
        return self

    def _named_parts(self):
        """(checkpoint name, parameter rows or columns it fills) for every
        tensor of the model; fused projections appear as slices."""
        yield "embed", self.embed
        if self.loop_step is not None:
            yield "loop.step", self.loop_step
        yield "final.norm", self.final_norm.weight
        yield "final.norm.b", self.final_norm.bias
        yield "head", self.head
        for i, layer in enumerate(self.layers):
            pre, mp = f"l{i}.", f"l{i}.mix."
            a = layer.mixer
            yield pre + "norm1", layer.norm1.weight
            yield pre + "norm1.b", layer.norm1.bias
            yield pre + "shift", layer.shift
            if layer.kind == "rglru":
                C, nb = a.inner, (a.blocks, a.inner // a.blocks)
                yield mp + "y", a.w_in[:C]
                yield mp + "x", a.w_in[C:]
                yield mp + "y.b", a.b_in[:C]
                yield mp + "x.b", a.b_in[C:]
                yield mp + "conv", a.conv
                yield mp + "conv.b", a.conv_b
                yield mp + "ra", a.w_r
                yield mp + "ra.b", a.b_r.view(nb)
                yield mp + "ri", a.w_i
                yield mp + "ri.b", a.b_i.view(nb)
                yield mp + "lam", a.lam
                yield mp + "o", a.w_o
            else:
                t = a.att
                cuts = [("left.q", t.heads * t.dim),
                        ("left.k", t.kv_heads * t.dim),
                        ("left.v", t.kv_heads * t.vdim),
                        ("right.q", a.n_qk), ("right.k", a.n_qk),
                        ("right.v", a.n_v), ("right.g", a.n_v)]
                at = 0
                for n, rows in cuts:
                    yield mp + n, a.w_in[at:at + rows]
                    at += rows
                yield mp + "left.o", a.w_o[:, :t.n_out]
                yield mp + "right.o", a.w_o[:, t.n_out:]
            m = layer.mlp
            if m is None:
                continue
            yield pre + "norm2", layer.norm2.weight
            yield pre + "norm2.b", layer.norm2.bias
            fp, ff = pre + "mlp.", m.w_gu.shape[0] // 2
            yield fp + "gate", m.w_gu[:ff]
            yield fp + "up", m.w_gu[ff:]
            yield fp + "down", m.w_down
            yield fp + "gate.b", m.b_gu[:ff]
            yield fp + "up.b", m.b_gu[ff:]
            yield fp + "down.b", m.b_down

    def load_named_tensors(self, t: dict):
        """Fill the parameters from tensors named as in the checkpoint
        (linear weights [out, in]; 'l<i>.mix.*', 'l<i>.mlp.*', ...)."""
        for name, p in self._named_parts():
            v = t[name]
            if tuple(p.shape) != tuple(v.shape):
                raise ValueError(f"{name}: shape {tuple(v.shape)} != "
                                 f"{tuple(p.shape)}")
            p.data.copy_(v.to(p.dtype))
        return self

    def named_tensors(self):
        """The parameters under their checkpoint names (the inverse of
        ``load_named_tensors``), for writing a model folder."""
        return {n: p.detach().contiguous() for n, p in self._named_parts()}

    # -------------------------------------------------------------- cache
    def build_cache(self, max_slots, max_tokens, dtype=None, device=None,
                    block_size=64, **_):
        """One K/V row stream per attention layer RUN; per request slot and
        layer run the previous normed row (fp32), the recurrences' states
        (fp32) and the convolution tail."""
        dtype = dtype or self.dtype
        device = device or self.embed.device
        dims = [self.layers[self.runs[r][0]].mixer.row_dim
                for r in sorted(self.stream_of, key=self.stream_of.get)]
        states = {}
        for r, (i, _) in enumerate(self.runs):
            states[f"shift{r}"] = ((self.cfg.width,), torch.float32)
            for k, s in self.layers[i].mixer.state_shapes(dtype).items():
                states[f"{k}{r}"] = s
        return PagedStateCache(dims, states, max_slots, max_tokens,
                               block_size=block_size, dtype=dtype,
                               device=device)

    # ------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, input_ids, positions=None, kv_cache=None, rows=None,
                taps=None):
        """input_ids: flat [T] tokens of ``kv_cache.batch``. ``rows`` selects
        the flat positions whose logits are returned (default all; fp32).
        ``taps`` (a list) receives the stream after every layer run."""
        cache = kv_cache
        assert cache is not None and cache.batch is not None, \
            "Redudra runs through a PagedStateCache step"
        ids = input_ids.reshape(-1)
        dt, cfg = self.dtype, self.cfg
        x, y = embed_rows(self.embed, ids, 1.0), None
        for r, (i, opens) in enumerate(self.runs):
            states = {k: cache.states[f"{k}{r}"]
                      for k in ("shift", "conv", "rec")
                      if f"{k}{r}" in cache.states}
            extra = None if opens is None else self.loop_step[opens]
            x, y = self.layers[i](x, y, extra, cache, self.stream_of.get(r),
                                  states, dt)
            if taps is not None:
                taps.append(x + cfg.residual_mult * y.float())
        n = self.final_norm
        if rows is None:
            _, h = residual_norm(x, y, cfg.residual_mult, n.weight, n.bias,
                                 n.eps, dt)
        else:
            _, h = residual_norm(x, y, cfg.residual_mult, n.weight, n.bias,
                                 n.eps, dt, index=rows)
        logits = F.linear(h, self.head)
        return softcap_rows(logits, cfg.logit_softcap) \
            if cfg.logit_softcap > 0 else logits

    def num_parameters(self):
        return sum(p.numel() for p in self.parameters())


def build_from_config(cfg: dict, dtype):
    return RedudraForCausalLM(RedudraConfig.from_dict(cfg), dtype)


def redudra_tiny(dtype=torch.float32):
    """A small configuration for tests: both mixer kinds, a layer without
    feed-forward, a looped block."""
    rg = {"width": 12, "blocks": 3, "conv": 3}
    par = {"left": {"heads": 4, "kv_heads": 2, "dim": 10, "vdim": 6,
                    "scale": 0.4, "mask": {"size": 9, "keep_first": 2},
                    "rot": {"base": 100.0, "dims": 8,
                            "scaling": {"factor": 3.0, "original": 24,
                                        "fast": 4.0, "slow": 1.0}}},
           "right": {"heads": 3, "dim": 8, "vdim": 5,
                     "rot": {"base": 50.0, "dims": 6},
                     "decay": [0.7, 0.9, 0.99]},
           "left_scale": 0.8, "right_scale": 1.3}
    ff = {"kind": "dense", "ff": 40}
    cfg = RedudraConfig(
        vocab_size=61, width=24, norm_eps=1e-5, residual_mult=0.7,
        logit_softcap=6.0, loop={"start": 1, "stop": 3, "times": 2},
        layers=[{"type": "parallel", "mixer": par, "mlp": ff},
                {"type": "rglru", "mixer": rg, "mlp": ff},
                {"type": "parallel", "mixer": par, "mlp": None},
                {"type": "rglru", "mixer": rg, "mlp": ff}])
    return RedudraForCausalLM(cfg, dtype)
