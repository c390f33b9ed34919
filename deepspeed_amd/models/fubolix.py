"""Fubolix: a decoder-only serving model with parallel layers without any norm
statistic over three kinds of grouped-query attention, assembled from the
framework's ragged-batch mechanisms.

* a layer reads the fp32 stream once, through a dynamic tanh ``h = tanh(alpha *
  x) * w + b`` (ops/norms.py ``residual_tanh``, which also adds the layer
  before), and both sublayers read that row: ``x += mixer(h) + ff(h)``. Their
  first products are therefore ONE matrix (``q | k | v | up | gate``), and as
  both results are only summed, their last products are ONE matrix too
  (``[W_o | W_down]`` over ``[heads ; activated up]``);
* mixer ``attention``: the projected keys are the values; interleaved partial
  rotary with YaRN frequencies, then queries and keys at unit RMS per head; a
  sliding window that keeps the first tokens; one added to the softmax's
  denominator; a sigmoid gate per head;
* mixer ``attention_2``: weighted query/key norms per head, no rotation, queries
  scaled by a factor that grows with the logarithm of the position, causal, one
  added to the denominator;
* mixer ``attention_3``: short causal convolutions over the projected queries,
  keys and values (their tails are carried per request slot), rotate-half
  partial rotary with YaRN frequencies, causal, a learned sink per head;
* feed-forward: dense, the square of relu.

All three mixers are ``GroupedAttention`` (models/savovik.py) with different
flags. The model runs only through a ``PagedStateCache`` step: ``forward``
takes the flat token list of a ragged batch. Every size and constant comes
from the config.
"""

from dataclasses import dataclass
from typing import List

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..inference.state_cache import PagedStateCache
from ..ops.norms import embed_rows, residual_tanh
from .savovik import GroupedAttention

# what each mixer kind asks of GroupedAttention
MIXERS = {
    "attention": dict(v_from_k=True, layout="interleaved", qk_norm="after",
                      mask="window", sink="one", gate=True),
    "attention_2": dict(qk_norm="head", q_temp=True, sink="one"),
    "attention_3": dict(conv=True, layout="half", sink="learned"),
}


@dataclass
class FubolixConfig:
    vocab_size: int
    width: int
    layers: List[dict]
    norm_eps: float = 1e-6
    embed_scale: float = 1.0
    max_seq_len: int = 1 << 16

    @classmethod
    def from_dict(cls, d: dict) -> "FubolixConfig":
        cfg = cls(vocab_size=int(d["vocab"]), width=int(d["width"]),
                  layers=list(d["layers"]), norm_eps=float(d["norm"]["eps"]),
                  embed_scale=float((d.get("embedding") or {})
                                    .get("scale", 1.0)))
        cfg.validate()
        return cfg

    def to_dict(self) -> dict:
        return {"architecture": "Fubolix", "vocab": self.vocab_size,
                "width": self.width, "layers": self.layers,
                "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embed_scale}}

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def validate(self):
        for i, spec in enumerate(self.layers):
            if spec["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {spec['type']!r}")
            m = spec["mixer"]
            if spec["type"] == "attention_2" and m.get("rot"):
                raise ValueError(f"layer {i}: attention_2 has no rotation")
            if spec["type"] != "attention" and m.get("mask"):
                raise ValueError(f"layer {i}: {spec['type']} has no window")
            mlp = spec.get("mlp")
            if mlp and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown mlp kind "
                                 f"{mlp['kind']!r}")


def _w(*shape, dtype):
    return nn.Parameter(torch.empty(*shape, dtype=dtype), requires_grad=False)


class DynamicTanh(nn.Module):
    """Weights of ``tanh(alpha * x) * weight + bias``."""

    def __init__(self, width):
        super().__init__()
        self.alpha = _w(1, dtype=torch.float32)
        self.weight = _w(width, dtype=torch.float32)
        self.bias = _w(width, dtype=torch.float32)

    def forward(self, x, pending, dtype, index=None):
        """Adds ``pending`` to the stream (in place without ``index``) and
        returns the new rows' dynamic tanh."""
        return residual_tanh(x, pending, self.alpha, self.weight, self.bias,
                             dtype, index)


class FubolixLayer(nn.Module):
    """``w_in`` = rows of q | k | v | up | gate (zero rows up to a multiple of
    8); ``w_out`` = columns of the output projection | the down projection."""

    def __init__(self, cfg: FubolixConfig, spec: dict, dtype):
        super().__init__()
        self.kind = spec["type"]
        self.att = GroupedAttention(spec["mixer"], cfg.norm_eps, dtype,
                                    **MIXERS[self.kind])
        self.norm1 = DynamicTanh(cfg.width)
        self.ff = int(spec["mlp"]["ff"]) if spec.get("mlp") else 0
        a = self.att
        self.g_col = a.n_in + self.ff
        rows = self.g_col + (a.heads if a.has_gate else 0)
        self.w_in = _w((rows + 7) // 8 * 8, cfg.width, dtype=dtype)
        self.w_in.data[rows:] = 0
        self.rows = rows
        self.w_out = _w(cfg.width, a.n_out + self.ff, dtype=dtype)

    def forward(self, h, cache: PagedStateCache, stream, states):
        """h: the layer's input row after its norm. Returns the sum of both
        sublayers' results."""
        a = self.att
        proj = F.linear(h, self.w_in)
        both = torch.empty(h.shape[0], a.n_out + self.ff, dtype=h.dtype,
                           device=h.device)
        gate = proj[:, self.g_col:self.g_col + a.heads] if a.has_gate else None
        side = (proj[:, a.n_in:self.g_col], both[:, a.n_out:], "relu2") \
            if self.ff else None
        a.run(proj[:, :a.n_in], cache, stream, out=both[:, :a.n_out],
              states=states, gate=gate, side=side)
        return F.linear(both, self.w_out)


class FubolixForCausalLM(nn.Module):
    architecture = "Fubolix"

    def __init__(self, cfg: FubolixConfig, dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        self.dtype = dtype
        W = cfg.width
        self.embed = _w(cfg.vocab_size, W, dtype=dtype)
        self.layers = nn.ModuleList([FubolixLayer(cfg, s, dtype)
                                     for s in cfg.layers])
        self.final_norm = DynamicTanh(W)
        self.head = _w(cfg.vocab_size, W, dtype=dtype)

    # ------------------------------------------------------------ weights
    def init_random(self, seed=0):
        """Random weights of a useful scale for tests and benchmarks."""
        g = torch.Generator().manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            rnd = torch.randn(p.shape, generator=g)
            if leaf in ("weight", "q_norm", "k_norm"):
                p.data.copy_(1 + 0.1 * rnd)
            elif leaf == "alpha":
                p.data.copy_(0.5 + 0.05 * rnd)
            elif leaf in ("bias", "sink"):
                p.data.copy_(0.3 * rnd)
            elif leaf == "conv":
                p.data.copy_(0.4 * rnd)
            elif name == "embed":
                p.data.copy_(0.7 * rnd)
            else:
                p.data.copy_(p.shape[-1] ** -0.5 * rnd)
        for layer in self.layers:
            layer.w_in.data[layer.rows:] = 0
        return self

    def _named_parts(self):
        """(checkpoint name, parameter rows or columns it fills) for every
        tensor of the model; fused projections appear as slices."""
        def norm(pre, n):
            yield pre, n.weight
            yield pre + ".b", n.bias
            yield pre + ".alpha", n.alpha.view(())

        yield "embed", self.embed
        yield from norm("final.norm", self.final_norm)
        yield "head", self.head
        for i, layer in enumerate(self.layers):
            pre, mp, a = f"l{i}.", f"l{i}.mix.", layer.att
            yield from norm(pre + "norm1", layer.norm1)
            cuts = [("q", a.heads * a.dim), ("k", a.kv_heads * a.dim)]
            if not a.v_from_k:
                cuts.append(("v", a.kv_heads * a.vdim))
            at = 0
            for n, rows in cuts:
                yield mp + n, layer.w_in[at:at + rows]
                if a.taps:
                    yield mp + n + ".conv", a.conv[at:at + rows]
                at += rows
            if a.has_gate:
                yield mp + "g", layer.w_in[layer.g_col:layer.rows]
            if a.norm == "head":
                yield mp + "q.norm", a.q_norm
                yield mp + "k.norm", a.k_norm
            if isinstance(a.sink, nn.Parameter):
                yield mp + "sink", a.sink
            yield mp + "o", layer.w_out[:, :a.n_out]
            if layer.ff:
                yield pre + "mlp.up", layer.w_in[a.n_in:layer.g_col]
                yield pre + "mlp.down", layer.w_out[:, a.n_out:]

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
        """One K/V row stream per layer; per request slot the convolutions'
        tails."""
        dtype = dtype or self.dtype
        device = device or self.embed.device
        states = {f"{k}{i}": s for i, layer in enumerate(self.layers)
                  for k, s in layer.att.state_shapes(dtype).items()}
        return PagedStateCache([layer.att.row_dim for layer in self.layers],
                               states, max_slots, max_tokens,
                               block_size=block_size, dtype=dtype,
                               device=device)

    # ------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, input_ids, positions=None, kv_cache=None, rows=None,
                taps=None):
        """input_ids: flat [T] tokens of ``kv_cache.batch``. ``rows`` selects
        the flat positions whose logits are returned (default all).
        ``taps`` (a list) receives the stream after every layer."""
        cache = kv_cache
        assert cache is not None and cache.batch is not None, \
            "Fubolix runs through a PagedStateCache step"
        ids = input_ids.reshape(-1)
        dt = self.dtype
        x, y = embed_rows(self.embed, ids, self.cfg.embed_scale), None
        for i, layer in enumerate(self.layers):
            states = {"conv": cache.states[f"conv{i}"]} \
                if layer.att.taps else None
            h = layer.norm1(x, y, dt)
            y = layer(h, cache, i, states)
            if taps is not None:
                taps.append(x + y.float())
        return F.linear(self.final_norm(x, y, dt, rows), self.head)

    def num_parameters(self):
        return sum(p.numel() for p in self.parameters())


def build_from_config(cfg: dict, dtype):
    return FubolixForCausalLM(FubolixConfig.from_dict(cfg), dtype)


def fubolix_tiny(dtype=torch.float32):
    """A small configuration for tests: every mixer kind, a layer without
    feed-forward."""
    yarn = {"factor": 3.0, "original": 24, "fast": 4.0, "slow": 1.0}
    win = {"heads": 4, "kv_heads": 2, "dim": 10, "vdim": 10, "scale": 0.4,
           "mask": {"size": 9, "keep_first": 2},
           "rot": {"base": 100.0, "dims": 8, "scaling": yarn}}
    temp = {"heads": 3, "kv_heads": 1, "dim": 8, "vdim": 6, "scale": 0.5,
            "q_temp": {"coef": 0.7, "every": 5}}
    conv = {"heads": 2, "kv_heads": 2, "dim": 12, "vdim": 6, "scale": 0.3,
            "conv": 3, "rot": {"base": 50.0, "dims": 6, "scaling": yarn}}
    ff = {"kind": "dense", "ff": 40}
    cfg = FubolixConfig(
        vocab_size=61, width=24, norm_eps=1e-5, embed_scale=1.7,
        layers=[{"type": "attention", "mixer": win, "mlp": ff},
                {"type": "attention_3", "mixer": conv, "mlp": ff},
                {"type": "attention_2", "mixer": temp, "mlp": None},
                {"type": "attention", "mixer": win, "mlp": ff}])
    return FubolixForCausalLM(cfg, dtype)
