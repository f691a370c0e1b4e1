"""Zopupel: a layer-list decoder with an RMS norm on both sides of every sublayer and two kinds of attention.

Per layer (``models/mixers.SandwichChainBlock``): ``x += m n1b(mixer(n1(x)))``, ``x += m n2b(ff(n2(x)))``. Mixers:
``attention`` (``DifferentialAttention``: two softmax maps per head over the same values, their weighted difference normed per
head; a layer may read another layer's keys and values) and ``attention_2`` (``WholeNormAttention``: biases, q / k norms over
the whole projections, values that are the keys as projected, one added to the softmax denominator), both with rotary
positions in the "halves" layout, the first with linearly scaled frequencies, the second with YaRN scaling. Feed-forward:
none, or a mixture of gated silu experts behind a biased softmax router plus a shared expert.

Checkpoint: ``config.json`` + ``model.safetensors`` with tensors ``embed``, ``l<i>.norm1|norm1b|norm2|norm2b``,
``l<i>.mix.q|k|v|o``, ``l<i>.mix.lq1|lk1|lq2|lk2`` (attention; without ``k`` and ``v`` in a layer with ``kv_from``),
``l<i>.mix.q|k|o`` with ``.b`` each and ``l<i>.mix.q.norm|k.norm`` (attention_2), ``l<i>.mlp.router|router.b``,
``l<i>.mlp.e<j>.gate|up|down``, ``l<i>.mlp.shared.gate|up|down``, ``final.norm``, ``head`` (linear weights ``[out, in]``).
Loading fuses a mixer's input projections into one matrix and the shared expert's gate / up rows with the router's into
another, stacks the experts, folds the residual factor into the output norms' gains, computes a differential layer's weight of
the second map, and keeps norms, biases and the rotary frequencies (float64) out of bf16 in both formats.
"""
from __future__ import annotations

import math
from typing import Dict

import torch

from ..config import DifferentialAttentionSpec, KeyValueAttentionSpec, ZopupelConfig
from .layer_list import LayerListLM
from .mixers import DifferentialAttention, SandwichChainBlock, SharedExpertMoE, WholeNormAttention

BF16 = torch.bfloat16
F32 = torch.float32


def cache_specs(config: ZopupelConfig) -> list:
    specs = []
    for ls in config.layers:
        m = ls.mixer
        if isinstance(m, KeyValueAttentionSpec):
            specs.append(("kv", m.kv_heads, m.dim, m.vdim))
        elif m.kv_from is not None:
            specs.append(("kv_from", m.kv_from))
        else:
            specs.append(("kv", m.kv_heads, 2 * m.dim, m.vdim))  # (a key row: both maps side by side)
    return specs


def random_state_dict(config: ZopupelConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """A random checkpoint of ``config`` with the checkpoint's tensor names (bf16): synthetic benchmarks and tests."""
    g = torch.Generator().manual_seed(seed)
    d = config.hidden_size

    def mat(n, k, std=None):
        return (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(BF16)

    def vec(n, lo, hi):
        return (torch.rand(n, generator=g) * (hi - lo) + lo).to(BF16)

    sd: Dict[str, torch.Tensor] = {"embed": mat(config.vocab_size, d, 1.0), "head": mat(config.vocab_size, d),
                                   "final.norm": vec(d, 0.7, 1.3)}
    for i, ls in enumerate(config.layers):
        p, m, f = f"l{i}.", ls.mixer, ls.mlp
        x = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
            sd[p + n] = vec(d, 0.7, 1.3)
        if isinstance(m, DifferentialAttentionSpec):
            sd[x + "q"] = mat(m.heads * 2 * m.dim, d)
            if m.kv_from is None:
                sd[x + "k"], sd[x + "v"] = mat(m.kv_heads * 2 * m.dim, d), mat(m.kv_heads * m.vdim, d)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                sd[x + n] = (torch.randn(m.dim, generator=g) * 0.3 * m.dim ** -0.25).to(BF16)
        else:
            for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim)):
                sd[x + n], sd[x + n + ".b"] = mat(rows, d), vec(rows, -0.3, 0.3)
                sd[x + n + ".norm"] = vec(rows, 0.7, 1.3)
            sd[x + "o.b"] = vec(d, -0.2, 0.2)
        sd[x + "o"] = mat(d, m.heads * m.vdim)

        def ff(pre, width):
            sd[pre + "gate"], sd[pre + "up"], sd[pre + "down"] = mat(width, d), mat(width, d), mat(d, width)

        if f is not None:
            sd[p + "mlp.router"], sd[p + "mlp.router.b"] = mat(f.experts, d, 2.0 * d ** -0.5), vec(f.experts, -1.0, 1.0)
            for e in range(f.experts):
                ff(p + f"mlp.e{e}.", f.ff)
            if f.shared_ff:
                ff(p + "mlp.shared.", f.shared_ff)
    return sd


class ZopupelForCausalLM(LayerListLM):
    """Zopupel on the layer-list step function (``models/layer_list.py``)."""

    config_class = ZopupelConfig
    family = "Zopupel"
    random_state_dict = staticmethod(random_state_dict)

    def cache_specs(self) -> list:
        return cache_specs(self.config)

    def load_state_dict(self, sd: Dict[str, torch.Tensor]) -> "ZopupelForCausalLM":
        c, dev, wdt, eps = self.config, self.device, self.param_dtype, self.eps
        d = c.hidden_size

        def get(name, *shape):
            if tuple(sd[name].shape) != shape:
                raise ValueError(f"{name}: shape {tuple(sd[name].shape)}, the configuration says {shape}")
            return sd[name]

        def mat(*tensors):  # one matrix, or several stacked along the rows
            t = torch.cat(tensors, 0) if len(tensors) > 1 else tensors[0]
            return t.to(dev, wdt).contiguous()

        def f32(*tensors):
            return torch.cat([t.reshape(-1) for t in tensors]).to(dev, F32).contiguous()

        self.embed, self.head = mat(get("embed", c.vocab_size, d)), mat(get("head", c.vocab_size, d))
        self.final_norm = f32(get("final.norm", d))
        self.chained_norms = True
        self.blocks = []
        for i, ls in enumerate(c.layers):
            p, m, f = f"l{i}.", ls.mixer, ls.mlp
            x = p + "mix."
            w_o = mat(get(x + "o", d, m.heads * m.vdim))
            freq, rot_gain = m.rot.freqs(dev) if m.rot is not None else (None, 1.0)
            if isinstance(m, DifferentialAttentionSpec):
                own = m.kv_from is None
                rows = dict(q=m.heads * 2 * m.dim, **(dict(k=m.kv_heads * 2 * m.dim, v=m.kv_heads * m.vdim) if own else {}))
                lq1, lk1, lq2, lk2 = (get(x + n, m.dim).double() for n in ("lq1", "lk1", "lq2", "lk2"))
                lam = math.exp(float(lq1 @ lk1)) - math.exp(float(lq2 @ lk2)) + m.diff
                mixer = DifferentialAttention(i, m, eps, mat(*(get(x + n, r, d) for n, r in rows.items())), freq, lam,
                                              1.0 - m.diff, w_o, own, rot_gain)
            else:
                rows = dict(q=m.heads * m.dim, k=m.kv_heads * m.dim)
                mixer = WholeNormAttention(
                    i, m, eps, mat(*(get(x + n, r, d) for n, r in rows.items())),
                    f32(*(get(x + n + ".b", r) for n, r in rows.items())), f32(get(x + "q.norm", rows["q"])),
                    f32(get(x + "k.norm", rows["k"])), freq, torch.zeros(m.heads, dtype=F32, device=dev), False, None, w_o,
                    f32(get(x + "o.b", d)), gated=False, interleaved=False, v_is_k=True, rot_gain=rot_gain)

            def gate_up(pre, width):
                return mat(get(pre + "gate", width, d), get(pre + "up", width, d))

            mlp = pre2 = post2 = None
            if f is not None:
                w_gu = torch.stack([gate_up(p + f"mlp.e{e}.", f.ff) for e in range(f.experts)])
                w_down = torch.stack([mat(get(p + f"mlp.e{e}.down", d, f.ff)) for e in range(f.experts)])
                shared = (gate_up(p + "mlp.shared.", f.shared_ff), mat(get(p + "mlp.shared.down", d, f.shared_ff))) \
                    if f.shared_ff else ()
                mlp = SharedExpertMoE(f.experts, f.top, mat(get(p + "mlp.router", f.experts, d)),
                                      f32(get(p + "mlp.router.b", f.experts)), w_gu, w_down, *shared)
                pre2, post2 = f32(get(p + "norm2", d)), f32(get(p + "norm2b", d)) * c.residual_mult
            self.blocks.append(SandwichChainBlock(mixer, f32(get(p + "norm1b", d)) * c.residual_mult, mlp, pre2, post2,
                                                  f32(get(p + "norm1", d)), eps))
        for blk, nxt in zip(self.blocks, self.blocks[1:] + [None]):
            blk.next_norm = nxt.pre1 if nxt is not None else self.final_norm
            blk.last = nxt is None
        return self
