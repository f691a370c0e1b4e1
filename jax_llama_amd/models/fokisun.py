"""Fokisun: a layer-list decoder whose layers run mixer and feed-forward side by side on one statistics-free norm, and
read a weighted sum of every earlier layer's result.

Per layer (``models/mixers.DepthAverageBlock``): ``h = tanh(alpha x) w + b``, ``X_(i+1) = x + m (mixer(h) + ff(h))``, and the
next layer's ``x`` is ``sum_{j <= i+1} dwa_i[j] X_j`` with ``X_0`` the embedding. Mixers: ``attention``
(``WholeNormAttention``: biases, q / k norms over the whole projections, interleaved rotary positions, a sliding window,
one added to the softmax denominator, values mixed with the first value-mixing layer's, a gate per output column),
``latent_attention`` (``RotaryLatentAttention`` with the "halves" rotation, no window, a gate per head) and ``hgrn2``
(``GatedRunningMixer``: a forget gate that also decides what is written). Feed-forward: none, dense (gated gelu), or a
mixture of gated silu experts behind a grouped sigmoid router plus a shared expert. The embedding table is the output
matrix too.

Checkpoint: ``config.json`` + ``model.safetensors`` with tensors ``embed``, ``l<i>.norm1``, ``l<i>.norm1.alpha|b``,
``l<i>.dwa``, ``l<i>.mix.q|k|v|o`` with ``.b`` each, ``l<i>.mix.q.norm|k.norm|g|vmix`` (attention),
``l<i>.mix.dq|dq.norm|uq|dkv|dkv.norm|uk|uv|g|o`` (latent attention), ``l<i>.mix.q|f|f.b|lower|v|norm|o`` (hgrn2),
``l<i>.mlp.gate|up|down`` (dense) or ``l<i>.mlp.router``, ``l<i>.mlp.e<j>.gate|up|down``, ``l<i>.mlp.shared.gate|up|down``,
``final.norm``, ``final.norm.alpha|b`` (linear weights ``[out, in]``). Loading fuses a mixer's input projections, its gate
rows and the router into one matrix, the mixer's and the dense side's output matrices into another, stacks the experts,
folds the logit scale into the final norm's gain and offset, and keeps norms, biases, gates' constants, the depth weights
and the rotary frequencies (float64) out of bf16 in both formats.
"""
from __future__ import annotations

from typing import Dict

import torch

from ..config import DenseFFSpec, FokisunConfig, GatedRunningSpec, RotaryLatentSpec, WholeNormAttentionSpec
from ..ops import hybrid as hy
from .layer_list import LayerListLM
from .mixers import DepthAverageBlock, GatedMoE, GatedRunningMixer, RotaryLatentAttention, WholeNormAttention

BF16 = torch.bfloat16
F32 = torch.float32


def cache_specs(config: FokisunConfig) -> list:
    specs = []
    for ls in config.layers:
        m = ls.mixer
        if isinstance(m, RotaryLatentSpec):
            specs.append(("latent", m.kv_rank + m.rot_dim))
        elif isinstance(m, GatedRunningSpec):
            specs.append(("linear", m.heads, m.dim, m.vdim))
        else:
            specs.append(("kv", m.kv_heads, m.dim, m.vdim))
    return specs


def random_state_dict(config: FokisunConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """A random checkpoint of ``config`` with the checkpoint's tensor names (bf16): synthetic benchmarks and tests.
    Scales keep every sublayer's output O(1), the forget gates spread over (0, 1) and the depth weights summing near 1."""
    g = torch.Generator().manual_seed(seed)
    d = config.hidden_size

    def mat(n, k, std=None):
        return (torch.randn(n, k, generator=g) * (std if std is not None else k ** -0.5)).to(BF16)

    def vec(n, lo, hi):
        return (torch.rand(n, generator=g) * (hi - lo) + lo).to(BF16)

    sd: Dict[str, torch.Tensor] = {"embed": mat(config.vocab_size, d, 1.0)}

    def norm(name):
        sd[name], sd[name + ".b"] = vec(d, 0.7, 1.3), vec(d, -0.1, 0.1)
        sd[name + ".alpha"] = vec(1, 0.4, 0.8).reshape(())

    norm("final.norm")
    for i, ls in enumerate(config.layers):
        p, m, f = f"l{i}.", ls.mixer, ls.mlp
        x = p + "mix."
        norm(p + "norm1")
        dwa = torch.randn(i + 2, generator=g) * 0.1
        dwa[-1] += 1.0
        sd[p + "dwa"] = dwa.to(BF16)
        if isinstance(m, RotaryLatentSpec):
            sd[x + "dq"], sd[x + "dq.norm"] = mat(m.q_rank, d), vec(m.q_rank, 0.7, 1.3)
            sd[x + "uq"] = mat(m.heads * (m.dim + m.rot_dim), m.q_rank)
            sd[x + "dkv"], sd[x + "dkv.norm"] = mat(m.kv_rank + m.rot_dim, d), vec(m.kv_rank, 0.7, 1.3)
            sd[x + "uk"], sd[x + "uv"] = mat(m.heads * m.dim, m.kv_rank), mat(m.heads * m.vdim, m.kv_rank)
            sd[x + "g"] = mat(m.heads, d)
        elif isinstance(m, GatedRunningSpec):
            sd[x + "q"], sd[x + "f"], sd[x + "v"] = mat(m.heads * m.dim, d), mat(m.heads * m.dim, d), mat(m.heads * m.vdim, d)
            sd[x + "f.b"], sd[x + "lower"] = vec(m.heads * m.dim, -1.0, 3.0), vec(m.heads * m.dim, 0.0, 0.9)
            sd[x + "norm"] = vec(m.vdim, 0.7, 1.3)
        else:
            for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
                sd[x + n], sd[x + n + ".b"] = mat(rows, d), vec(rows, -0.3, 0.3)
            sd[x + "q.norm"], sd[x + "k.norm"] = vec(m.heads * m.dim, 0.7, 1.3), vec(m.kv_heads * m.dim, 0.7, 1.3)
            sd[x + "g"] = mat(m.heads * m.vdim, d)
            sd[x + "o.b"] = vec(d, -0.2, 0.2)
            if m.v_mix:
                sd[x + "vmix"] = vec(1, 0.2, 0.8).reshape(())
        sd[x + "o"] = mat(d, m.heads * m.vdim)

        def ff(pre, width):
            sd[pre + "gate"], sd[pre + "up"], sd[pre + "down"] = mat(width, d), mat(width, d), mat(d, width)

        if isinstance(f, DenseFFSpec):
            ff(p + "mlp.", f.ff)
        elif f is not None:
            sd[p + "mlp.router"] = mat(f.experts, d, 2.0 * d ** -0.5)
            for e in range(f.experts):
                ff(p + f"mlp.e{e}.", f.ff)
            if f.shared_ff:
                ff(p + "mlp.shared.", f.shared_ff)
    return sd


class FokisunForCausalLM(LayerListLM):
    """Fokisun on the layer-list step function (``models/layer_list.py``)."""

    config_class = FokisunConfig
    family = "Fokisun"
    random_state_dict = staticmethod(random_state_dict)

    def cache_specs(self) -> list:
        return cache_specs(self.config)

    def load_state_dict(self, sd: Dict[str, torch.Tensor]) -> "FokisunForCausalLM":
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

        def norm(name, gain=1.0):
            return hy.SquashNorm(f32(sd[name + ".alpha"].reshape(1)), f32(get(name, d)) * gain, f32(get(name + ".b", d)) * gain)

        self.embed = self.head = mat(get("embed", c.vocab_size, d))
        self.final_norm = norm("final.norm", c.logit_scale)
        self.depth_history = True
        self.blocks = []
        leader = False  # a value-mixing layer has been seen
        for i, ls in enumerate(c.layers):
            p, m, f = f"l{i}.", ls.mixer, ls.mlp
            x = p + "mix."
            w_o = mat(get(x + "o", d, m.heads * m.vdim))
            if isinstance(m, RotaryLatentSpec):
                w_uk = get(x + "uk", m.heads * m.dim, m.kv_rank).reshape(m.heads, m.dim, m.kv_rank).to(dev, wdt)
                w_uv = get(x + "uv", m.heads * m.vdim, m.kv_rank).reshape(m.heads, m.vdim, m.kv_rank).to(dev, wdt).contiguous()
                w_in = mat(get(x + "dq", m.q_rank, d), get(x + "dkv", m.kv_rank + m.rot_dim, d), get(x + "g", m.heads, d))
                mixer = RotaryLatentAttention(i, m, eps, w_in, f32(get(x + "dq.norm", m.q_rank)),
                                              mat(get(x + "uq", m.heads * (m.dim + m.rot_dim), m.q_rank)),
                                              f32(get(x + "dkv.norm", m.kv_rank)), w_uk, w_uv,
                                              hy.rotary_freqs(m.rot_base, m.rot_dims, dev) if m.rot_dims else None, w_o,
                                              interleaved=False)
            elif isinstance(m, GatedRunningSpec):
                hd = m.heads * m.dim
                mixer = GatedRunningMixer(i, m, eps, mat(get(x + "q", hd, d), get(x + "f", hd, d),
                                                         get(x + "v", m.heads * m.vdim, d)),
                                          f32(get(x + "f.b", hd)), f32(sd[x + "lower"].reshape(hd)),
                                          f32(get(x + "norm", m.vdim)), w_o)
            elif isinstance(m, WholeNormAttentionSpec):
                rows = dict(q=m.heads * m.dim, k=m.kv_heads * m.dim, v=m.kv_heads * m.vdim)
                freq = hy.rotary_freqs(m.rot_base, m.rot_dims, dev) / m.rot_factor if m.rot_dims else None
                mixer = WholeNormAttention(
                    i, m, eps, mat(*(get(x + n, r, d) for n, r in rows.items()), get(x + "g", m.heads * m.vdim, d)),
                    f32(*(get(x + n + ".b", r) for n, r in rows.items())), f32(get(x + "q.norm", rows["q"])),
                    f32(get(x + "k.norm", rows["k"])), freq, torch.zeros(m.heads, dtype=F32, device=dev),
                    m.v_mix and not leader, f32(sd[x + "vmix"].reshape(1)) if m.v_mix and leader else None, w_o,
                    f32(get(x + "o.b", d)))
                leader = leader or m.v_mix
            else:
                raise ValueError(f"layer {i}: unknown mixer {m!r}")

            def gate_up(pre, width):
                return mat(get(pre + "gate", width, d), get(pre + "up", width, d))

            moe = side_gu = side_down = None
            act = hy.ACT_SWIGLU
            if isinstance(f, DenseFFSpec):
                side_gu, side_down, act = gate_up(p + "mlp.", f.ff), mat(get(p + "mlp.down", d, f.ff)), hy.ACT_GELU_GLU
            elif f is not None:
                w_gu = torch.stack([gate_up(p + f"mlp.e{e}.", f.ff) for e in range(f.experts)])
                w_down = torch.stack([mat(get(p + f"mlp.e{e}.down", d, f.ff)) for e in range(f.experts)])
                rule = hy.RouterRule(sigmoid=True, group_top=2, normalise=True, scale=f.scale)
                moe = GatedMoE(f.experts, f.top, f.groups, f.keep_groups, rule, mat(get(p + "mlp.router", f.experts, d)), w_gu,
                               w_down)
                if f.shared_ff:
                    side_gu = gate_up(p + "mlp.shared.", f.shared_ff)
                    side_down = mat(get(p + "mlp.shared.down", d, f.shared_ff))
            self.blocks.append(DepthAverageBlock(i, mixer, moe, side_gu, side_down, act, norm(p + "norm1"),
                                                 f32(get(p + "dwa", i + 2)), c.residual_mult))
        for blk, nxt in zip(self.blocks, self.blocks[1:] + [None]):
            blk.next_norm = nxt.norm if nxt is not None else self.final_norm
            blk.last = nxt is None
        return self
