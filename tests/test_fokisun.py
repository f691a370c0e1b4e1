"""Fokisun through the framework (model, cache, stepper, engine) against the plain float64 oracle
(tests/oracle_fokisun.py), on the CPU op path and, marked gpu, on the HIP kernels. Small configurations built here: sizes
that are multiples of nothing, every mixer first / last / repeated, layers without a feed-forward, without a window, without
rotation or frequency scaling, without value mixing, routers with and without groups and shared experts, top-1 routing,
one layer only."""
import numpy as np
import pytest
import torch

import oracle_fokisun as of
from jax_llama_amd.config import (DenseFFSpec, FokisunConfig, GatedMoESpec, GatedRunningSpec, RotaryLatentSpec,
                                  WholeNormAttentionSpec)
from jax_llama_amd.models.fokisun import FokisunForCausalLM, random_state_dict
from jax_llama_amd.models.kv_cache import HybridCache
from jax_llama_amd.models.mixers import (GatedMoE, GatedRunningMixer, RotaryLatentAttention, StepContext,
                                         WholeNormAttention)
from jax_llama_amd.ops import hybrid as hy
from jax_llama_amd.runtime.engine import GenerationConfig
from jax_llama_amd.runtime.stepper import SequenceStepper

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32, BF16 = torch.float32, torch.bfloat16


def _att(heads, kv_heads, dim, vdim, scale, window=None, rot_dims=None, base=10000.0, factor=None, v_mix=True):
    out = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, v_mix=v_mix)
    if window:
        out["mask"] = {"size": window}
    if rot_dims:
        out["rot"] = {"base": base, "dims": rot_dims}
        if factor:
            out["rot"]["scaling"] = {"factor": factor}
    return out


def _lat(heads, dim, rot_dim, vdim, rank, q_rank, scale, base=10000.0):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=rank, q_rank=q_rank, scale=scale,
                rot={"base": base, "dims": rot_dim})


def _rec(heads, dim, vdim):
    return dict(heads=heads, dim=dim, vdim=vdim)


def _moe(experts, top, ff, groups=None, scale=1.0, shared=0):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def cfg_full():
    """Every mixer twice, a recurrent layer first, value mixing with a layer that does not take part between."""
    return {"architecture": "Fokisun", "vocab": 67, "width": 40, "norm": {"eps": 1e-5}, "residual_mult": 0.7,
            "logit_scale": 0.3,
            "layers": [
                {"type": "hgrn2", "mixer": _rec(3, 12, 20), "mlp": _moe(6, 2, 24, (3, 2), 2.5, 40)},
                {"type": "attention", "mixer": _att(4, 2, 12, 20, 0.3, 13, 8, 500.0, 3.0), "mlp": {"kind": "dense", "ff": 52}},
                {"type": "latent_attention", "mixer": _lat(3, 16, 8, 24, 20, 28, 0.2), "mlp": _moe(5, 3, 16, None, 0.6)},
                {"type": "attention", "mixer": _att(6, 3, 8, 8, 0.5, 5, v_mix=False), "mlp": None},
                {"type": "attention", "mixer": _att(2, 2, 16, 20, 0.25, None, 16), "mlp": _moe(8, 3, 8, (2, 1), 1.3, 24)},
                {"type": "hgrn2", "mixer": _rec(2, 24, 8), "mlp": None},
                {"type": "latent_attention", "mixer": _lat(2, 8, 12, 8, 36, 16, 0.25, 300.0), "mlp": {"kind": "dense", "ff": 8}},
            ]}


def cfg_bare():
    """One layer of one head, no window, no rotation, no value mixing to do, one expert."""
    return {"architecture": "Fokisun", "vocab": 37, "width": 24, "norm": {"eps": 1e-6}, "residual_mult": 1.0,
            "logit_scale": 1.0,
            "layers": [{"type": "attention", "mixer": _att(1, 1, 8, 40, 1.0), "mlp": _moe(1, 1, 16)}]}


def cfg_latent_first():
    return {"architecture": "Fokisun", "vocab": 50, "width": 33, "norm": {"eps": 1e-6}, "residual_mult": 1.4,
            "logit_scale": 2.0,
            "layers": [
                {"type": "latent_attention", "mixer": _lat(5, 6, 2, 10, 12, 9, 0.4), "mlp": None},
                {"type": "hgrn2", "mixer": _rec(1, 17, 5), "mlp": {"kind": "dense", "ff": 19}},
                {"type": "attention", "mixer": _att(3, 1, 10, 7, 0.4, 1, 4, 100.0, 0.5), "mlp": _moe(9, 4, 5, (9, 5), 1.0)},
            ]}


def build(cfg, device, dtype=F32, seed=0, edit=None):
    config = FokisunConfig.from_dict(cfg)
    sd = random_state_dict(config, seed=seed)
    for k in list(sd):
        if k.endswith("mlp.router"):  # clearly separated scores: no near-ties in the choice
            sd[k] = (sd[k].float() * 3.0).to(BF16)
    if edit:
        edit(sd)
    model = FokisunForCausalLM(config, device=device, dtype=dtype, _do_init=False).load_state_dict(sd)
    return model, sd


def toks(n, vocab, seed=1):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def err(got, ref):
    got, ref = np.asarray(got, dtype=np.float64), np.asarray(ref, dtype=np.float64)
    d = got - ref
    return float(np.sqrt(np.mean(d * d)) / np.sqrt(np.mean(ref * ref)))


def tol(dtype=F32):
    return 3e-2 if dtype == BF16 else 2e-5


def run_portions(model, tokens, portions, rid="r", stepper=None, max_tokens=None):
    """Logits of every position through the stepper, the prompt cut into ``portions``."""
    st = stepper or SequenceStepper(model, max_tokens or len(tokens))
    out, at = [], 0
    for n in portions:
        out.append(st.feed(rid, tokens[at:at + n], list(range(n))).float().cpu())
        at += n
    assert at == len(tokens)
    st.end(rid)
    return torch.cat(out).numpy()


# ---------------------------------------------------------------------------------------------- configuration
def test_config_round_trip():
    c = FokisunConfig.from_dict(cfg_full())
    assert FokisunConfig.from_dict(c.to_dict()) == c and c.num_hidden_layers == 7
    assert [type(ls.mixer) for ls in c.layers[:3]] == [GatedRunningSpec, WholeNormAttentionSpec, RotaryLatentSpec]
    a = c.layers[1].mixer
    assert (a.window, a.rot_dims, a.rot_base, a.rot_factor, a.v_mix) == (13, 8, 500.0, 3.0, True)
    assert c.layers[3].mixer.rot_dims == 0 and not c.layers[3].mixer.v_mix and c.layers[4].mixer.window == 0
    f = c.layers[0].mlp
    assert isinstance(f, GatedMoESpec) and (f.experts, f.top, f.groups, f.keep_groups, f.scale, f.ff, f.shared_ff) == \
        (6, 2, 3, 2, 2.5, 24, 40)
    assert isinstance(c.layers[1].mlp, DenseFFSpec) and c.layers[3].mlp is None and c.layers[2].mlp.shared_ff == 0
    assert (c.residual_mult, c.logit_scale, c.norm_eps) == (0.7, 0.3, 1e-5)
    for breaker in (lambda d: d["layers"][0]["mlp"]["router"].update(top=5),               # more than the kept groups hold
                    lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(count=4),   # 6 experts in 4 groups
                    lambda d: d["layers"][1].update(type="delta"),
                    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7),
                    lambda d: d["layers"][1]["mixer"].update(kv_heads=3),
                    lambda d: d["layers"][4]["mixer"].update(vdim=21),                     # mixed values differ in number
                    lambda d: d["layers"][1]["mlp"].update(kind="table")):
        bad = cfg_full()
        breaker(bad)
        with pytest.raises(ValueError):
            FokisunConfig.from_dict(bad)


# ---------------------------------------------------------------------------------------------- mechanisms alone
def _run_mixer(mixer, cache, h, portions, device, v_first=None):
    """A mixer on hand-made inputs in portions: input product, features, output product (+ bias). Returns the outputs and,
    of a mixer that leads the value mixing, the values it left."""
    outs, vals, s0 = [], [], 0
    for s in portions:
        ids = torch.zeros(s, dtype=torch.int32, device=device)
        pos = torch.arange(s0, s0 + s, dtype=torch.int32, device=device)
        ctx = StepContext(ids, pos, 1, s, cache, s0)
        if v_first is not None:
            ctx.v_first = v_first[s0:s0 + s].contiguous().to(device)
        x = h[s0:s0 + s].to(device)
        # (features into a column slice of a wider buffer, as the blocks do)
        feats, part, rest = hy.feature_rows(s, [mixer.width, 3], mixer.head, F32, torch.device(device))
        rest.zero_()
        mixer.features(hy.linear(x, mixer.w_in), ctx, part)
        assert float(rest.abs().max()) == 0.0
        y = hy.linear(part, mixer.w_o)
        outs.append((y + mixer.o_bias if mixer.o_bias is not None else y).cpu())
        if ctx.v_first is not None and v_first is None:
            vals.append(ctx.v_first.cpu())
        s0 += s
    assert s0 == h.shape[0]
    return torch.cat(outs).numpy(), torch.cat(vals).numpy() if vals else None


def _attn_weights(g, mc, d):
    r = lambda *s, sc: torch.randn(*s, generator=g) * sc  # noqa: E731
    nq, nk, nv = mc["heads"] * mc["dim"], mc["kv_heads"] * mc["dim"], mc["kv_heads"] * mc["vdim"]
    w = {"m.q": r(nq, d, sc=0.4), "m.k": r(nk, d, sc=0.4), "m.v": r(nv, d, sc=0.4), "m.q.b": r(nq, sc=0.5),
         "m.k.b": r(nk, sc=0.5), "m.v.b": r(nv, sc=0.5), "m.q.norm": torch.rand(nq, generator=g) + 0.5,
         "m.k.norm": torch.rand(nk, generator=g) + 0.5, "m.g": r(mc["heads"] * mc["vdim"], d, sc=0.5),
         "m.o": r(d, mc["heads"] * mc["vdim"], sc=0.2), "m.o.b": r(d, sc=0.3), "m.vmix": torch.tensor(0.35)}
    return w


def _attn_mixer(w, mc, eps, device, dtype=F32, leads=False, mixes=False):
    sp = WholeNormAttentionSpec.from_dict(mc)
    to = lambda n: w["m." + n].to(device)  # noqa: E731
    freq = hy.rotary_freqs(sp.rot_base, sp.rot_dims, device) / sp.rot_factor if sp.rot_dims else None
    return WholeNormAttention(0, sp, eps, torch.cat([w["m." + n] for n in "qkvg"]).to(device, dtype),
                              torch.cat([w[f"m.{n}.b"] for n in "qkv"]).to(device), to("q.norm"), to("k.norm"), freq,
                              torch.zeros(sp.heads, device=device), leads, to("vmix").reshape(1) if mixes else None,
                              w["m.o"].to(device, dtype), to("o.b"))


def _run_attn(w, mc, h, eps, device, portions, dtype=F32, v_first=None, leads=False):
    cache = HybridCache([("kv", mc["kv_heads"], mc["dim"], mc["vdim"])], 1, h.shape[0], device, dtype)
    return _run_mixer(_attn_mixer(w, mc, eps, device, dtype, leads, v_first is not None), cache, h, portions, device, v_first)


ATT_SHAPES = [  # heads, kv_heads, dim, vdim, window, rot_dims, factor
    (4, 2, 12, 20, 13, 8, 3.0), (1, 1, 8, 72, None, None, None), (6, 6, 17, 8, 1, 16, None), (70, 35, 8, 4, 64, 2, 0.5),
    (8, 1, 24, 40, 30, 24, 7.0), (2, 2, 64, 64, 65, 64, 4.0), (3, 3, 130, 9, 40, 100, 2.0)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,window,rot_dims,factor", ATT_SHAPES)
def test_attention_mechanism(device, heads, kv_heads, dim, vdim, window, rot_dims, factor):
    """One attention sublayer against the oracle: biases, norms over the whole projections, grouped heads, partial
    rotation with scaled frequencies, windows of one key, a 64-key chunk and one more, the added one in the denominator,
    column gates, value mixing; in portions with single tokens and pairs, and token by token."""
    mc = _att(heads, kv_heads, dim, vdim, 0.4, window, rot_dims, 300.0, factor)
    t, d, eps = 90, 48, 1e-5
    g = torch.Generator().manual_seed(5)
    w = _attn_weights(g, mc, d)
    h = torch.randn(t, d, generator=g)
    hn = h.double().numpy()
    vf = torch.randn(t, kv_heads * vdim, generator=g)
    vf_n = vf.double().numpy().reshape(t, kv_heads, vdim)
    plain, mixed = of.attention(w, "m.", mc, hn, eps), of.attention(w, "m.", mc, hn, eps, vf_n)
    for portions in ([11, 1, 2, 38, 1, 1, 30, 6], [1] * t):
        got, vals = _run_attn(w, mc, h, eps, device, portions, leads=True)
        assert err(got, plain) < 2e-5
        assert err(vals.reshape(t, kv_heads, vdim), of.attention_values(w, "m.", mc, hn)) < 2e-6
        got, vals = _run_attn(w, mc, h, eps, device, portions, v_first=vf)
        assert vals is None and err(got, mixed) < 2e-5
    assert err(plain, mixed) > 0.05


def test_oracle_faults_show():
    """What the attention comparison above would see of a fault: each planted in the oracle's inputs, each far above the
    tolerance -- per-head instead of whole norms, the other pair layout, unscaled frequencies, no added one, a window one
    off, gates per head."""
    mc = _att(4, 2, 12, 20, 0.4, 13, 8, 300.0, 3.0)
    t, d, eps = 40, 48, 1e-5
    g = torch.Generator().manual_seed(5)
    w = _attn_weights(g, mc, d)
    h = torch.randn(t, d, generator=g).double().numpy()
    ref = of.attention(w, "m.", mc, h, eps)
    faults = [dict(mc, rot={"base": 300.0, "dims": 8}), dict(mc, mask={"size": 12}), dict(mc, mask={"size": 14}),
              dict(mc, rot=dict(mc["rot"], dims=10)), dict(mc, scale=0.41)]
    for f in faults:
        assert err(of.attention(w, "m.", f, h, eps), ref) > 1e-3
    rot, wts = of.rotate, of.weights_of
    try:
        of.rotate = lambda x, pos, r, adjacent: rot(x, pos, r, not adjacent)
        assert err(of.attention(w, "m.", mc, h, eps), ref) > 1e-3
        of.rotate = rot
        of.weights_of = lambda q, k, s, win, extra: wts(q, k, s, win, 0.0)
        assert err(of.attention(w, "m.", mc, h, eps), ref) > 1e-2
    finally:
        of.rotate, of.weights_of = rot, wts


@pytest.mark.parametrize("device", DEVICES)
def test_added_one_decides_at_the_first_tokens(device):
    """Scores of a few tokens held near zero: the first token keeps about half of its value, the second two thirds. A
    denominator without the added one would return the whole mean."""
    mc = _att(3, 1, 8, 16, 1e-4, 20, 8)
    t, d, eps = 6, 24, 1e-6
    g = torch.Generator().manual_seed(3)
    w = _attn_weights(g, mc, d)
    h = torch.randn(t, d, generator=g)
    ref, pw = of.attention(w, "m.", mc, h.double().numpy(), eps, return_weights=True)
    for i in range(t):
        assert abs(pw[:, i].sum(-1).max() - (i + 1) / (i + 2)) < 1e-3
    for portions in ([t], [1] * t, [2, 4]):
        assert err(_run_attn(w, mc, h, eps, device, portions)[0], ref) < 2e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_attention_at_the_mfma_head_sizes(device, dtype):
    """Head sizes of the flash prefill kernel and the fast decode kernel (bf16), windows that end inside the 32-key tiles,
    portions that start at unaligned slots."""
    t, d, eps = 300, 96, 1e-6
    g = torch.Generator().manual_seed(9)
    h = torch.randn(t, d, generator=g).to(BF16).float()
    for dim, vdim, window, rot in [(64, 128, 45, 32), (128, 64, 70, 128), (64, 64, 33, 64), (128, 128, None, 96),
                                   (96, 64, 100, 32), (80, 128, 31, 80)]:
        mc = _att(4, 2, dim, vdim, dim ** -0.5 * 4.0, window, rot, 1e4, 2.0)
        w = {k: v.to(BF16).float() for k, v in _attn_weights(g, mc, d).items()}
        ref = of.attention(w, "m.", mc, h.double().numpy(), eps)
        got, _ = _run_attn(w, mc, h, eps, device, [100, 2, 147, 1, 50], dtype)
        assert err(got, ref) < tol(dtype), (dim, vdim, window)


def _point_at(wq, key):
    """An input whose projection by ``wq [n, d]`` (n <= d) is ``key``: the least-squares solution."""
    return np.linalg.lstsq(wq, key, rcond=None)[0]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_attention_keys_at_the_window_edge_decide(device, dtype):
    """Queries inside a portion and decoded alone are solved so that head 0 points at one (rotated) key each: the oldest
    key inside its window, the newest outside, one ten tokens back. A window that is one off moves those rows by far more
    than the tolerance."""
    heads, dim, vdim, d, t, eps, window = 2, 24, 20, 64, 333, 1e-6, 37
    mc = _att(heads, 1, dim, vdim, 4.0, window, 24, 1e4, 2.0)
    g = torch.Generator().manual_seed(7)
    w = {k: v.to(BF16).float() for k, v in _attn_weights(g, mc, d).items()}
    w["m.q.norm"], w["m.k.norm"] = torch.ones(heads * dim), torch.ones(dim)
    h = (torch.randn(t, d, generator=g) * 0.3).to(BF16).float()
    hn = h.double().numpy()
    keys = of.rms(hn @ w["m.k"].double().numpy().T + w["m.k.b"].double().numpy(), eps)
    wq, bq = w["m.q"].double().numpy(), w["m.q.b"].double().numpy()
    rows = {}
    for base in (296, 329):  # inside the portion 290 .. 326, and among the tokens decoded alone
        for n, (kind, back) in enumerate((("in", window - 1), ("out", window), ("near", 10))):
            i = base + n
            # the query that, turned by its own position, meets the key turned by the key's position; head 1 stays small
            want = of.rotate(keys[i - back][None, None], [-float(back)], mc["rot"], True)[0, 0] * 3.0
            h[i] = torch.tensor(_point_at(wq, np.concatenate([want, 0.3 * bq[dim:]]) - bq), dtype=F32).to(BF16).float()
            rows[i] = (kind, i - back)
    hn = h.double().numpy()
    ref, pw = of.attention(w, "m.", mc, hn, eps, return_weights=True)
    for i, (kind, j) in rows.items():
        assert (pw[0, i, j] == 0.0) if kind == "out" else (pw[0, i, j] > 0.9), (i, kind, pw[0, i, j])
    got, _ = _run_attn(w, mc, h, eps, device, [290, 37] + [1] * 6, dtype)
    assert err(got, ref) < tol(dtype)
    for i in rows:
        assert err(got[i], ref[i]) < 2 * tol(dtype), (i, rows[i])
    for kind, size in (("in", window - 1), ("out", window + 1)):
        off = of.attention(w, "m.", dict(mc, mask={"size": size}), hn, eps)
        for i, (k2, _) in rows.items():
            if k2 == kind:
                assert err(off[i], ref[i]) > 0.2, (i, kind)


def _latent_weights(g, mc, d):
    r = lambda *s, sc: torch.randn(*s, generator=g) * sc  # noqa: E731
    nh, kd, rank = mc["heads"], mc["dim"] + mc["rot_dim"], mc["kv_rank"]
    return {"m.dq": r(mc["q_rank"], d, sc=0.4), "m.dq.norm": torch.rand(mc["q_rank"], generator=g) + 0.5,
            "m.uq": r(nh * kd, mc["q_rank"], sc=0.4), "m.dkv": r(rank + mc["rot_dim"], d, sc=0.4),
            "m.dkv.norm": torch.rand(rank, generator=g) + 0.5, "m.uk": r(nh * mc["dim"], rank, sc=0.4),
            "m.uv": r(nh * mc["vdim"], rank, sc=0.4), "m.g": r(nh, d, sc=0.5), "m.o": r(d, nh * mc["vdim"], sc=0.2)}


def _run_latent(w, mc, h, eps, device, portions, dtype=F32, form=None):
    sp = RotaryLatentSpec.from_dict(mc)
    cache = HybridCache([("latent", sp.kv_rank + sp.rot_dim)], 1, h.shape[0], device, dtype)
    mixer = RotaryLatentAttention(0, sp, eps, torch.cat([w["m.dq"], w["m.dkv"], w["m.g"]]).to(device, dtype),
                                  w["m.dq.norm"].to(device), w["m.uq"].to(device, dtype), w["m.dkv.norm"].to(device),
                                  w["m.uk"].reshape(sp.heads, sp.dim, sp.kv_rank).to(device, dtype),
                                  w["m.uv"].reshape(sp.heads, sp.vdim, sp.kv_rank).contiguous().to(device, dtype),
                                  hy.rotary_freqs(sp.rot_base, sp.rot_dims, device), w["m.o"].to(device, dtype),
                                  interleaved=False)
    if form is not None:
        mixer.expands = lambda s, n, bf16: form == "expanded"
    return _run_mixer(mixer, cache, h, portions, device)[0]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,dim,rot_dim,vdim,rank,q_rank", [
    (3, 16, 8, 24, 20, 28), (1, 8, 2, 72, 56, 8), (12, 8, 4, 8, 24, 16), (70, 8, 6, 4, 16, 8), (2, 16, 16, 16, 200, 24),
    (2, 16, 64, 16, 512, 24), (2, 16, 8, 16, 520, 24)])
def test_latent_attention_mechanism(device, heads, dim, rot_dim, vdim, rank, q_rank):
    """One latent-attention sublayer against the oracle (which materialises every head's keys and values) in both forms and
    in portions with single tokens and pairs; rotated pairs half the rotated part apart (the other layout fails)."""
    mc = _lat(heads, dim, rot_dim, vdim, rank, q_rank, 0.31, 300.0)
    t, d, eps = 71, 48, 1e-6
    g = torch.Generator().manual_seed(3)
    w = _latent_weights(g, mc, d)
    h = torch.randn(t, d, generator=g)
    ref = of.latent_attention(w, "m.", mc, h.double().numpy(), eps)
    for form in ("latent", "expanded", None):
        got = _run_latent(w, mc, h, eps, device, [11, 1, 2, 29, 1, 1, 20, 6], form=form)
        assert err(got, ref) < 2e-5, form
    if rot_dim > 2:
        rot = of.rotate
        try:
            of.rotate = lambda x, pos, r, adjacent: rot(x, pos, r, not adjacent)
            assert err(of.latent_attention(w, "m.", mc, h.double().numpy(), eps), ref) > 1e-3
        finally:
            of.rotate = rot


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_latent_far_keys_decide(device, dtype):
    """Late queries (in a portion and decoded alone) solved so that head 0 points at the plain key of one token 300 and
    more positions back, at a page-sized distance and at the sequence's first token; both forms."""
    heads, dim, rot, vdim, rank, q_rank, d, t, eps = 2, 32, 4, 24, 40, 36, 48, 390, 1e-6
    mc = _lat(heads, dim, rot, vdim, rank, q_rank, 0.8, 100.0)
    g = torch.Generator().manual_seed(12)
    w = {k: v.to(BF16).float() for k, v in _latent_weights(g, mc, d).items()}
    w["m.dq.norm"] = torch.ones(q_rank)
    w["m.g"][0] = 0.0
    h = (torch.randn(t, d, generator=g) * 0.3).to(BF16).float()
    hn = h.double().numpy()
    c = of.rms(hn @ w["m.dkv"].double().numpy()[:rank].T, eps) * w["m.dkv.norm"].double().numpy()
    k_plain = c @ w["m.uk"].double().numpy()[:dim].T
    uq0 = w["m.uq"].double().numpy()[:dim]
    rows = {}
    for base in (370, 385):
        for n, j in enumerate((0, 1, 63, 64)):
            h[base + n] = torch.tensor(_point_at(w["m.dq"].double().numpy(), _point_at(uq0, k_plain[j])), dtype=F32).to(
                BF16).float()
            rows[base + n] = j
    ref, pw = of.latent_attention(w, "m.", mc, h.double().numpy(), eps, return_weights=True)
    for i, j in rows.items():
        assert pw[0, i, j] > 0.7, (i, j, pw[0, i, j])
    for form in ("latent", "expanded"):
        got = _run_latent(w, mc, h, eps, device, [360, 22] + [1] * 8, dtype, form)
        assert err(got, ref) < tol(dtype), form
        for i in rows:
            assert err(got[i], ref[i]) < 2 * tol(dtype), (form, i)


def _rec_weights(g, mc, d, bias=(-1.0, 3.0), lower=(0.0, 0.9)):
    r = lambda *s, sc: torch.randn(*s, generator=g) * sc  # noqa: E731
    n, nv = mc["heads"] * mc["dim"], mc["heads"] * mc["vdim"]
    u = lambda lo, hi: torch.rand(n, generator=g) * (hi - lo) + lo  # noqa: E731
    return {"m.q": r(n, d, sc=0.3), "m.f": r(n, d, sc=0.3), "m.v": r(nv, d, sc=0.3), "m.f.b": u(*bias), "m.lower": u(*lower),
            "m.norm": torch.rand(mc["vdim"], generator=g) + 0.5, "m.o": r(d, nv, sc=0.3)}


def _run_rec(w, mc, h, eps, device, portions, dtype=F32):
    sp = GatedRunningSpec.from_dict(mc)
    cache = HybridCache([("linear", sp.heads, sp.dim, sp.vdim)], 1, 8, device, dtype)
    mixer = GatedRunningMixer(0, sp, eps, torch.cat([w["m.q"], w["m.f"], w["m.v"]]).to(device, dtype), w["m.f.b"].to(device),
                              w["m.lower"].to(device), w["m.norm"].to(device), w["m.o"].to(device, dtype))
    out, _ = _run_mixer(mixer, cache, h, portions, device)
    return out, cache.recurrent(0)[0][0].cpu().numpy()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,dim,vdim,t", [(3, 12, 20, 70), (1, 1, 1, 9), (2, 64, 64, 300), (5, 17, 33, 200), (1, 130, 9, 260),
                                              (9, 16, 257, 40), (1, 600, 4, 210)])
def test_running_memory_mechanism(device, heads, dim, vdim, t):
    """The recurrence against the oracle, output and carried state: one pass, segments side by side (128 tokens and more),
    portions with single tokens and pairs, token by token."""
    mc = _rec(heads, dim, vdim)
    d, eps = 40, 1e-6
    g = torch.Generator().manual_seed(8)
    w = _rec_weights(g, mc, d)
    h = torch.randn(t, d, generator=g)
    ref, state = of.hgrn2(w, "m.", mc, h.double().numpy(), eps, return_state=True)
    for portions in ([t], [1] * t, [2, 1, t - 6, 3]):
        got, st = _run_rec(w, mc, h, eps, device, portions)
        assert err(got, ref) < 2e-5 and err(st, state) < 2e-5, portions


@pytest.mark.gpu
@pytest.mark.parametrize("seg_min", [4, 16])
def test_running_memory_in_short_segments(seg_min, monkeypatch):
    """Many short segments side by side, an uneven last one, a second portion that starts from a carried state."""
    monkeypatch.setattr(hy, "SCAN_SEG_MIN", seg_min)
    t, d, eps = 75, 40, 1e-6
    g = torch.Generator().manual_seed(11)
    h = torch.randn(t, d, generator=g)
    for mc in (_rec(3, 8, 12), _rec(2, 40, 33), _rec(1, 130, 4)):
        w = _rec_weights(g, mc, d)
        ref, state = of.hgrn2(w, "m.", mc, h.double().numpy(), eps, return_state=True)
        for portions in ([75], [40, 35], [9, 66]):
            assert hy._scan_segments(1, portions[-1], mc["heads"], mc["dim"], mc["vdim"], "cuda")[0] > 1
            got, st = _run_rec(w, mc, h, eps, "cuda", portions)
            assert err(got, ref) < 2e-5 and err(st, state) < 2e-5, (mc, portions)


@pytest.mark.parametrize("device", DEVICES)
def test_running_memory_keeps_and_forgets(device):
    """Gates within 1e-3 of one (the write factor is then a small difference of near-equal numbers, which must keep its
    relative accuracy over 400 tokens, and the first tokens still weigh in at the end) and gates near zero (the state is
    the last value)."""
    mc = _rec(2, 24, 16)
    t, d, eps = 400, 40, 1e-6
    g = torch.Generator().manual_seed(4)
    h = torch.randn(t, d, generator=g)
    w = _rec_weights(g, mc, d, bias=(4.0, 6.0), lower=(0.85, 0.95))
    ref, state = of.hgrn2(w, "m.", mc, h.double().numpy(), eps, return_state=True)
    _, lost = of.hgrn2(w, "m.", mc, h[64:].double().numpy(), eps, return_state=True)
    assert err(lost, state) > 0.03  # a state lost at token 64 shows at token 400
    for portions in ([t], [390] + [1] * 10, [64] * 6 + [16]):
        got, st = _run_rec(w, mc, h, eps, device, portions)
        assert err(got, ref) < 2e-5 and err(st, state) < 2e-5
    w = _rec_weights(g, mc, d, bias=(-12.0, -9.0), lower=(0.0, 1e-3))
    ref, state = of.hgrn2(w, "m.", mc, h.double().numpy(), eps, return_state=True)
    got, st = _run_rec(w, mc, h, eps, device, [t])
    assert err(got, ref) < 2e-5 and err(st, state) < 2e-5


def _moe_weights(g, d, fc, scale=1.0):
    r = lambda *s, sc: torch.randn(*s, generator=g) * sc  # noqa: E731
    w = {"f.router": r(fc["router"]["experts"], d, sc=scale)}
    names = [(f"f.e{e}.", fc["expert"]["ff"]) for e in range(fc["router"]["experts"])]
    if fc.get("shared"):
        names.append(("f.shared.", fc["shared"]["ff"]))
    for pre, ff in names:
        w.update({pre + "gate": r(ff, d, sc=0.4), pre + "up": r(ff, d, sc=0.4), pre + "down": r(d, ff, sc=0.3)})
    return w


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("m,experts,top,groups,scale", [
    (1, 4, 2, None, 1.0), (2, 6, 3, (3, 2), 2.5), (3, 8, 4, (4, 2), 0.7), (40, 9, 2, (3, 2), 1.5), (70, 1, 1, None, 1.0),
    (9, 64, 4, (8, 3), 1.5), (300, 6, 1, (3, 1), 3.0), (17, 6, 3, (6, 4), 1.0), (5, 96, 5, (12, 4), 1.2), (21, 130, 3, (2, 1), 0.9)])
def test_gated_mixture(device, m, experts, top, groups, scale):
    """Router (sigmoid scores, groups scored by two members, normalised and scaled weights; one expert per lane and the
    form for more than 64 experts, groups of one) and gated experts at the row counts of all three linear paths."""
    d = 40
    fc = _moe(experts, top, 24, groups, scale)
    g = torch.Generator().manual_seed(5)
    w = _moe_weights(g, d, fc, 0.2)
    x = torch.randn(m, d, generator=g)
    chosen, weight = of.route(w, "f.", fc, x.double().numpy())
    rule = hy.RouterRule(True, 2, True, scale)
    up = torch.stack([torch.cat([w[f"f.e{e}.gate"], w[f"f.e{e}.up"]]) for e in range(experts)])
    moe = GatedMoE(experts, top, groups[0] if groups else 1, groups[1] if groups else 1, rule, w["f.router"].to(device),
                   up.to(device), torch.stack([w[f"f.e{e}.down"] for e in range(experts)]).to(device))
    # the router's logits sit in the middle of a wider projection
    z = torch.cat([torch.full((m, 3), 99.0), x @ w["f.router"].t(), torch.full((m, 2), 99.0)], 1).to(device)[:, 3:3 + experts]
    y, row_w = moe(x.to(device), z)
    assert y.shape == (m * top, d)
    assert err(row_w.reshape(m, top).cpu().numpy(), weight) < 1e-5
    assert np.allclose(row_w.reshape(m, top).sum(-1).cpu().numpy(), scale, rtol=1e-5)
    hist = torch.zeros(2, m, d, device=device)
    xo = torch.empty(m, d, device=device)
    zero = torch.zeros(m, d, device=device)
    hy.depth_update_(hist, 0, zero, xo, 1.0, zero, torch.tensor([0.0, 1.0], device=device), ye=y, nsum=top, row_w=row_w)
    assert err(xo.cpu().numpy(), of.moe(w, "f.", fc, x.double().numpy())) < 2e-5
    ex, wt = hy.route_grouped(x @ w["f.router"].t(), None, top, groups[0] if groups else 1, groups[1] if groups else 1, rule)
    assert np.array_equal(ex.reshape(m, top).numpy(), chosen) and err(wt.reshape(m, top).numpy(), weight) < 1e-5


def test_two_scores_make_a_group():
    """A group with the single largest score loses to one whose two largest sum higher, and the chosen weights are
    normalised over the chosen, not over the kept."""
    z = torch.tensor([[3.0, -4.0, -4.0, 1.2, 1.1, -4.0, 0.0, 0.1, 0.2]])  # groups of 3: sums .97, 1.52, 1.07
    rule = hy.RouterRule(True, 2, True, 2.0)
    ex, wt = hy.route_grouped(z, None, 2, 3, 1, rule)
    assert ex.tolist() == [3, 4] and abs(float(wt.sum()) - 2.0) < 1e-6
    assert hy.route_grouped(z, None, 2, 3, 1, hy.RouterRule(True, 1, True, 2.0))[0].tolist()[0] == 0
    w = {"f.router": torch.eye(9)}
    chosen, weight = of.route(w, "f.", _moe(9, 2, 4, (3, 1), 2.0), z.double().numpy())
    assert chosen.tolist() == [[3, 4]] and np.allclose(weight, wt.numpy(), atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("m,d,ff,act,fn", [(1, 40, 24, hy.ACT_GELU_GLU, of.gelu), (7, 33, 19, hy.ACT_GELU_GLU, of.gelu),
                                           (70, 64, 100, hy.ACT_SWIGLU, of.silu), (300, 96, 48, hy.ACT_GELU_GLU, of.gelu)])
def test_gated_halves_into_a_slice(device, m, d, ff, act, fn):
    """The gated first half of a feed-forward into columns 8 .. of a wider buffer, fp32 and (prompt-sized) bf16."""
    g = torch.Generator().manual_seed(2)
    x, w = torch.randn(m, d, generator=g), torch.randn(2 * ff, d, generator=g) * d ** -0.5
    for dtype in (F32, BF16):
        h = x.to(BF16).float() if dtype == BF16 else x
        wd = w.to(dtype)
        ref = fn(h.double().numpy() @ wd[:ff].double().numpy().T) * (h.double().numpy() @ wd[ff:].double().numpy().T)
        act_t = BF16 if hy.prompt_bf16(m, d, dtype) else F32
        buf = torch.zeros(m, ff + 11, dtype=act_t, device=device)
        hy.linear_glu(h.to(act_t).to(device), wd.to(device), act, buf[:, 8:8 + ff])
        assert err(buf[:, 8:8 + ff].float().cpu().numpy(), ref) < (5e-3 if act_t == BF16 else 1e-5)
        assert float(buf[:, :8].abs().max()) == 0.0 and float(buf[:, 8 + ff:].abs().max()) == 0.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("i,m,d,top", [(0, 3, 40, 0), (1, 1, 33, 2), (4, 70, 256, 3), (9, 5, 301, 1), (2, 2, 2052, 0), (30, 300, 64, 8)])
def test_depth_update(device, i, m, d, top):
    """The residual step alone: residual add with its constant, output bias, weighted expert rows, the new plane, the
    weighted sum over all planes (distinct weights: an order or index that is off shows), the next layer's norm in both
    formats; in place and from another tensor; planes behind the new one untouched."""
    g = torch.Generator().manual_seed(6)
    r = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    hist, x, y, bias, coef = r(i + 3, m, d), r(m, d), r(m, d), r(d), r(i + 2)
    ye, rw = (r(m * top, d), r(m * top)) if top else (None, None)
    nw, nb = r(d), r(d)
    v = y.double() + bias.double()
    if top:
        v = v + (ye.double() * rw.double()[:, None]).reshape(m, top, d).sum(1)
    new = (x.double() + 0.6 * v).numpy()
    states = [hist[j].double().numpy() for j in range(i + 1)] + [new]
    want = of.depth_average(coef, states)
    h_want = of.squash({"n": nw, "n.b": nb, "n.alpha": torch.tensor(0.5)}, "n", want)
    norm = hy.SquashNorm(torch.tensor([0.5], device=device), nw.to(device), nb.to(device))
    to = lambda t: t.to(device) if t is not None else None  # noqa: E731
    for dtype, place in ((F32, True), (BF16, False)):
        hd, xd = hist.to(device).clone(), x.to(device).clone()
        xo = xd if place else torch.empty_like(xd)
        h = hy.depth_update_(hd, i, xd, xo, 0.6, to(y), to(coef), to(bias), to(ye), max(top, 1), to(rw), norm=norm, h_dtype=dtype)
        assert err(hd[i + 1].cpu().numpy(), new) < 1e-6 and err(xo.cpu().numpy(), want) < 1e-6
        assert torch.equal(hd[:i + 1].cpu(), hist[:i + 1]) and torch.equal(hd[i + 2].cpu(), hist[i + 2])
        assert h.dtype == dtype and err(h.float().cpu().numpy(), h_want) < (3e-3 if dtype == BF16 else 2e-6)
        assert err(hy.squash_rows(xo, norm, dtype).float().cpu().numpy(), h_want) < (3e-3 if dtype == BF16 else 2e-6)
    hd, xd = hist.to(device).clone(), x.to(device).clone()
    assert hy.depth_update_(hd, i, xd, xd, 0.6, to(y), to(coef), to(bias), to(ye), max(top, 1), to(rw), store=False) is None
    assert torch.equal(hd.cpu(), hist) and err(xd.cpu().numpy(), want) < 1e-6


# ---------------------------------------------------------------------------------------------- whole model
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [cfg_full, cfg_bare, cfg_latent_first])
def test_prompt_logits_and_residual_stream(device, cfg):
    model, sd = build(cfg(), device)
    t = toks(45, model.config.vocab_size)
    ref, ref_hidden = of.forward(cfg(), sd, t)
    ids = torch.tensor([t], dtype=torch.int32)
    out = model(ids, output_hidden_states=True)
    assert len(out.hidden_states) == len(ref_hidden)
    for i, hs in enumerate(out.hidden_states):
        assert err(hs[0].cpu().numpy(), ref_hidden[i]) < tol(), f"layer {i}"
    assert err(out.logits[0].cpu().numpy(), ref) < tol()
    assert err(out.logits[0, :3].cpu().numpy(), ref[:3]) < tol()  # the first tokens of a sequence
    # the last token alone (what a prefill of the engine asks for) and no logits at all
    cache = model.init_cache(1, 45)
    pos = torch.arange(45, dtype=torch.int32, device=device).reshape(1, -1)
    last, *_ = model.forward_tokens(ids.to(device), pos, cache, 0, logits_mode="last")
    assert err(last[0].cpu().numpy(), ref[-1]) < tol()
    assert model.forward_tokens(ids.to(device), pos, model.init_cache(1, 45), 0, logits_mode="none")[0] is None


def test_depth_weights_and_value_mixing_matter():
    """Faults the whole-model comparison must see, planted in the oracle's weights: depth weights in another order, the
    mixing weight of the first value-mixing layer (which is unused) and of the second one (which is not)."""
    _, sd = build(cfg_full(), "cpu")
    t = toks(20, 67)
    ref, _ = of.forward(cfg_full(), sd, t)
    bad = dict(sd)
    bad["l4.dwa"] = sd["l4.dwa"].flip(0)
    assert err(of.forward(cfg_full(), bad, t)[0], ref) > 1e-2
    bad = dict(sd)
    bad["l1.mix.vmix"] = sd["l1.mix.vmix"] * 0
    assert err(of.forward(cfg_full(), bad, t)[0], ref) == 0.0
    bad["l4.mix.vmix"] = sd["l4.mix.vmix"] * 0
    assert err(of.forward(cfg_full(), bad, t)[0], ref) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_bfloat16_serving_format(device):
    model, sd = build(cfg_full(), device, dtype=BF16)
    t = toks(40, 67)
    ref, _ = of.forward(cfg_full(), sd, t)
    got = run_portions(model, t, [33] + [1] * 7)
    assert err(got, ref) < 5e-2
    cache = model.init_cache(1, 8)
    state, none = cache.recurrent(0)
    assert state.dtype == F32 and state.shape == (1, 3, 12, 20) and none is None
    k, v = cache.layer(1)
    assert k.dtype == BF16 and k.shape == (1, 2, 8, 12) and v.shape == (1, 2, 8, 20)
    k, v = cache.layer(2)
    assert k is v and k.shape == (1, 1, 8, 20 + 8)  # the latent and the rotated key part
    kv = 2 * 8 * (2 * 32 + 28 + 3 * 16 + 2 * 36 + 48)
    assert cache.nbytes() == model.cache_nbytes(1, 8) == kv + 4 * (3 * 12 * 20 + 2 * 24 * 8)
    rows = cache.rows(0, 1)
    assert rows.recurrent(0)[1] is None and rows.recurrent(0)[0].data_ptr() == state.data_ptr()
    blk = model.blocks[1]
    assert blk.coef.dtype == F32 and blk.mixer.bias.dtype == F32 and blk.norm.w.dtype == F32 and blk.w_out.dtype == BF16
    assert model.head is model.embed


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [cfg_full, cfg_bare, cfg_latent_first])
def test_prefill_against_token_by_token(device, cfg):
    model, sd = build(cfg(), device)
    t = toks(34, model.config.vocab_size, seed=2)
    ref, _ = of.forward(cfg(), sd, t)
    whole = run_portions(model, t, [34])
    single = run_portions(model, t, [1] * 34)
    assert err(whole, ref) < tol() and err(single, ref) < tol() and err(single, whole) < tol()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("portions", [[2] * 20, [3, 2, 9, 1, 1, 17, 2, 5], [12, 13, 14, 1], [1, 39], [38, 2]])
def test_portions_of_any_size(device, portions):
    model, sd = build(cfg_full(), device, seed=1)
    t = toks(sum(portions), 67, seed=3)
    ref, _ = of.forward(cfg_full(), sd, t)
    assert err(run_portions(model, t, portions), ref) < tol()


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    """150 single-token steps after a short prompt: the windows pass over decoded tokens, the unwindowed layers go past the
    64-key chunks and the key splits of the decode kernels."""
    model, sd = build(cfg_full(), device, seed=2)
    t = toks(156, 67, seed=4)
    ref, _ = of.forward(cfg_full(), sd, t)
    got = run_portions(model, t, [6] + [1] * 150)
    e = [err(got[i], ref[i]) for i in range(156)]
    assert max(e) < 3 * tol(), int(np.argmax(e))


@pytest.mark.parametrize("device", DEVICES)
def test_rows_are_reset_and_reused(device):
    """A finished request's cache row serves the next request from a clean start; two live requests fed in turns do not
    touch each other."""
    model, sd = build(cfg_full(), device)
    a, b = toks(21, 67, seed=6), toks(17, 67, seed=7)
    ref_a, _ = of.forward(cfg_full(), sd, a)
    ref_b, _ = of.forward(cfg_full(), sd, b)
    st = SequenceStepper(model, 32)
    assert err(run_portions(model, a, [20, 1], "a", st), ref_a) < tol()
    assert st.live() == [] and len(st._free) == 1
    assert err(run_portions(model, b, [5, 12], "b", st), ref_b) < tol()  # the same row again, shorter
    assert len(st._free) == 1
    got_a, got_b = [], []
    for lo in range(0, 21, 3):  # interleaved: two rows live at once
        got_a.append(st.feed("a", a[lo:lo + 3], list(range(len(a[lo:lo + 3])))).cpu())
        if lo < 17:
            got_b.append(st.feed("b", b[lo:lo + 3], list(range(len(b[lo:lo + 3])))).cpu())
    assert st.live() == ["a", "b"] and st.held("a") == 21 and st.held("b") == 17
    assert err(torch.cat(got_a).numpy(), ref_a) < tol() and err(torch.cat(got_b).numpy(), ref_b) < tol()
    with pytest.raises(ValueError):
        st.feed("a", toks(12, 67), [])  # more than the row holds


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_batch_rows_against_each_alone(device, dtype):
    model, sd = build(cfg_full(), device, dtype)
    rows = [toks(19, 67, seed=8), toks(19, 67, seed=9), toks(19, 67, seed=10)]
    cache = model.init_cache(3, 24)
    out = model(torch.tensor(rows, dtype=torch.int32), past_key_values=cache).logits
    nxt = [[5], [6], [7]]
    out2 = model(torch.tensor(nxt, dtype=torch.int32), past_key_values=cache).logits  # one decode step of the batch
    for r in range(3):
        ref, _ = of.forward(cfg_full(), sd, rows[r] + nxt[r])
        lim = 5e-2 if dtype == BF16 else tol()
        assert err(out[r].cpu().numpy(), ref[:19]) < lim
        assert err(out2[r].cpu().numpy(), ref[19:]) < 2 * lim


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [cfg_full, cfg_bare, cfg_latent_first])
def test_greedy_generation_through_the_engine(device, cfg):
    """model.generate (prefill + decode steps of the engine, hipGraph replay on the GPU): every generated token is the
    oracle's argmax of the sequence so far (up to rounding between near-equal logits)."""
    model, sd = build(cfg(), device)
    v = model.config.vocab_size
    prompt = toks(9, v, seed=11)
    seq = model.generate(torch.tensor([prompt], dtype=torch.int32),
                         generation_config=GenerationConfig(max_length=40, pad_token_id=0)).sequences[0].cpu().tolist()
    assert seq[:9] == prompt and len(seq) == 40 and all(0 <= x < v for x in seq)
    ref, _ = of.forward(cfg(), sd, seq)
    for i in range(9, 40):
        row = ref[i - 1]
        assert row.max() - row[seq[i]] <= 1e-4 * np.abs(row).max(), i
    again = model.generate(torch.tensor([prompt], dtype=torch.int32),
                           generation_config=GenerationConfig(max_length=40, pad_token_id=0)).sequences[0].cpu().tolist()
    assert again == seq  # the engine's cached cache row starts clean


@pytest.mark.parametrize("device", DEVICES)
def test_batched_generation_through_the_engine(device):
    """Three prompts in one batch generate what each generates alone."""
    model, _ = build(cfg_full(), device)
    prompts = [toks(8, 67, seed=s) for s in (31, 32, 33)]
    gc = GenerationConfig(max_length=26, pad_token_id=0)
    both = model.generate(torch.tensor(prompts, dtype=torch.int32), generation_config=gc).sequences.cpu().tolist()
    for p, seq in zip(prompts, both):
        alone = model.generate(torch.tensor([p], dtype=torch.int32), generation_config=gc).sequences[0].cpu().tolist()
        assert alone == seq


@pytest.mark.parametrize("device", DEVICES)
def test_sampled_generation_through_the_engine(device):
    """The framework's sampler (temperature, top-k, top-p, seeded) on Fokisun logits: reproducible per seed, different
    across seeds, and every token inside the top-k of the oracle's logits."""
    model, sd = build(cfg_full(), device)
    prompt = torch.tensor([toks(7, 67, seed=14)], dtype=torch.int32)
    gc = dict(max_length=27, pad_token_id=0, do_sample=True, temperature=0.9, top_k=5, top_p=0.95)
    a = model.generate(prompt, generation_config=GenerationConfig(seed=3, **gc)).sequences[0].cpu().tolist()
    b = model.generate(prompt, generation_config=GenerationConfig(seed=3, **gc)).sequences[0].cpu().tolist()
    c = model.generate(prompt, generation_config=GenerationConfig(seed=4, **gc)).sequences[0].cpu().tolist()
    assert a == b and a != c and all(0 <= x < 67 for x in a + c)
    ref, _ = of.forward(cfg_full(), sd, a)
    for i in range(7, 27):
        row = ref[i - 1]
        assert row[a[i]] >= np.sort(row)[-5] - 1e-4 * np.abs(row).max(), i


def test_checkpoint_directory_round_trip(tmp_path):
    from jax_llama_amd.models import registry
    model, sd = build(cfg_full(), "cpu")
    model.save_pretrained(str(tmp_path), sd)
    assert registry.architecture_of(str(tmp_path)) == "fokisun"
    again = registry.load_model(str(tmp_path), device="cpu", dtype=F32)
    ids = torch.tensor([toks(12, 67)], dtype=torch.int32)
    assert torch.equal(again(ids).logits, model(ids).logits)
    assert registry.supports_dtype("fokisun", F32) and registry.supports_dtype("fokisun", BF16)
    assert again.weight_bytes() > 0
    for name in ("l2.mix.uk", "l0.mix.v", "l1.mix.q.norm", "l4.dwa", "l1.mlp.down", "final.norm.b"):
        bad = dict(sd)
        bad[name] = bad[name][:-1]
        with pytest.raises(ValueError):
            FokisunForCausalLM(model.config, _do_init=False).load_state_dict(bad)


def test_trace_runner_program(tmp_path):
    """bin/trace_run as a user starts it: steps on standard input, logits files, 'done' lines, rows given back."""
    import json
    import os
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    model, sd = build(cfg_full(), "cpu")
    ckpt, out = str(tmp_path / "ckpt"), str(tmp_path / "out")
    model.save_pretrained(ckpt, sd)
    a, b = toks(9, 67, seed=12), toks(5, 67, seed=13)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [0, 5]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[6:8], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[8:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [4]}], "end": ["b"]}]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", ckpt, "--dtype", "float32",
                        "--out", out, "--max-tokens", "16", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not os.path.exists(os.path.join(out, "1.f32"))
    ref_a, _ = of.forward(cfg_full(), sd, a)
    ref_b, _ = of.forward(cfg_full(), sd, b)
    got0 = np.fromfile(os.path.join(out, "0.f32"), dtype="<f4").reshape(2, 67)
    got2 = np.fromfile(os.path.join(out, "2.f32"), dtype="<f4").reshape(1, 67)
    got3 = np.fromfile(os.path.join(out, "3.f32"), dtype="<f4").reshape(1, 67)
    assert err(got0, ref_a[[0, 5]]) < 2e-5 and err(got2, ref_a[[8]]) < 2e-5 and err(got3, ref_b[[4]]) < 2e-5


def cfg_kernel_shapes():
    """Head sizes of the MFMA attention kernels beside plain ones, a cache row wide enough for the shared-latent decode
    kernel, experts with enough rows for the expert-grouped tiles, matrices in whole tiles (the packed GEMM takes them)."""
    return {"architecture": "Fokisun", "vocab": 320, "width": 192, "norm": {"eps": 1e-6}, "residual_mult": 0.8,
            "logit_scale": 0.7,
            "layers": [{"type": "attention", "mixer": _att(6, 3, 64, 64, 0.2, 70, 64, 1e4, 2.0), "mlp": {"kind": "dense", "ff": 256}},
                       {"type": "latent_attention", "mixer": _lat(6, 64, 32, 64, 128, 96, 0.11), "mlp": _moe(6, 2, 96, (3, 2), 1.5, 64)},
                       {"type": "hgrn2", "mixer": _rec(3, 64, 64), "mlp": _moe(4, 1, 64, None, 0.8)},
                       {"type": "attention", "mixer": _att(4, 1, 128, 192, 0.09, 333, 32), "mlp": None},
                       {"type": "latent_attention", "mixer": _lat(4, 96, 32, 128, 232, 80, 0.1), "mlp": {"kind": "dense", "ff": 96}},
                       {"type": "hgrn2", "mixer": _rec(2, 128, 96), "mlp": _moe(8, 3, 96, (4, 2), 1.2, 128)}]}


def _router_margins(model, ids, monkeypatch):
    """Per position, the smallest gap that decides a router's choice over the model's layers: between the last chosen and
    the first rejected score among the kept groups, and between the last kept and the first dropped group."""
    gaps = []
    grouped = hy.moe_grouped

    def spy(x, z, correction, top, groups, keep, *a, **k):
        sc = torch.sigmoid(z.float())
        gap = torch.full((z.shape[0],), 1.0)
        if groups > 1:
            gs = sc.reshape(z.shape[0], groups, -1).sort(-1, descending=True).values[..., :2].sum(-1).sort(-1, descending=True)
            if keep < groups:
                gap = torch.minimum(gap, gs.values[:, keep - 1] - gs.values[:, keep])
            allowed = torch.zeros(z.shape[0], groups, dtype=torch.bool).scatter_(1, gs.indices[:, :keep], True)
            sc = sc.masked_fill(~allowed.repeat_interleave(z.shape[1] // groups, 1), float("-inf"))
        cs = sc.sort(-1, descending=True).values
        if top < z.shape[1]:
            nxt = cs[:, top]
            gap = torch.minimum(gap, torch.where(torch.isinf(nxt), gap, cs[:, top - 1] - nxt))
        gaps.append(gap)
        return grouped(x, z, correction, top, groups, keep, *a, **k)

    monkeypatch.setattr(hy, "moe_grouped", spy)
    with torch.no_grad():
        logits = model(ids).logits[0].numpy()
    monkeypatch.undo()
    return logits, torch.stack(gaps).min(0).values.numpy()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_longer_prompts_at_the_kernel_shapes(dtype, monkeypatch):
    """600 tokens in uneven portions (prompt-sized GEMMs with bf16 activations, the flash prefill at unaligned slots, scan
    segments, decode over several key splits and past the windows) on the GPU against the framework's fp32 CPU path, which
    the tests above tie to the oracle. Positions where a router's choice hangs on a gap that bf16 rounding can close are
    left out of the bf16 comparison, and so is what such a position's other expert moves behind it (its keys and state)."""
    cfg = cfg_kernel_shapes()
    ref_model, sd = build(cfg, "cpu", F32)
    t = toks(600, 320, seed=21)
    ref, gap = _router_margins(ref_model, torch.tensor([t], dtype=torch.int32), monkeypatch)
    clear = gap > (0.01 if dtype == BF16 else 1e-4)
    assert clear.sum() > 200
    model = FokisunForCausalLM(FokisunConfig.from_dict(cfg), device="cuda", dtype=dtype, _do_init=False).load_state_dict(sd)
    got = run_portions(model, t, [261, 3, 2, 190, 64, 37] + [1] * 43)
    e = np.array([err(got[i], ref[i]) for i in range(600)])
    assert np.isfinite(got).all()
    assert np.median(e[clear]) < (1e-5 if dtype == F32 else 2e-2)
    assert e[clear].max() < (2e-4 if dtype == F32 else 1e-1), (int(np.argmax(e * clear)), e[clear].max())
    whole = run_portions(model, t, [600])
    assert err(whole[clear], got[clear]) < (2e-5 if dtype == F32 else 3e-2)
