"""Plain, slow float64 implementation of the Zopupel decoder for the tests: one function per mechanism, written from the
equations, no cache (a whole sequence is recomputed from its first token) and no code shared with the package. Inputs: the
config as a plain dict (the config.json layout) and a checkpoint-named dict of tensors.

Equations (eps = norm.eps, m = residual_mult, n(y; g) = y / sqrt(mean(y^2) + eps) * g):
  layer        x <- x + m n(mixer(n(x; norm1)); norm1b);  x <- x + m n(ff(n(x; norm2)); norm2b)
  rotation     pair (c, c + dims / 2) of a head's first `dims` numbers turned by p * w_c, w_c from base^(-2c / dims):
               scaling {factor}: w_c / factor
               scaling {factor, original, fast, slow}: between w_c (fast pairs) and w_c / factor (slow pairs), by a ramp in c
               between the pairs that make `fast` and `slow` full turns over `original` positions; cosine and sine times
               0.1 ln(factor) + 1
  attention    differential: q, k hold two maps per head, [map 1 | map 2] of `dim` numbers each, rotated one by one;
               A_b = softmax_j(scale q_b . k_b), j <= i, b = 1, 2, both over the same values;
               lambda = e^(lq1 . lk1) - e^(lq2 . lk2) + diff;  o = A_1 v - lambda A_2 v per head
               out = W_o concat_heads((1 - diff) n(o; 1));  kv_from: keys and values of that layer for the same tokens
  attention_2  q = W_q h + b_q, k = W_k h + b_k, v = k; then q = n(q; q.norm), k = n(k; k.norm), each over the whole
               projection, and rotated;  p_ij = e^{s_ij} / (1 + sum_j e^{s_ij}), s = scale q . k, j <= i
               out = W_o concat_heads(sum_j p_ij v_j) + b_o
  moe          z = W_router h + b; the `top` largest z chosen, weights softmax over the chosen z;
               out = sum weight_e expert_e(h) + shared(h), expert(h) = W_down (silu(W_gate h) * W_up h)
  logits       head n(x; final.norm)
"""
import math

import numpy as np


def _np(t):
    return t.detach().to("cpu").double().numpy() if hasattr(t, "detach") else np.asarray(t, dtype=np.float64)


def rms(y, eps):
    return y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)


def silu(z):
    return z / (1.0 + np.exp(-z))


def turns(rot):
    """``(angle per position of every pair, factor on cosine and sine)`` of a ``rot`` entry."""
    dims, base = rot["dims"], float(rot["base"])
    freq = [base ** (-2.0 * c / dims) for c in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return np.array(freq), 1.0
    factor = float(sc["factor"])
    if "original" not in sc:
        return np.array(freq) / factor, 1.0

    def pair_of(t):  # the (fractional) pair that makes t full turns over the original length
        return dims * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(pair_of(sc["fast"])), 0), min(math.ceil(pair_of(sc["slow"])), dims - 1)
    out = []
    for c, f in enumerate(freq):
        ramp = min(max((c - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * ramp + f * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(factor) + 1.0


def rotate(x, pos, rot):
    """``x [t, heads, n]``, number ``c`` paired with ``c + dims / 2``."""
    out = x.copy()
    half = rot["dims"] // 2
    w, gain = turns(rot)
    for c in range(half):
        ang = (np.asarray(pos, dtype=np.float64) * w[c])[:, None]
        u, v = x[..., c], x[..., c + half]
        out[..., c] = (u * np.cos(ang) - v * np.sin(ang)) * gain
        out[..., c + half] = (v * np.cos(ang) + u * np.sin(ang)) * gain
    return out


def weights_of(q, k, scale, extra):
    """One head's causal weights ``[t, t]``, ``extra`` in the denominator beside the exponentials."""
    t = q.shape[0]
    s = (q @ k.T) * scale
    s[np.triu_indices(t, 1)] = -np.inf
    top = s.max(-1, keepdims=True)
    if extra:
        top = np.maximum(top, 0.0)
    e = np.exp(s - top)
    return e / (e.sum(-1, keepdims=True) + extra * np.exp(-top))


def diff_keys_values(w, pre, mc, h, pos=None):
    """Rotated keys ``[t, G, 2, dim]`` and values ``[t, G, vdim]`` of a differential layer with projections of its own."""
    t = h.shape[0]
    pos = np.arange(t) if pos is None else np.asarray(pos)
    g, d = mc.get("kv_heads", mc["heads"]), mc["dim"]
    k = (h @ _np(w[pre + "k"]).T).reshape(t, g * 2, d)
    if mc.get("rot"):
        k = rotate(k, pos, mc["rot"])
    return k.reshape(t, g, 2, d), (h @ _np(w[pre + "v"]).T).reshape(t, g, mc.get("vdim", d))


def diff_lambda(w, pre, mc):
    a = [_np(w[pre + n]).reshape(-1) for n in ("lq1", "lk1", "lq2", "lk2")]
    return math.exp(float(a[0] @ a[1])) - math.exp(float(a[2] @ a[3])) + mc["diff"]


def attention(w, pre, mc, h, eps, kv=None, pos=None, return_weights=False):
    """``kv``: another layer's keys and values (None: this layer projects its own)."""
    t = h.shape[0]
    pos = np.arange(t) if pos is None else np.asarray(pos)
    nh, d = mc["heads"], mc["dim"]
    g, dv = mc.get("kv_heads", nh), mc.get("vdim", mc["dim"])
    q = (h @ _np(w[pre + "q"]).T).reshape(t, nh * 2, d)
    if mc.get("rot"):
        q = rotate(q, pos, mc["rot"])
    q = q.reshape(t, nh, 2, d)
    k, v = kv if kv is not None else diff_keys_values(w, pre, mc, h, pos)
    lam = diff_lambda(w, pre, mc)
    o = np.zeros((t, nh, dv))
    pw = np.zeros((nh, 2, t, t))
    for a in range(nh):
        kv_a = a // (nh // g)
        for b in range(2):
            pw[a, b] = weights_of(q[:, a, b], k[:, kv_a, b], mc["scale"], 0.0)
        o[:, a] = pw[a, 0] @ v[:, kv_a] - lam * (pw[a, 1] @ v[:, kv_a])
    o = rms(o, eps) * (1.0 - mc["diff"])
    out = o.reshape(t, nh * dv) @ _np(w[pre + "o"]).T
    return (out, pw) if return_weights else out


def attention_2(w, pre, mc, h, eps, pos=None, return_weights=False):
    t = h.shape[0]
    pos = np.arange(t) if pos is None else np.asarray(pos)
    nh, d = mc["heads"], mc["dim"]
    g = mc.get("kv_heads", nh)
    q = h @ _np(w[pre + "q"]).T + _np(w[pre + "q.b"])
    k = h @ _np(w[pre + "k"]).T + _np(w[pre + "k.b"])
    v = k.reshape(t, g, d)
    q = (rms(q, eps) * _np(w[pre + "q.norm"])).reshape(t, nh, d)
    k = (rms(k, eps) * _np(w[pre + "k.norm"])).reshape(t, g, d)
    if mc.get("rot"):
        q, k = rotate(q, pos, mc["rot"]), rotate(k, pos, mc["rot"])
    o = np.zeros((t, nh, d))
    pw = np.zeros((nh, t, t))
    for a in range(nh):
        pw[a] = weights_of(q[:, a], k[:, a // (nh // g)], mc["scale"], 1.0)
        o[:, a] = pw[a] @ v[:, a // (nh // g)]
    out = o.reshape(t, nh * d) @ _np(w[pre + "o"]).T + _np(w[pre + "o.b"])
    return (out, pw) if return_weights else out


def router(w, pre, fc, h):
    """``(chosen [t, top], weights [t, top])``."""
    z = h @ _np(w[pre + "router"]).T + _np(w[pre + "router.b"])
    pick = np.argsort(-z, axis=-1, kind="stable")[:, :fc["router"]["top"]]
    zc = np.take_along_axis(z, pick, -1)
    e = np.exp(zc - zc.max(-1, keepdims=True))
    return pick, e / e.sum(-1, keepdims=True)


def expert(w, pre, h):
    return (silu(h @ _np(w[pre + "gate"]).T) * (h @ _np(w[pre + "up"]).T)) @ _np(w[pre + "down"]).T


def mixture(w, pre, fc, h):
    pick, wt = router(w, pre, fc, h)
    out = np.zeros_like(h)
    for e in range(fc["router"]["experts"]):
        weight = (wt * (pick == e)).sum(-1, keepdims=True)
        rows = np.nonzero(weight[:, 0])[0]
        if len(rows):
            out[rows] += weight[rows] * expert(w, f"{pre}e{e}.", h[rows])
    return out + expert(w, pre + "shared.", h) if fc.get("shared") else out


def forward(cfg, w, tokens):
    """``(logits [t, vocab], residual after every layer [layers, t, width])``."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = _np(w["embed"])[np.asarray(tokens)]
    held, streams = {}, []
    for i, ls in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", ls["mixer"]
        h = rms(x, eps) * _np(w[p + "norm1"])
        if ls["type"] == "attention":
            j = mc.get("kv_from")
            if j is None:
                held[i] = diff_keys_values(w, p + "mix.", mc, h)
            y = attention(w, p + "mix.", mc, h, eps, kv=held[i if j is None else j])
        else:
            y = attention_2(w, p + "mix.", mc, h, eps)
        x = x + mult * rms(y, eps) * _np(w[p + "norm1b"])
        if ls.get("mlp") is not None:
            y = mixture(w, p + "mlp.", ls["mlp"], rms(x, eps) * _np(w[p + "norm2"]))
            x = x + mult * rms(y, eps) * _np(w[p + "norm2b"])
        streams.append(x)
    return (rms(x, eps) * _np(w["final.norm"])) @ _np(w["head"]).T, np.stack(streams)
