"""Plain, slow float64 implementation of the Fokisun decoder for the tests: one function per mechanism, written from the
equations, no cache (a whole sequence is recomputed from its first token; every head's keys and values are materialised)
and no code shared with the package. Inputs: the config as a plain dict (the config.json layout) and a checkpoint-named
dict of tensors.

Equations (eps = norm.eps, m = residual_mult, n(y; g) = y / sqrt(mean(y^2) + eps) * g):
  squash norm  T(x; alpha, g, b) = tanh(alpha x) g + b, element by element, no statistic
  layer i      h = T(x; norm1);  X_(i+1) = x + m (mixer(h) + ff(h));  the next layer's x = sum_{j <= i+1} dwa_i[j] X_j,
               X_0 = embed[token] and x = X_0 for layer 0
  attention    q = n(W_q h + b_q; q.norm), k = n(W_k h + b_k; k.norm), each over the whole projection, v = W_v h + b_v
               heads of q / k rotated: pair (2c, 2c+1), c < dims / 2, by p * base^(-2c / dims) / factor
               in a v_mix layer behind the first one, v <- (1 - vmix) v + vmix * (v of the first v_mix layer, same token)
               s_ij = scale * q_i . k_j for 0 <= i - j < mask.size;  p_ij = e^{s_ij} / (1 + sum_j e^{s_ij})
               out = W_o (concat_heads(sum_j p_ij v_j) * sigmoid(W_g h)) + b_o      (query head a: kv head a // (H / G))
  latent attn  q = W_uq n(W_dq h; dq.norm), per head [dim plain | rot_dim rotated];  [c' | r] = W_dkv h
               c = n(c'; dkv.norm), r rotated (one per token for all heads); pair (c, c + dims/2) by p * base^(-2c / dims)
               per head: s_ij = scale (q_plain_i . (W_uk c_j) + q_rot_i . r_j), j <= i;  softmax
               out = W_o concat_heads(sigmoid(W_g h)_a * sum_j p_ij W_uv c_j)
  hgrn2        f = l + (1 - l) sigmoid(W_f h + f.b), l = lower;  q = silu(W_q h);  v = W_v h;  per head
               S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,  o_t = S_t^T q_t;  out = W_o concat_heads(n(o; norm))
  dense ff     W_down (gelu(W_gate h) * W_up h), gelu(z) = z/2 (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))
  moe          s = sigmoid(W_router h); groups of neighbours, a group's score = its two largest s summed; the `top` largest
               s inside the groups.keep best groups are chosen; weight = router.scale * s / (sum of the chosen s + 1e-20)
               out = sum_chosen weight_e expert_e(h) + shared(h), expert(h) = W_down (silu(W_gate h) * W_up h)
  logits       logit_scale * embed T(x; final.norm)
"""
import numpy as np


def _np(t):
    return t.detach().to("cpu").double().numpy() if hasattr(t, "detach") else np.asarray(t, dtype=np.float64)


def rms(y, eps):
    return y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def squash(w, name, x):
    return np.tanh(float(_np(w[name + ".alpha"]).reshape(-1)[0]) * x) * _np(w[name]) + _np(w[name + ".b"])


def rotate(x, pos, rot, adjacent):
    """``x [t, heads, n]``: the first ``rot.dims`` numbers of a head turned in pairs, adjacent numbers (2c, 2c + 1) or
    numbers half the rotated part apart (c, c + dims / 2)."""
    out = x.copy()
    dims = rot["dims"]
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    for c in range(dims // 2):
        a, b = (2 * c, 2 * c + 1) if adjacent else (c, c + dims // 2)
        ang = (np.asarray(pos, dtype=np.float64) * float(rot["base"]) ** (-2.0 * c / dims) / factor)[:, None]
        u, v = x[..., a], x[..., b]
        out[..., a] = u * np.cos(ang) - v * np.sin(ang)
        out[..., b] = v * np.cos(ang) + u * np.sin(ang)
    return out


def weights_of(q, k, scale, window, extra):
    """One head's weights ``[t, t]``: the last ``window`` keys up to the query's own (None: all), ``extra`` in the
    denominator beside the exponentials."""
    t = q.shape[0]
    w = np.zeros((t, t))
    for i in range(t):
        lo = 0 if not window else max(0, i - window + 1)
        s = (k[lo:i + 1] @ q[i]) * scale
        top = max(s.max(), 0.0) if extra else s.max()
        e = np.exp(s - top)
        w[i, lo:i + 1] = e / (e.sum() + extra * np.exp(-top))
    return w


def attention_values(w, pre, mc, h):
    g, dv = mc.get("kv_heads", mc["heads"]), mc.get("vdim", mc["dim"])
    return (h @ _np(w[pre + "v"]).T + _np(w[pre + "v.b"])).reshape(-1, g, dv)


def attention(w, pre, mc, h, eps, v_first=None, pos=None, return_weights=False):
    """``v_first``: the first v_mix layer's values (None: this layer's own are used as they are)."""
    t = h.shape[0]
    pos = np.arange(t) if pos is None else np.asarray(pos)
    nh, d = mc["heads"], mc["dim"]
    g, dv = mc.get("kv_heads", nh), mc.get("vdim", d)
    q = rms(h @ _np(w[pre + "q"]).T + _np(w[pre + "q.b"]), eps) * _np(w[pre + "q.norm"])
    k = rms(h @ _np(w[pre + "k"]).T + _np(w[pre + "k.b"]), eps) * _np(w[pre + "k.norm"])
    q, k = q.reshape(t, nh, d), k.reshape(t, g, d)
    if mc.get("rot"):
        q, k = rotate(q, pos, mc["rot"], True), rotate(k, pos, mc["rot"], True)
    v = attention_values(w, pre, mc, h)
    if v_first is not None:
        lam = float(_np(w[pre + "vmix"]).reshape(-1)[0])
        v = (1.0 - lam) * v + lam * v_first
    window = (mc.get("mask") or {}).get("size")
    o = np.zeros((t, nh, dv))
    pw = np.zeros((nh, t, t))
    for a in range(nh):
        kv = a // (nh // g)
        pw[a] = weights_of(q[:, a], k[:, kv], mc["scale"], window, 1.0)
        o[:, a] = pw[a] @ v[:, kv]
    o = o.reshape(t, nh * dv) * sigmoid(h @ _np(w[pre + "g"]).T)
    out = o @ _np(w[pre + "o"]).T + _np(w[pre + "o.b"])
    return (out, pw) if return_weights else out


def latent_attention(w, pre, mc, h, eps, pos=None, return_weights=False):
    t = h.shape[0]
    pos = np.arange(t) if pos is None else np.asarray(pos)
    nh, d, dr, dv, rank = mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"], mc["kv_rank"]
    q = (rms(h @ _np(w[pre + "dq"]).T, eps) * _np(w[pre + "dq.norm"])) @ _np(w[pre + "uq"]).T
    q = q.reshape(t, nh, d + dr)
    down = h @ _np(w[pre + "dkv"]).T
    c = rms(down[:, :rank], eps) * _np(w[pre + "dkv.norm"])
    r = rotate(down[:, None, rank:], pos, mc["rot"], False)[:, 0]
    q_rot = rotate(q[:, :, d:], pos, mc["rot"], False)
    k = (c @ _np(w[pre + "uk"]).T).reshape(t, nh, d)
    v = (c @ _np(w[pre + "uv"]).T).reshape(t, nh, dv)
    gate = sigmoid(h @ _np(w[pre + "g"]).T)
    o = np.zeros((t, nh, dv))
    pw = np.zeros((nh, t, t))
    for a in range(nh):
        pw[a] = weights_of(np.concatenate([q[:, a, :d], q_rot[:, a]], -1), np.concatenate([k[:, a], r], -1),
                           mc["scale"], None, 0.0)
        o[:, a] = (pw[a] @ v[:, a]) * gate[:, a:a + 1]
    out = o.reshape(t, nh * dv) @ _np(w[pre + "o"]).T
    return (out, pw) if return_weights else out


def hgrn2(w, pre, mc, h, eps, state=None, return_state=False):
    t = h.shape[0]
    nh, d = mc["heads"], mc["dim"]
    dv = mc.get("vdim", d)
    q = silu(h @ _np(w[pre + "q"]).T).reshape(t, nh, d)
    v = (h @ _np(w[pre + "v"]).T).reshape(t, nh, dv)
    low = _np(w[pre + "lower"]).reshape(-1)
    f = (low + (1.0 - low) * sigmoid(h @ _np(w[pre + "f"]).T + _np(w[pre + "f.b"]))).reshape(t, nh, d)
    s = np.zeros((nh, d, dv)) if state is None else np.array(state, dtype=np.float64)
    o = np.zeros((t, nh, dv))
    for i in range(t):
        for a in range(nh):
            s[a] = f[i, a][:, None] * s[a] + (1.0 - f[i, a])[:, None] * v[i, a][None, :]
            o[i, a] = s[a].T @ q[i, a]
    out = (rms(o, eps) * _np(w[pre + "norm"])).reshape(t, nh * dv) @ _np(w[pre + "o"]).T
    return (out, s) if return_state else out


def gated_ff(w, pre, h, act):
    return (act(h @ _np(w[pre + "gate"]).T) * (h @ _np(w[pre + "up"]).T)) @ _np(w[pre + "down"]).T


def route(w, pre, fc, h):
    """Per token: the chosen experts, largest score first (ties to the lower number), and their weights."""
    rc = fc["router"]
    s = sigmoid(h @ _np(w[pre + "router"]).T)
    choice = s.copy()
    gr = rc.get("groups")
    if gr:
        per = s.shape[1] // gr["count"]
        for i in range(h.shape[0]):
            score = [np.sort(s[i, a * per:(a + 1) * per])[-2:].sum() for a in range(gr["count"])]
            best = sorted(range(gr["count"]), key=lambda a: (-score[a], a))[:gr["keep"]]
            for a in range(gr["count"]):
                if a not in best:
                    choice[i, a * per:(a + 1) * per] = -np.inf
    order = np.argsort(-choice, axis=-1, kind="stable")[:, :rc["top"]]
    sel = np.take_along_axis(s, order, -1)
    return order, sel / (sel.sum(-1, keepdims=True) + 1e-20) * rc.get("scale", 1.0)


def moe(w, pre, fc, h):
    chosen, weight = route(w, pre, fc, h)
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e, s in zip(chosen[i], weight[i]):
            out[i] += s * gated_ff(w, f"{pre}e{e}.", h[i][None], silu)[0]
    if fc.get("shared"):
        out += gated_ff(w, pre + "shared.", h, silu)
    return out


def depth_average(coef, states):
    """``sum_j coef[j] states[j]``."""
    out = np.zeros_like(states[0])
    for c, x in zip(_np(coef).reshape(-1), states):
        out += c * x
    return out


def forward(cfg, w, tokens, pos=None):
    """Logits ``[t, vocab]`` and what every layer hands on ``[layers, t, width]``."""
    eps, m = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    x = _np(w["embed"])[np.asarray(tokens)]
    states, hidden, v_first = [x], [], None
    for i, lc in enumerate(cfg["layers"]):
        p, mc, fc = f"l{i}.", lc["mixer"], lc.get("mlp")
        h = squash(w, p + "norm1", x)
        if lc["type"] == "attention":
            mix = bool(mc.get("v_mix"))
            y = attention(w, p + "mix.", mc, h, eps, v_first if mix else None, pos)
            if mix and v_first is None:
                v_first = attention_values(w, p + "mix.", mc, h)
        elif lc["type"] == "latent_attention":
            y = latent_attention(w, p + "mix.", mc, h, eps, pos)
        else:
            y = hgrn2(w, p + "mix.", mc, h, eps)
        if fc is not None:
            y = y + (gated_ff(w, p + "mlp.", h, gelu) if fc["kind"] == "dense" else moe(w, p + "mlp.", fc, h))
        states.append(x + m * y)
        x = depth_average(w[p + "dwa"], states)
        hidden.append(x)
    return cfg.get("logit_scale", 1.0) * (squash(w, "final.norm", x) @ _np(w["embed"]).T), np.stack(hidden)
