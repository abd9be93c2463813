"""A plain, slow float64 statement of the Tugelorn decoder and of the mechanisms it is made of, one function per mechanism: the
yardstick of tests/test_*tugelorn*.py.  It shares no code with the product path, keeps whole sequences in memory and walks the
delta rule token by token.

Weights come as a dict name -> float64 array; a config is the parsed config.json."""
import numpy as np

from plain_hybrid import causal_conv, rms, silu, softplus, under


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def rotate_pairs(x, positions, base, dims, factor):
    """x [t, heads, d]: the first `dims` elements are rotated in neighbouring pairs (2 i, 2 i + 1), the others pass; the angle of pair i
    is position * base^(-2 i / dims) / factor."""
    freq = float(base) ** (-2.0 * np.arange(dims // 2) / dims) / factor
    ang = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def query_temperature(positions, coef, every):
    """What the queries at these positions are multiplied by."""
    return 1.0 + coef * np.log(np.floor((np.asarray(positions, np.float64) + 1.0) / every) + 1.0)


def grouped_attention(q, k, v, scale, window=None, first=0):
    """q [t, H, d] at positions first .. first + t - 1, k [s, G, d], v [s, G, vd] of positions 0 .. s - 1 (s = first + t); query head h
    reads key head h // (H / G).  window: a position sees itself and the window - 1 positions in front of it."""
    t, H = q.shape[:2]
    per = H // k.shape[1]
    out = np.zeros((t, H, v.shape[2]))
    for i in range(t):
        p = first + i
        lo = 0 if window is None else max(0, p - window + 1)
        for h in range(H):
            s = k[lo : p + 1, h // per] @ q[i, h] * scale
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[lo : p + 1, h // per]
    return out


def attention(h, w, mc, kind):
    t, H, G, d, vd = len(h), mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    bias = lambda n: w[n + ".b"] if kind == "attention_2" else 0.0
    q = (h @ w["q"].T + bias("q")).reshape(t, H, d)
    k = (h @ w["k"].T + bias("k")).reshape(t, G, d)
    v = (h @ w["v"].T + bias("v")).reshape(t, G, vd)
    pos, window = np.arange(t), None
    if kind == "attention":
        rot = mc["rot"]
        q, k = (rotate_pairs(x, pos, rot["base"], rot["dims"], rot["scaling"]["factor"]) for x in (q, k))
        window = mc["mask"]["size"]
    else:
        q = q * query_temperature(pos, mc["q_temp"]["coef"], mc["q_temp"]["every"])[:, None, None]
    return grouped_attention(q, k, v, mc["scale"], window).reshape(t, H * vd) @ w["o"].T


def delta_scan(q, k, v, log_g, beta):
    """q, k [t, G, d] (unit vectors, q scaled), v [t, H, vd], log_g [t, H, d] (<= 0), beta [t, H] -> o [t, H, vd]."""
    t, H, vd = v.shape
    per = H // k.shape[1]
    S, o = np.zeros((H, k.shape[2], vd)), np.zeros_like(v)
    for i in range(t):
        for h in range(H):
            kk, qq = k[i, h // per], q[i, h // per]
            S[h] *= np.exp(log_g[i, h])[:, None]
            S[h] += np.outer(kk, beta[i, h] * (v[i, h] - S[h].T @ kk))
            o[i, h] = S[h].T @ qq
    return o


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def delta_gates(h, w, mc):
    """-> (log of the decays [t, H, d], beta [t, H], output gate [t, H, vd])"""
    t, H, d, vd = len(h), mc["heads"], mc["dim"], mc["vdim"]
    step = softplus(h @ w["a1"].T @ w["a2"].T + w["dt_bias"]).reshape(t, H, d)
    return -np.exp(w["A_log"])[:, None] * step, sigmoid(h @ w["b"].T), sigmoid(h @ w["g1"].T @ w["g2"].T).reshape(t, H, vd)


def channel_delta(h, w, mc, eps):
    t, H, G, d, vd = len(h), mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"], 0.0)) for n in "qkv")
    q, k, v = unit(q.reshape(t, G, d)) * d ** -0.5, unit(k.reshape(t, G, d)), v.reshape(t, H, vd)
    log_g, beta, gate = delta_gates(h, w, mc)
    o = rms(delta_scan(q, k, v, log_g, beta), eps) * w["norm"] * gate
    return o.reshape(t, H * vd) @ w["o"].T


def clamped_glu(gate, up, limit, alpha=1.702):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(alpha * g) * (u + 1.0)


def layer_runs(cfg):
    """(layer, whether a pass but the first starts here) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b = loop["start"], loop["stop"]
    runs = [(i, False) for i in range(a)]
    for p in range(loop["times"]):
        runs += [(i, p > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, weights, tokens, layer_outputs=None):
    """Logits [t, vocab] of the whole sequence at once.  layer_outputs: a list that receives the residual behind every layer run."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    embedded = weights["embed"][np.asarray(tokens)]
    x = embedded
    norm = lambda v, name: rms(v, eps) * weights[name]
    for i, again in layer_runs(cfg):
        if again:
            x = x + embedded
        layer, p = cfg["layers"][i], f"l{i}."
        w, h = under(weights, p + "mix."), norm(x, p + "norm1")
        y = channel_delta(h, w, layer["mixer"], eps) if layer["type"] == "channel_delta" else attention(h, w, layer["mixer"], layer["type"])
        x = x + m * norm(y, p + "norm1b")
        if layer["mlp"]:
            w, h = under(weights, p + "mlp."), norm(x, p + "norm2")
            y = clamped_glu(h @ w["gate"].T, h @ w["up"].T, layer["mlp"]["limit"]) @ w["down"].T
            x = x + m * norm(y, p + "norm2b")
        if layer_outputs is not None:
            layer_outputs.append(x.copy())
    return norm(x, "final.norm") @ weights["head"].T
