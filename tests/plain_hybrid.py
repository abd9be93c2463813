"""A plain, slow float64 statement of the Tanolorn decoder and of the mechanisms it is made of, one function per
mechanism: the yardstick of tests/test_hybrid_*.py.  It shares no code with the product path, keeps whole sequences in
memory and walks recurrences token by token.

Weights come as a dict name -> float64 array; a config is the parsed config.json."""
import numpy as np


def rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def silu(z):
    return z / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def rotate_half(x, positions, base, dims):
    """x [t, heads, d]: the first `dims` elements are rotated in pairs (i, i + dims / 2), the others pass."""
    half = dims // 2
    freq = float(base) ** (-2.0 * np.arange(half) / dims)
    ang = np.asarray(positions, np.float64)[:, None] * freq[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def latent_rows(h, w, mc, eps):
    """The cached rows of a layer that has its own: (c [t, kv_rank], rotated key part [t, rot_dim]) for positions 0 .. t - 1."""
    r = mc["kv_rank"]
    kv = h @ w["dkv"].T
    c = rms(kv[:, :r], eps) * w["dkv.norm"]
    k_rot = rotate_half(kv[:, None, r:], np.arange(len(h)), mc["rot"]["base"], mc["rot"]["dims"])[:, 0]
    return c, k_rot


def latent_attention(h, w, mc, eps, latent):
    """h [t, width] -> [t, width] over the latent rows of the same positions."""
    t, H, d, rd, vd = len(h), mc["heads"], mc["dim"], mc["rot_dim"], mc["vdim"]
    c, k_rot = latent
    q = ((rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).reshape(t, H, d + rd)
    q_rot = rotate_half(q[..., d:], np.arange(t), mc["rot"]["base"], mc["rot"]["dims"])
    k = (c @ w["uk"].T).reshape(t, H, d)
    v = (c @ w["uv"].T).reshape(t, H, vd)
    out = np.zeros((t, H, vd))
    for i in range(t):
        for hh in range(H):
            s = (k[: i + 1, hh] @ q[i, hh, :d] + k_rot[: i + 1] @ q_rot[i, hh]) * mc["scale"]
            p = np.exp(s - s.max())
            out[i, hh] = (p / p.sum()) @ v[: i + 1, hh]
    return out.reshape(t, H * vd) @ w["o"].T


def causal_conv(x, taps, bias):
    """x [t, channels]; taps [channels, n], the last column meets the current row; zeros before the start."""
    n = taps.shape[1]
    pad = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return sum(pad[j : j + len(x)] * taps[:, j] for j in range(n)) + bias


def ssm_scan(x, B, C, dt, A_log, D):
    """x [t, heads, vdim], B and C [t, groups, N], dt [t, heads] (after softplus) -> y [t, heads, vdim]."""
    t, heads, vd = x.shape
    per = heads // B.shape[1]
    S = np.zeros((heads, B.shape[2], vd))
    y = np.zeros_like(x)
    for i in range(t):
        for hh in range(heads):
            g = hh // per
            S[hh] = np.exp(-np.exp(A_log[hh]) * dt[i, hh]) * S[hh] + dt[i, hh] * np.outer(B[i, g], x[i, hh])
            y[i, hh] = S[hh].T @ C[i, g] + D[hh] * x[i, hh]
    return y


def grouped_gated_norm(y, z, weight, groups, eps):
    g = y * silu(z)
    t, n = g.shape
    return rms(g.reshape(t, groups, n // groups), eps).reshape(t, n) * weight


def mamba2(h, w, mc, eps):
    t, H, vd, N, G = len(h), mc["heads"], mc["vdim"], mc["state"], mc["groups"]
    inner, gn = H * vd, G * N
    p = h @ w["in"].T
    z, xbc, dt = p[:, :inner], p[:, inner : 2 * inner + 2 * gn], p[:, 2 * inner + 2 * gn :]
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = xbc[:, :inner], xbc[:, inner : inner + gn], xbc[:, inner + gn :]
    y = ssm_scan(x.reshape(t, H, vd), B.reshape(t, G, N), C.reshape(t, G, N), softplus(dt + w["dt_bias"]), w["A_log"], w["D"]).reshape(t, inner)
    return grouped_gated_norm(y, z, w["norm"], mc["norm_groups"], eps) @ w["o"].T


def dense_ff(h, w):
    a = silu(h @ w["gate"].T + w["gate.b"]) * (h @ w["up"].T + w["up.b"])
    return a @ w["down"].T + w["down.b"]


def route(h, w, rc):
    """One row -> (chosen experts, their weights)."""
    s = 1.0 / (1.0 + np.exp(-(w["router"] @ h)))
    choice = s + w["correction"]
    n, count = rc["experts"], rc["groups"]["count"]
    size = n // count
    best2 = np.array([np.sort(choice[g * size : (g + 1) * size])[::-1][:2].sum() for g in range(count)])
    kept = np.argsort(-best2, kind="stable")[: rc["groups"]["keep"]]
    masked = np.full(n, -np.inf)
    for g in kept:
        masked[g * size : (g + 1) * size] = choice[g * size : (g + 1) * size]
    chosen = np.argsort(-masked, kind="stable")[: rc["top"]]
    return chosen, s[chosen]


def moe_ff(h, w, rc):
    out = np.zeros_like(h)
    for i, row in enumerate(h):
        for e, weight in zip(*route(row, w, rc)):
            a = silu(w[f"e{e}.gate"] @ row) * (w[f"e{e}.up"] @ row)
            out[i] += weight * (w[f"e{e}.down"] @ a)
    return out


def under(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, layer_outputs=None):
    """Logits [t, vocab] of the whole sequence at once.  layer_outputs: a list that receives the residual behind every layer."""
    tokens = np.asarray(tokens)
    eps, x = cfg["norm"]["eps"], weights["embed"][tokens]
    side = cfg["token_side"]["dim"]
    post = lambda y, name: rms(y, eps) * (1.0 + weights[name])
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        w, mc = under(weights, f"l{i}.mix."), layer["mixer"]
        if layer["type"] == "latent_attention":
            latents[i] = latents[mc["kv_from"]] if mc.get("kv_from") is not None else latent_rows(x, w, mc, eps)
            y = latent_attention(x, w, mc, eps, latents[i])
        elif layer["type"] == "mamba2":
            y = mamba2(x, w, mc, eps)
        else:
            raise ValueError(layer["type"])
        x = x + post(y, f"l{i}.norm1")
        if layer["mlp"]:
            w = under(weights, f"l{i}.mlp.")
            y = dense_ff(x, w) if layer["mlp"]["kind"] == "dense" else moe_ff(x, w, layer["mlp"]["router"])
            x = x + post(y, f"l{i}.norm2")
        e = weights["side.embed"][tokens, i * side : (i + 1) * side]
        y = (gelu_tanh(x @ weights[f"l{i}.side.gate"].T) * e) @ weights[f"l{i}.side.proj"].T
        x = x + rms(y, eps) * weights[f"l{i}.side.norm"]
        if layer_outputs is not None:
            layer_outputs.append(x.copy())
    return post(x, "final.norm") @ weights["head"].T
