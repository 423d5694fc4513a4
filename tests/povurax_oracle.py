"""Plain, slow oracle of the Povurax design for the tests: one function per
mechanism, whole sequences, dense [T, T] score matrices, token-by-token
recurrences, float64 throughout.  It shares nothing with the engine's model,
ops or kernels; it consumes a config dict (the keys of a checkpoint's
config.json) and a name -> tensor dict in the checkpoint's naming.

Notation: T tokens of one sequence at positions 0 .. T-1; x [T, width] the
residual, which the sublayers read as it is; weights stored [out, in], applied
as x @ W^T.
"""
from __future__ import annotations

import torch

F = torch.float64
FF_ALPHA = 1.702


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0.0)


# ----------------------------------------------------------------- attention (left half of 'parallel')
def rotate_pairs(x, pos, dims, base):
    """x [T, H, n]: columns (2i, 2i+1), i < dims/2, rotated by pos * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = pos.to(F) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def attention_weights(q, k, scale):
    """q, k [T, d] of one head -> causal softmax weights [T, T]."""
    T = q.shape[0]
    sc = (q @ k.T) * scale
    return torch.softmax(sc.masked_fill(torch.ones(T, T).triu(1).bool(), float("-inf")), -1)


def attention(h, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    # one norm over all heads' rows together, before they are split
    q = (unit_rms(h @ p["q"].T, eps) * p["q.norm"]).view(T, H, d)
    k = (unit_rms(h @ p["k"].T, eps) * p["k.norm"]).view(T, G, d)
    v = (h @ p["v"].T).view(T, G, dv)
    rot = m.get("rot")
    if rot:
        q, k = rotate_pairs(q, pos, rot["dims"], rot["base"]), rotate_pairs(k, pos, rot["dims"], rot["base"])
    o = torch.stack([attention_weights(q[:, i], k[:, i // (H // G)], m["scale"]) @ v[:, i // (H // G)]
                     for i in range(H)], 1).reshape(T, H * dv)
    return (o * sigmoid(h @ p["g"].T)) @ p["o"].T


# ----------------------------------------------------------------- state-space duality (right half)
def channel_conv(u, w, b):
    """y_t = b + sum_j w[:, j] u_(t - taps + 1 + j) per channel, zeros before t = 0."""
    T, taps = u.shape[0], w.shape[1]
    y = b.repeat(T, 1)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def ssd_scan(x, B, C, dt, A_log, D):
    """x [T, H, P], B, C [T, G, N], dt [T, H] (after softplus):
    S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T,   y_t = S_t^T C_t + D x_t."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=F)
    y = torch.zeros(T, H, P, dtype=F)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, w, groups, eps):
    """y silu(z), then every one of `groups` equal parts divided by its own root mean square, times w."""
    T = y.shape[0]
    return unit_rms((y * silu(z)).view(T, groups, -1), eps).reshape(T, -1) * w


def mamba2(h, p, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, x, B, C, dt = torch.split(h @ p["in"].T, [inner, inner, G * N, G * N, H], -1)
    xbc = silu(channel_conv(torch.cat([x, B, C], -1), p["conv"], p["conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    y, _ = ssd_scan(x.view(T, H, P), B.view(T, G, N), C.view(T, G, N), softplus(dt + p["dt_bias"]), p["A_log"], p["D"])
    return gated_group_norm(y.reshape(T, inner), z, p["norm"], m["norm_groups"], eps) @ p["o"].T


def parallel(h, p, m, eps):
    def sub(side):
        return {k[len(side) + 1:]: v for k, v in p.items() if k.startswith(side + ".")}

    return m["left_scale"] * attention(h, sub("left"), m["left"], eps) + \
        m["right_scale"] * mamba2(h, sub("right"), m["right"], eps)


# ----------------------------------------------------------------- gated linear attention
def gla_scan(q, k, v, alpha):
    """q, k, alpha [T, H, d], v [T, H, dv]:  S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    o = torch.zeros(T, H, v.shape[-1], dtype=F)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hi,hij->hj", q[t], S)
    return o, S


def gla(h, p, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ p["k"].T).view(T, H, d)
    v = (h @ p["v"].T).view(T, H, dv)
    z = (h @ p["a1"].T) @ p["a2"].T + p["a2.b"]
    alpha = torch.exp(-softplus(-z) / float(m["tau"])).view(T, H, d)  # sigmoid(z)^(1 / tau)
    o, _ = gla_scan(q, k, v, alpha)
    o = (unit_rms(o, eps) * p["norm"]).reshape(T, H * dv)
    return (o * silu(h @ p["g"].T)) @ p["o"].T


MIXERS = {"parallel": parallel, "gla": gla}


# ----------------------------------------------------------------- feed-forward, the model
def clamped_ff(h, gate, up, down, limit):
    g = (h @ gate.T).clamp(max=limit)
    u = (h @ up.T).clamp(-limit, limit)
    return (g * sigmoid(FF_ALPHA * g) * (u + 1.0)) @ down.T


def forward(cfg: dict, sd: dict, tokens, upto: int | None = None):
    """Logits [T, vocab] of one sequence, and the residual after every layer."""
    sd = {k: v.to(F) for k, v in sd.items()}
    eps = float(cfg["norm"]["eps"])
    x = sd["embed"][torch.as_tensor(tokens)] * float(cfg["embedding"]["scale"])
    after = []
    for i, L in enumerate(cfg["layers"][:upto]):
        pre = f"l{L.get('weights_of', i)}."
        p = {k[len(pre) + 4:]: v for k, v in sd.items() if k.startswith(pre + "mix.")}
        x = x + unit_rms(MIXERS[L["type"]](x, p, L["mixer"], eps), eps) * sd[pre + "norm1"]
        if L.get("mlp"):
            y = clamped_ff(x, sd[pre + "mlp.gate"], sd[pre + "mlp.up"], sd[pre + "mlp.down"], float(L["mlp"]["limit"]))
            x = x + unit_rms(y, eps) * sd[pre + "norm2"]
        after.append(x)
    return (unit_rms(x, eps) * sd["final.norm"]) @ sd["head"].T, after
