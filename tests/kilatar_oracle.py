"""Plain, slow oracle of the Kilatar design for the tests: one function per
mechanism, whole sequences, dense [T, T] score matrices, token-by-token
recurrences, every expert of every token on its own, float64 throughout.  It
shares nothing with the engine's model, ops or kernels; it consumes a config
dict (the keys of a checkpoint's config.json) and a name -> tensor dict in the
checkpoint's naming.

Notation: T tokens of one sequence at positions 0 .. T-1; x [T, width] the
residual, h = rms(x) w the one normed input that a layer's mixer and its
feed-forward both read; weights stored [out, in], applied as h @ W^T.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0.0)


# ----------------------------------------------------------------- positions
def frequencies(rot):
    """Angle per position of every rotated pair, with the banded scaling where the config gives it:
    short wavelengths stay, long ones are divided by the factor, a linear blend in between."""
    out = []
    sc = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if sc:
            turns = sc["original"] * f / (2.0 * math.pi)  # how often the wave fits the original length
            s = min(max((turns - sc["low"]) / (sc["high"] - sc["low"]), 0.0), 1.0)
            f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_pairs(x, pos, rot):
    """x [T, H, n]: columns (2i, 2i+1), i < dims/2, rotated by pos * f_i."""
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        a = pos.to(F) * f
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


# ----------------------------------------------------------------- attention
def visible(T, chunk=0):
    """[T, T] of i, j: j <= i, and with `chunk` both in the same chunk of positions."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    return m & (i // chunk == j // chunk) if chunk else m


def softmax_attention(q, k, v, scale, vis):
    """q, k [T, d], v [T, dv] of one head."""
    return torch.softmax((q @ k.T * scale).masked_fill(~vis, float("-inf")), -1) @ v


def latent_attention(h, p, m, eps):
    T = h.shape[0]
    H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos, vis = torch.arange(T), visible(T)
    q = (h @ p["q"].T).view(T, H, d + dr)
    down = h @ p["dkv"].T
    c = unit_rms(down[:, :r], eps) * p["dkv.norm"]
    kr = rotate_pairs(down[:, None, r:], pos, m["rot"])[:, 0]  # one rotated part for all heads
    k, v = (c @ p["uk"].T).view(T, H, d), (c @ p["uv"].T).view(T, H, dv)
    qr = rotate_pairs(q[..., d:], pos, m["rot"])
    o = torch.stack([softmax_attention(torch.cat([q[:, i, :d], qr[:, i]], -1), torch.cat([k[:, i], kr], -1), v[:, i],
                                       m["scale"], vis) for i in range(H)], 1).reshape(T, H * dv)
    return (o * sigmoid(h @ p["g"].T)) @ p["o"].T


def chunk_attention(h, p, m):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos, vis = torch.arange(T), visible(T, int((m.get("mask") or {}).get("size") or 0))
    q, k, v = (h @ p["q"].T).view(T, H, d), (h @ p["k"].T).view(T, G, d), (h @ p["v"].T).view(T, G, dv)
    if m.get("rot"):
        q, k = rotate_pairs(q, pos, m["rot"]), rotate_pairs(k, pos, m["rot"])
    o = torch.stack([softmax_attention(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], vis)
                     for i in range(H)], 1).reshape(T, H * dv)
    return o @ p["o"].T


# ----------------------------------------------------------------- recurrences
def lightning_scan(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv]:  S_t = decay_h S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    o = torch.zeros(T, H, v.shape[-1], dtype=F)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + torch.outer(k[t, h], v[t, h])
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def lightning(h, p, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = silu(h @ p["q"].T).view(T, H, d), silu(h @ p["k"].T).view(T, H, d), silu(h @ p["v"].T).view(T, H, dv)
    o, _ = lightning_scan(q, k, v, m["decay"])
    return (unit_rms(o.reshape(T, H * dv), eps) * p["norm"] * sigmoid(h @ p["g"].T)) @ p["o"].T


def parallel(h, p, m, eps):
    def sub(side):
        return {k[len(side) + 1:]: v for k, v in p.items() if k.startswith(side + ".")}

    lo, ro = chunk_attention(h, sub("left"), m["left"]), lightning(h, sub("right"), m["right"], eps)
    return 0.5 * (unit_rms(lo, eps) * p["left.out"] + unit_rms(ro, eps) * p["right.out"])


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


def mamba2(h, p, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, x, B, C, dt = torch.split(h @ p["in"].T, [inner, inner, G * N, G * N, H], -1)
    xbc = silu(channel_conv(torch.cat([x, B, C], -1), p["conv"], p["conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    y, _ = ssd_scan(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + p["dt_bias"]), p["A_log"],
                    p["D"])
    y = (y.reshape(T, inner) * silu(z)).view(T, m["norm_groups"], -1)  # the gate, then the norm in equal parts
    return (unit_rms(y, eps).reshape(T, inner) * p["norm"]) @ p["o"].T


MIXERS = {"latent_attention": latent_attention, "mamba2": mamba2, "parallel": parallel}


# ----------------------------------------------------------------- feed-forwards
def dense_ff(h, p):
    g, u = h @ p["gate"].T + p["gate.b"], h @ p["up"].T + p["up.b"]
    return (gelu_tanh(g) * u) @ p["down"].T + p["down.b"]


def expert(h, p, pre):
    return (silu(h @ p[pre + "gate"].T) * (h @ p[pre + "up"].T)) @ p[pre + "down"].T


def route(z, correction, top, scale):
    """z [n] of one token -> (chosen outputs, their weights)."""
    s = torch.exp(z - z.max())
    s = s / s.sum()
    order = sorted(range(len(s)), key=lambda e: -float(s[e] + correction[e]))[:top]
    w = torch.stack([s[e] for e in order])
    return order, w / (w.sum() + 1e-20) * scale


def moe_ff(h, p, mlp):
    r, T = mlp["router"], h.shape[0]
    z = h @ p["router"].T
    corr = p.get("correction", torch.zeros(z.shape[1], dtype=F))
    y = torch.zeros_like(h)
    for t in range(T):
        for e, w in zip(*route(z[t], corr, r["top"], float(r["scale"]))):
            y[t] += w * (expert(h[t], p, f"e{e}.") if e < r["experts"] else h[t])
    if mlp.get("shared"):
        y = y + expert(h, p, "shared.") * sigmoid(h @ p["shared.sg"].T)
    return y


def feed_forward(h, p, mlp):
    return dense_ff(h, p) if mlp["kind"] == "dense" else moe_ff(h, p, mlp)


# ----------------------------------------------------------------- the model
def layer_order(cfg):
    """(layer, whether the embedding output is added in front of it) of every layer run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    body = list(range(lp["start"], lp["stop"]))
    runs = [(i, False) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t > 0 and i == body[0]) for i in body]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg: dict, sd: dict, tokens):
    """Logits [T, vocab] of one sequence, and the residual after every layer run."""
    sd = {k: v.to(F) for k, v in sd.items()}
    eps = float(cfg["norm"]["eps"])
    x0 = unit_rms(sd["embed"][torch.as_tensor(tokens)], eps) * sd["embed.norm"]
    x, after = x0, []
    for i, again in layer_order(cfg):
        L, pre = cfg["layers"][i], f"l{i}."
        p = {k[len(pre) + 4:]: v for k, v in sd.items() if k.startswith(pre + "mix.")}
        if again:
            x = x + x0
        h = unit_rms(x, eps) * sd[pre + "norm1"]
        y = MIXERS[L["type"]](h, p, L["mixer"], eps)
        if L.get("mlp"):
            y = y + feed_forward(h, {k[len(pre) + 4:]: v for k, v in sd.items() if k.startswith(pre + "mlp.")}, L["mlp"])
        x = x + y
        after.append(x)
    return (unit_rms(x, eps) * sd["final.norm"]) @ sd["head"].T, after
