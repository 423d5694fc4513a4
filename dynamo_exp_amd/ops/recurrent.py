"""Ops with per-sequence state: the generalized delta rule (a running matrix
per head), linear recurrences (a running matrix whose decay is fixed per head:
retention; a function of the token's step size: state-space duality; or one per
key channel and token: gated linear attention), short causal convolutions over
time fused with rotary positions and the paged cache write, the query / key
preparation of latent attention with a rotated key part, and the norms + gates
that follow a recurrent mixer.

State lives in slots: state tensors are [slots, ...], the engine's KV manager
hands a slot to every live request, and a step names the slot of each of its
sequences (`state_slots` [n_seq] int32, -1: a padding row that touches
nothing).  A step's rows are grouped by sequence: `seq_rows` [n_seq + 1] int32
holds the first row of every sequence (None: row i is sequence i, a decode
step); within a sequence rows are consecutive positions.  A sequence whose
first row of the step is at position 0 starts from zero state, whatever its
slot held before, so slots need no clearing when they change hands.

GPU tensors run the gfx950 kernels of ``_C_mixers`` (csrc/mixers/recurrent.hip,
linear_scan.hip);
CPU tensors run the PyTorch forms below.  Decays, removal rates, unit keys and
the state are fp32 in every dtype.
"""
from __future__ import annotations

import math

import torch

from .mixers import _f32, _fp32_param, _m, _ptr, _stream


def _seq_bounds(seq_rows: torch.Tensor | None, n_seq: int) -> list[int]:
    return list(range(n_seq + 1)) if seq_rows is None else seq_rows.tolist()


def _check_step(positions, seq_rows, state_slots):
    if positions.dtype != torch.int64 or state_slots.dtype != torch.int32 or \
            (seq_rows is not None and (seq_rows.dtype != torch.int32 or seq_rows.numel() != state_slots.numel() + 1)):
        raise TypeError("int64 positions, int32 state_slots [n_seq] and seq_rows [n_seq + 1]")


# ----------------------------------------------------------------- rotary frequencies
def rotary_frequencies(dims: int, base: float, scaling: dict | None = None) -> torch.Tensor:
    """f_i = base^(-2 i / dims), i < dims / 2 (fp32, computed in float64).  With
    scaling = {factor, low, high, original}: a frequency whose wavelength
    l = 2 pi / f is below original / high stays, one above original / low is
    divided by factor, and between the two it is (1 - s) f / factor + s f with
    s = (original / l - low) / (high - low)."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            fac, low, high, orig = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            wl = 2.0 * math.pi / f
            if wl > orig / low:
                f = f / fac
            elif wl >= orig / high:
                s = (orig / wl - low) / (high - low)
                f = (1.0 - s) * f / fac + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64).to(torch.float32)


def yarn_frequencies(dims: int, base: float, scaling: dict | None = None) -> tuple[torch.Tensor, float]:
    """(f [dims / 2] fp32, mag): f_i = base^(-2 i / dims), and with scaling =
    {factor, original, fast, slow} (YaRN) the blend
        f_i / factor * ramp_i + f_i * (1 - ramp_i),   ramp_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1)
    between the dimensions lo = max(floor(dim(fast)), 0) and hi = min(ceil(dim(slow)), dims - 1), where
    dim(t) = dims * ln(original / (2 pi t)) / (2 ln base) is the dimension whose wavelength fits t
    times into the original length; mag = 0.1 ln(factor) + 1 multiplies cosines and sines
    (1 without scaling).  Computed in float64."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    mag = 1.0
    if scaling:
        fac, orig = float(scaling["factor"]), float(scaling["original"])

        def dim_of(turns: float) -> float:
            return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(float(base)))

        lo = max(math.floor(dim_of(float(scaling["fast"]))), 0)
        hi = min(math.ceil(dim_of(float(scaling["slow"]))), dims - 1)
        for i in range(dims // 2):
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f[i] = f[i] / fac * ramp + f[i] * (1.0 - ramp)
        mag = 0.1 * math.log(fac) + 1.0
    return torch.tensor(f, dtype=torch.float64).to(torch.float32), mag


def latent_rope(qa: torch.Tensor, q: torch.Tensor, q_head: int, q_off: int, kv: torch.Tensor, r: int, dr: int,
                norm_w: torch.Tensor, eps: float, inv_freq: torch.Tensor | None, mag: float,
                positions: torch.Tensor, kv_slots: torch.Tensor, cache: torch.Tensor,
                interleaved: bool = False) -> torch.Tensor:
    """Query / key preparation of latent attention with a rotated key part.
    Per token row t: the latent kv[t, :r] is RMS-normed (weight norm_w) into
    cache[slot, :r]; the key part kv[t, r:r + dr], shared by all heads and not
    normed, is rotated into cache[slot, r:]; and head h's query is assembled
    as [qa[h, t] (r) | rotate(q[t, h * q_head + q_off : + dr])] -- qa [H, T, r]
    is the head's unrotated query part already times the head's key
    up-projection.  Returns q' [T, H * (r + dr)].  Rotation: the first
    2 len(inv_freq) columns of a part, column i paired with i + len(inv_freq)
    (interleaved: column 2 i with 2 i + 1), by the angle position * inv_freq[i], cosines and sines times mag; the rest
    pass unchanged.  Rows with slot < 0 cache nothing."""
    H, T, _ = qa.shape
    half = 0 if inv_freq is None else inv_freq.numel()
    _fp32_param(norm_w, "norm_w")
    _fp32_param(inv_freq, "inv_freq")
    Wc = r + dr
    if qa.shape != (H, T, r) or not qa.is_contiguous() or kv.shape[0] != T or kv.shape[1] < Wc or kv.stride(1) != 1 or \
            q.shape[0] != T or q.stride(1) != 1 or q.shape[1] < (H - 1) * q_head + q_off + dr or 2 * half > dr or \
            q_off + dr > q_head or norm_w.numel() != r:
        raise ValueError("latent_rope: sections do not fit the rows")
    if cache.shape[-1] != Wc or not cache.is_contiguous() or any(t.dtype != qa.dtype for t in (q, kv, cache)):
        raise ValueError("latent_rope: cache rows are [latent | rotated key] of the activation dtype")
    if not qa.is_cuda:
        def rot(x):  # [T, ..., dr]
            if not half:
                return x
            ang = positions.to(torch.float32)[:, None] * inv_freq[None, :]
            shape = [T] + [1] * (x.dim() - 2) + [half]
            c, s_ = (torch.cos(ang) * mag).view(shape), (torch.sin(ang) * mag).view(shape)
            if interleaved:
                a_, b_ = x[..., 0:2 * half:2], x[..., 1:2 * half:2]
                y = torch.stack([a_ * c - b_ * s_, b_ * c + a_ * s_], -1).flatten(-2)
                return torch.cat([y, x[..., 2 * half:]], -1)
            a_, b_ = x[..., :half], x[..., half:2 * half]
            return torch.cat([a_ * c - b_ * s_, b_ * c + a_ * s_, x[..., 2 * half:]], -1)

        kvf = kv.float()
        c = kvf[:, :r]
        c = c * torch.rsqrt((c * c).mean(-1, keepdim=True) + eps) * norm_w
        row = torch.cat([c, rot(kvf[:, r:Wc])], -1).to(cache.dtype)
        ok = kv_slots >= 0
        cache[kv_slots[ok]] = row[ok]
        qr = torch.stack([q[:, h * q_head + q_off:h * q_head + q_off + dr] for h in range(H)], 1).float()
        out = torch.cat([qa.transpose(0, 1).float(), rot(qr)], -1).to(qa.dtype)
        return out.reshape(T, H * Wc)
    if positions.dtype != torch.int64 or kv_slots.dtype != torch.int64:
        raise TypeError("latent_rope: int64 positions and kv_slots")
    out = torch.empty((T, H * Wc), dtype=qa.dtype, device=qa.device)
    _m().latent_rope(out.data_ptr(), qa.data_ptr(), q.data_ptr(), q.stride(0), q_head, q_off, kv.data_ptr(),
                     kv.stride(0), norm_w.data_ptr(), float(eps), _ptr(inv_freq), half, float(mag),
                     positions.data_ptr(), kv_slots.data_ptr(), cache.data_ptr(), T, H, r, dr, int(interleaved), _f32(qa),
                     _stream())
    return out


# ----------------------------------------------------------------- short convolution + rotary + cache write
def conv_rope_cache(x: torch.Tensor, conv_w: torch.Tensor, conv_state: torch.Tensor, positions: torch.Tensor,
                    kv_slots: torch.Tensor, row_seq: torch.Tensor | None, seq_rows: torch.Tensor | None,
                    state_slots: torch.Tensor, n_q: int, n_k: int, d: int, dv: int, inv_freq: torch.Tensor | None,
                    kc: torch.Tensor | None, vc: torch.Tensor | None, bias: torch.Tensor | None = None,
                    act: str | None = None) -> torch.Tensor:
    """Per row of a fused projection x = [q (n_q d) | k (n_k d) | v (n_k dv) | ...]:
    every channel c of the C = n_q d + n_k (d + dv) leading columns is
    convolved over time, y_t = sum_j conv_w[j, c] u_(t - taps + 1 + j) (conv_w
    [taps, C] fp32, tap-major: the transpose of a checkpoint's [C, taps]), where u
    at a position before the step's first row of the sequence comes from
    conv_state [slots, taps - 1, C] (the last taps - 1 projected rows the
    sequence had before this step) and is zero before position 0; with bias
    [C] (fp32) y_t += bias, and with act 'silu' y_t <- y_t sigmoid(y_t).  Then the
    first 2 len(inv_freq) columns of every q and k head are rotated by the
    angles position * inv_freq, column i paired with column i + len(inv_freq).
    Returns q [T, n_q d]; k and v go to the paged caches kc [slots, n_k d],
    vc [slots, n_k dv] at kv_slots (rows with slot < 0 cache nothing; n_k = 0:
    no caches, a layer that reads another layer's).  conv_state is not changed
    (conv_state_update does that, after this)."""
    T = x.shape[0]
    taps, C = conv_w.shape
    n_seq = state_slots.numel()
    _fp32_param(conv_w, "conv_w")
    _fp32_param(bias, "bias")
    _fp32_param(inv_freq, "inv_freq")
    if act not in (None, "silu") or (bias is not None and bias.numel() != C):
        raise ValueError("conv_rope_cache: act is None or 'silu', bias one number per channel")
    _check_step(positions, seq_rows, state_slots)
    half = 0 if inv_freq is None else inv_freq.numel()
    if C != n_q * d + n_k * (d + dv) or x.shape[1] < C or x.stride(1) != 1 or 2 * half > d or taps < 1:
        raise ValueError("conv_rope_cache: sections do not fit the row")
    if conv_state.shape[1:] != (taps - 1, C) or conv_state.dtype != x.dtype or not conv_state.is_contiguous():
        raise ValueError("conv_rope_cache: conv_state is [slots, taps - 1, C] of x's dtype")
    if n_k and (kc.shape[-1] != n_k * d or vc.shape[-1] != n_k * dv or kc.dtype != x.dtype or vc.dtype != x.dtype or
                not kc.is_contiguous() or not vc.is_contiguous()):
        raise ValueError("conv_rope_cache: cache row widths / dtype do not match the sections")
    if not x.is_cuda:
        y = torch.zeros((T, C), dtype=torch.float32)
        b = _seq_bounds(seq_rows, n_seq)
        for s in range(n_seq):
            r0, r1 = b[s], b[s + 1]
            sl = int(state_slots[s])
            if sl < 0 or r1 <= r0:
                continue
            p0 = int(positions[r0])
            hist = conv_state[sl].float().clone()  # positions p0 - taps + 1 .. p0 - 1
            for m in range(taps - 1):
                if p0 - (taps - 1) + m < 0:
                    hist[m] = 0.0
            u = torch.cat([hist, x[r0:r1, :C].float()], 0)
            if bias is not None:
                y[r0:r1] += bias
            for j in range(taps):
                y[r0:r1] += u[j:j + r1 - r0] * conv_w[j]
        if act == "silu":
            y = y * torch.sigmoid(y)
        qk = y[:, : (n_q + n_k) * d].reshape(T, n_q + n_k, d)
        if half:
            ang = positions.to(torch.float32)[:, None] * inv_freq[None, :]
            c, s_ = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
            a_, b_ = qk[..., :half].clone(), qk[..., half:2 * half].clone()
            qk[..., :half] = a_ * c - b_ * s_
            qk[..., half:2 * half] = b_ * c + a_ * s_
        qk = qk.reshape(T, (n_q + n_k) * d)
        if n_k:
            ok = kv_slots >= 0
            kc[kv_slots[ok]] = qk[ok, n_q * d:].to(kc.dtype)
            vc[kv_slots[ok]] = y[ok, (n_q + n_k) * d:].to(vc.dtype)
        return qk[:, : n_q * d].to(x.dtype).contiguous()
    if kv_slots.dtype != torch.int64 or (row_seq is not None and row_seq.dtype != torch.int32) or \
            ((row_seq is None) != (seq_rows is None)):
        raise TypeError("conv_rope_cache: int64 kv_slots, int32 row_seq together with seq_rows")
    q = torch.empty((T, n_q * d), dtype=x.dtype, device=x.device)
    _m().conv_rope_cache(q.data_ptr(), x.data_ptr(), x.stride(0), conv_w.data_ptr(), _ptr(bias),
                         int(act == "silu"), taps, conv_state.data_ptr(),
                         conv_state.shape[0], positions.data_ptr(), kv_slots.data_ptr(), _ptr(row_seq), _ptr(seq_rows),
                         state_slots.data_ptr(), n_seq, T, n_q, n_k, d, dv, _ptr(inv_freq), half, _ptr(kc), _ptr(vc),
                         _f32(x), _stream())
    return q


def conv_state_update(x: torch.Tensor, conv_state: torch.Tensor, positions: torch.Tensor,
                      seq_rows: torch.Tensor | None, state_slots: torch.Tensor) -> None:
    """After a step: conv_state [slots, taps - 1, C] of every sequence of the
    step becomes the last taps - 1 projected rows (the leading C columns of x)
    up to and including this step's; a step shorter than taps - 1 rows shifts
    the older ones down.  Entries that lie before position 0 are zero."""
    n_seq = state_slots.numel()
    m, C = conv_state.shape[1:]
    _check_step(positions, seq_rows, state_slots)
    if x.shape[1] < C or x.stride(1) != 1 or conv_state.dtype != x.dtype or not conv_state.is_contiguous():
        raise ValueError("conv_state_update: x covers the state's channels, in its dtype")
    if m == 0:
        return
    if not x.is_cuda:
        b = _seq_bounds(seq_rows, n_seq)
        for s in range(n_seq):
            r0, r1 = b[s], b[s + 1]
            sl = int(state_slots[s])
            if sl < 0 or r1 <= r0:
                continue
            p0 = int(positions[r0])
            old = conv_state[sl].clone()
            for i in range(m):
                if p0 - m + i < 0:
                    old[i] = 0
            conv_state[sl] = torch.cat([old, x[r0:r1, :C]], 0)[-m:]
        return
    _m().conv_state_update(conv_state.data_ptr(), conv_state.shape[0], x.data_ptr(), x.stride(0),
                           positions.data_ptr(), _ptr(seq_rows), state_slots.data_ptr(), n_seq, x.shape[0], C, m + 1,
                           _f32(x), _stream())


def causal_conv(x: torch.Tensor, conv_w: torch.Tensor, conv_state: torch.Tensor, positions: torch.Tensor,
                row_seq: torch.Tensor | None, seq_rows: torch.Tensor | None, state_slots: torch.Tensor,
                bias: torch.Tensor | None = None, act: str | None = None) -> torch.Tensor:
    """The short convolution of conv_rope_cache alone -- on x [T, C], a column
    section, with optional bias and act 'silu' -- together with the update of its
    state: conv_state [slots, taps - 1, C] then holds the last taps - 1 rows of x of
    every sequence of the step.  Returns [T, C]."""
    T, C = x.shape
    taps = conv_w.shape[0]
    if x.is_cuda and _m().conv_run_ok(x.stride(0), C, taps, T, x.data_ptr() | conv_w.data_ptr() | conv_state.data_ptr(),
                                      _f32(x)):
        _fp32_param(conv_w, "conv_w")
        _fp32_param(bias, "bias")
        _check_step(positions, seq_rows, state_slots)
        if act not in (None, "silu") or conv_w.shape[1] != C or (bias is not None and bias.numel() != C) or \
                x.stride(1) != 1 or conv_state.shape[1:] != (taps - 1, C) or conv_state.dtype != x.dtype or \
                not conv_state.is_contiguous():
            raise ValueError("causal_conv: one weight column, bias and state column per channel of x, in its dtype")
        if (row_seq is None) != (seq_rows is None) or (row_seq is not None and row_seq.dtype != torch.int32):
            raise TypeError("causal_conv: int32 row_seq together with seq_rows")
        out = torch.empty((T, C), dtype=x.dtype, device=x.device)
        _m().conv_run(out.data_ptr(), x.data_ptr(), x.stride(0), conv_w.data_ptr(), _ptr(bias), int(act == "silu"), taps,
                      conv_state.data_ptr(), conv_state.shape[0], positions.data_ptr(), _ptr(row_seq), _ptr(seq_rows),
                      state_slots.data_ptr(), state_slots.numel(), T, C, _f32(x), _stream())
        if row_seq is not None:  # (a decode step's kernel has written the new state)
            conv_state_update(x, conv_state, positions, seq_rows, state_slots)
        return out
    out = conv_rope_cache(x, conv_w, conv_state, positions, torch.full_like(positions, -1), row_seq, seq_rows, state_slots,
                          1, 0, C, 0, None, None, None, bias=bias, act=act)
    conv_state_update(x, conv_state, positions, seq_rows, state_slots)
    return out


# ----------------------------------------------------------------- generalized delta rule
DELTA_DECAY_SCALE = math.exp(-0.5)


def delta_rule(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, a: torch.Tensor, w: torch.Tensor,
               a_bias: torch.Tensor | None, w_bias: torch.Tensor | None, state: torch.Tensor, positions: torch.Tensor,
               seq_rows: torch.Tensor | None, state_slots: torch.Tensor, n_heads: int, dk: int, dv: int,
               decay_scale: float = DELTA_DECAY_SCALE, key_eps: float = 1e-6) -> torch.Tensor:
    """The generalized delta rule over the rows of a step, per sequence and head
    from the sequence's state S [dk, dv] (fp32; stored column by column,
    state [slots, H, dv, dk] with state[s, h, j, i] = S[i, j], so that the
    kernel's threads, which own columns, read and write contiguous runs;
    updated in place):
        decay   w_t = exp(-decay_scale * sigmoid(w + w_bias))       per key channel
        removal a_t = sigmoid(a + a_bias)                           per key channel
        unit key u_t = k_t / sqrt(sum(k_t^2) + key_eps)
        S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T      (both terms read S_(t-1))
        o_t = S_t^T r_t
    r, k, a, w [T, H dk] and v [T, H dv] are column sections (contiguous rows,
    any row stride) of projection outputs.  Returns o [T, H dv] fp32.
    Everything but reading the inputs is fp32."""
    T = r.shape[0]
    n_seq = state_slots.numel()
    _fp32_param(a_bias, "a_bias")
    _fp32_param(w_bias, "w_bias")
    _check_step(positions, seq_rows, state_slots)
    for t, wd in ((r, dk), (k, dk), (a, dk), (w, dk), (v, dv)):
        if t.shape != (T, n_heads * wd) or t.stride(1) != 1 or t.dtype != r.dtype:
            raise ValueError("delta_rule: r, k, a, w [T, H dk] and v [T, H dv] with contiguous rows, one dtype")
    if state.shape[1:] != (n_heads, dv, dk) or state.dtype != torch.float32 or not state.is_contiguous():
        raise ValueError("delta_rule: state is contiguous float32 [slots, H, dv, dk]")
    if not r.is_cuda:
        out = torch.zeros((T, n_heads, dv), dtype=torch.float32)
        H = n_heads
        rf, kf, vf = r.float().view(T, H, dk), k.float().view(T, H, dk), v.float().view(T, H, dv)
        wf = torch.exp(-decay_scale * torch.sigmoid(w.float() + (w_bias if w_bias is not None else 0.0))).view(T, H, dk)
        af = torch.sigmoid(a.float() + (a_bias if a_bias is not None else 0.0)).view(T, H, dk)
        uf = kf * torch.rsqrt((kf * kf).sum(-1, keepdim=True) + key_eps)
        b = _seq_bounds(seq_rows, n_seq)
        for s in range(n_seq):
            r0, r1 = b[s], b[s + 1]
            sl = int(state_slots[s])
            if sl < 0 or r1 <= r0:
                continue
            S = state[sl].transpose(1, 2).clone() if int(positions[r0]) > 0 else \
                torch.zeros((H, dk, dv), dtype=torch.float32)
            for t in range(r0, r1):
                uS = torch.einsum("hi,hij->hj", uf[t], S)
                S = wf[t][:, :, None] * S - (af[t] * uf[t])[:, :, None] * uS[:, None, :] + \
                    kf[t][:, :, None] * vf[t][:, None, :]
                out[t] = torch.einsum("hi,hij->hj", rf[t], S)
            state[sl] = S.transpose(1, 2)
        return out.view(T, H * dv)
    out = torch.empty((T, n_heads * dv), dtype=torch.float32, device=r.device)
    # unit key, decay and removal rate * unit key of every row, formed by a pass of its own in front of the scan
    prep = torch.empty((T, n_heads, 3, dk), dtype=torch.float32, device=r.device)
    _m().delta_rule(out.data_ptr(), state.data_ptr(), state.shape[0], prep.data_ptr(), r.data_ptr(), r.stride(0), k.data_ptr(),
                    k.stride(0), v.data_ptr(), v.stride(0), a.data_ptr(), a.stride(0), w.data_ptr(), w.stride(0),
                    _ptr(a_bias), _ptr(w_bias), float(decay_scale), float(key_eps), positions.data_ptr(),
                    _ptr(seq_rows), state_slots.data_ptr(), n_seq, T, n_heads, dk, dv, _f32(r), _stream())
    return out


SCAN_MODES = {"fixed": 0, "step": 1, "channel": 2}


def _linear_scan(mode: str, q, k, v, state, positions, seq_rows, state_slots, n_heads: int, dk: int, dv: int,
                 q_scale: float = 1.0, k_scale: float = 1.0, qk_heads: int | None = None, decay=None, gate=None,
                 g_bias=None, rate=None, skip=None, tau: float = 1.0) -> torch.Tensor:
    """S_t = D_t S_(t-1) + (k_scale k_t) (u_t v_t)^T,  o_t = S_t^T (q_scale q_t) + skip[h] v_t, with D_t and
    u_t by mode (csrc/mixers/linear_scan.hip); head h reads q / k head h // (n_heads / qk_heads)."""
    T, H, n_seq = q.shape[0], n_heads, state_slots.numel()
    G = qk_heads or H
    for t, n in ((decay, "decay"), (g_bias, "bias"), (rate, "rate"), (skip, "skip")):
        _fp32_param(t, n)
    _check_step(positions, seq_rows, state_slots)
    if H % G:
        raise ValueError(f"linear scan: {H} heads over {G} query / key heads")
    gw = {"fixed": None, "step": H, "channel": H * dk}[mode]
    for t, wd in ((q, G * dk), (k, G * dk), (v, H * dv)) + (((gate, gw),) if gw else ()):
        if t.shape != (T, wd) or t.stride(1) != 1 or t.dtype != q.dtype:
            raise ValueError("linear scan: q, k [T, heads dk], v [T, H dv] and the decay / step logits with contiguous "
                             "rows, one dtype")
    if state.shape[1:] != (H, dv, dk) or state.dtype != torch.float32 or not state.is_contiguous():
        raise ValueError("linear scan: state is contiguous float32 [slots, H, dv, dk]")
    for t, wd in ((decay, H), (rate, H), (skip, H), (g_bias, gw)):
        if t is not None and t.numel() != wd:
            raise ValueError("linear scan: one decay / rate / skip per head, one bias per logit")
    if not q.is_cuda:
        out = torch.zeros((T, H, dv), dtype=torch.float32)
        qf = (q.float() * q_scale).view(T, G, dk).repeat_interleave(H // G, 1)
        kf = (k.float() * k_scale).view(T, G, dk).repeat_interleave(H // G, 1)
        vf = v.float().reshape(T, H, dv)
        z = gate.float() + (g_bias if g_bias is not None else 0.0) if gw else None
        uv = vf
        if mode == "fixed":
            D = decay[None, :, None].expand(T, H, 1)
        elif mode == "step":
            u = torch.nn.functional.softplus(z, threshold=1e4)
            D, uv = torch.exp(-rate * u)[:, :, None], vf * u[:, :, None]
        else:
            D = torch.exp(torch.nn.functional.logsigmoid(z) / tau).view(T, H, dk)
        b = _seq_bounds(seq_rows, n_seq)
        for s in range(n_seq):
            r0, r1 = b[s], b[s + 1]
            sl = int(state_slots[s])
            if sl < 0 or r1 <= r0:
                continue
            S = state[sl].transpose(1, 2).clone() if int(positions[r0]) > 0 else \
                torch.zeros((H, dk, dv), dtype=torch.float32)
            for t in range(r0, r1):
                S = D[t][:, :, None] * S + kf[t][:, :, None] * uv[t][:, None, :]
                out[t] = torch.einsum("hi,hij->hj", qf[t], S)
                if skip is not None:
                    out[t] += skip[:, None] * vf[t]
            state[sl] = S.transpose(1, 2)
        return out.view(T, H * dv)
    out = torch.empty((T, H * dv), dtype=torch.float32, device=q.device)
    _m().linear_scan(SCAN_MODES[mode], out.data_ptr(), state.data_ptr(), state.shape[0], q.data_ptr(), q.stride(0),
                     k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0), float(q_scale), float(k_scale), H // G,
                     _ptr(decay), _ptr(gate), gate.stride(0) if gate is not None else 0, _ptr(g_bias), _ptr(rate),
                     _ptr(skip), 1.0 / float(tau), positions.data_ptr(), _ptr(seq_rows), state_slots.data_ptr(), n_seq, T,
                     H, dk, dv, _f32(q), _stream())
    return out


def retention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, k_scale: float,
              state: torch.Tensor, positions: torch.Tensor, seq_rows: torch.Tensor | None, state_slots: torch.Tensor,
              n_heads: int, dk: int, dv: int) -> torch.Tensor:
    """Retention (linear attention with a fixed decay per head, no softmax and
    no denominator) over the rows of a step, per sequence and head from the
    sequence's state S [dk, dv] (fp32; stored column by column, state
    [slots, H, dv, dk] with state[s, h, j, i] = S[i, j]; updated in place):
        S_t = decay[h] S_(t-1) + (k_scale k_t) v_t^T,     o_t = S_t^T q_t.
    q, k [T, H dk] and v [T, H dv] are column sections (contiguous rows, any
    row stride) of projection outputs; decay fp32 [H].  Returns o [T, H dv]
    fp32.  Everything but reading the inputs is fp32."""
    return _linear_scan("fixed", q, k, v, state, positions, seq_rows, state_slots, n_heads, dk, dv, k_scale=k_scale,
                        decay=decay)


def ssd(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, dt_bias: torch.Tensor | None,
        rate: torch.Tensor, skip: torch.Tensor | None, state: torch.Tensor, positions: torch.Tensor,
        seq_rows: torch.Tensor | None, state_slots: torch.Tensor, n_heads: int, n_groups: int, N: int,
        P: int) -> torch.Tensor:
    """State-space duality (Mamba-2's recurrence) over the rows of a step, per
    sequence and head from the sequence's state S [N, P] (fp32, stored as for
    retention: [slots, H, P, N]; updated in place), with the step size
    u_t = softplus(dt_t + dt_bias[h]):
        S_t = exp(-rate[h] u_t) S_(t-1) + u_t B_t x_t^T,     y_t = S_t^T C_t + skip[h] x_t.
    x [T, H P]; B, C [T, n_groups N] shared by H / n_groups heads each; dt [T, H]
    -- column sections, any row stride.  Returns y [T, H P] fp32."""
    return _linear_scan("step", C, B, x, state, positions, seq_rows, state_slots, n_heads, N, P, qk_heads=n_groups,
                        gate=dt, g_bias=dt_bias, rate=rate, skip=skip)


def gated_linear_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, z: torch.Tensor,
                           z_bias: torch.Tensor | None, tau: float, q_scale: float, state: torch.Tensor,
                           positions: torch.Tensor, seq_rows: torch.Tensor | None, state_slots: torch.Tensor,
                           n_heads: int, dk: int, dv: int) -> torch.Tensor:
    """Gated linear attention over the rows of a step, per sequence and head
    from the sequence's state S [dk, dv] (fp32, stored as for retention; updated
    in place), with a decay per key channel and token, alpha_t =
    sigmoid(z_t + z_bias)^(1 / tau):
        S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,     o_t = S_t^T (q_scale q_t).
    q, k, z [T, H dk] and v [T, H dv] are column sections.  Returns o [T, H dv] fp32."""
    return _linear_scan("channel", q, k, v, state, positions, seq_rows, state_slots, n_heads, dk, dv, q_scale=q_scale,
                        gate=z, g_bias=z_bias, tau=tau)


GATE_ACTS = {"sigmoid": 0, "silu": 1}


def head_norm_gate(o: torch.Tensor, n_heads: int, weight: torch.Tensor | None, gate: torch.Tensor | None, eps: float,
                   out_dtype: torch.dtype, gate_act: str = "sigmoid") -> torch.Tensor:
    """o [T, H dv] fp32 -> every head divided by its root mean square
    (sqrt(mean(o_h^2) + eps)), times weight [H dv] (fp32), times act(gate)
    (gate [T, H dv], a column section of the activation dtype; gate_act
    'sigmoid', or 'silu': z sigmoid(z)), in out_dtype."""
    if gate_act not in GATE_ACTS:
        raise ValueError(f"unknown gate activation {gate_act!r}")
    T, W = o.shape
    if o.dtype != torch.float32 or not o.is_contiguous() or W % n_heads:
        raise TypeError("head_norm_gate: o is contiguous float32 [T, H dv]")
    _fp32_param(weight, "weight")
    if gate is not None and (gate.shape != o.shape or gate.stride(1) != 1 or gate.dtype != out_dtype):
        raise ValueError("head_norm_gate: gate [T, H dv] of the output dtype with contiguous rows")
    if not o.is_cuda:
        oh = o.view(T, n_heads, W // n_heads)
        y = (oh * torch.rsqrt((oh * oh).mean(-1, keepdim=True) + eps)).reshape(T, W)
        if weight is not None:
            y = y * weight
        if gate is not None:
            g = gate.float()
            y = y * (torch.sigmoid(g) if gate_act == "sigmoid" else g * torch.sigmoid(g))
        return y.to(out_dtype)
    out = torch.empty((T, W), dtype=out_dtype, device=o.device)
    _m().head_norm_gate(out.data_ptr(), o.data_ptr(), _ptr(weight), _ptr(gate), gate.stride(0) if gate is not None else 0,
                        T, n_heads, W // n_heads, float(eps), GATE_ACTS[gate_act], int(out_dtype == torch.float32),
                        _stream())
    return out


def gate_group_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, n_groups: int, eps: float,
                    out_dtype: torch.dtype, out: torch.Tensor | None = None) -> torch.Tensor:
    """y [T, W] fp32 times silu(z) (z [T, W], a column section of the
    activation dtype), then every one of n_groups equal parts of the row divided
    by its own root mean square (sqrt(mean + eps)), times weight [W] (fp32), in
    out_dtype: the gate enters in front of the norm.  out: where the result
    goes, e.g. a column section of the next projection's input."""
    T, W = y.shape
    _fp32_param(weight, "weight")
    if y.dtype != torch.float32 or not y.is_contiguous() or W % n_groups or weight.numel() != W:
        raise ValueError("gate_group_norm: y is contiguous float32 [T, W], one weight per column, equal parts")
    if z.shape != y.shape or z.stride(1) != 1 or z.dtype != out_dtype:
        raise ValueError("gate_group_norm: gate [T, W] of the output dtype with contiguous rows")
    if out is None:
        out = torch.empty((T, W), dtype=out_dtype, device=y.device)
    elif out.shape != y.shape or out.stride(1) != 1 or out.dtype != out_dtype:
        raise ValueError("gate_group_norm: out is [T, W] of the output dtype with contiguous rows")
    if not y.is_cuda:
        zf = z.float()
        o = (y * zf * torch.sigmoid(zf)).view(T, n_groups, W // n_groups)
        o = (o * torch.rsqrt((o * o).mean(-1, keepdim=True) + eps)).reshape(T, W) * weight
        return out.copy_(o.to(out_dtype))
    _m().gate_group_norm(out.data_ptr(), out.stride(0), y.data_ptr(), z.data_ptr(), z.stride(0), weight.data_ptr(), T,
                         n_groups, W // n_groups, float(eps), int(out_dtype == torch.float32), _stream())
    return out
