"""Povurax in the engine against the plain oracle (tests/povurax_oracle.py).

Every test builds its own small configuration and random (or crafted) weights
in the checkpoint's naming, runs the engine -- scheduler, page and state-slot
manager, model runner, the model's ops -- and compares with the oracle's
dense, whole-sequence float64 arithmetic.  On `cpu` the ops run their PyTorch
forms, on `cuda` (gpu marker) the gfx950 kernels, in float32 and bfloat16.
"""
from __future__ import annotations

import copy
import math

import pytest
import torch

import povurax_oracle as O
from dynamo_exp_amd.engine.engine import EngineConfig, LLMEngine
from dynamo_exp_amd.engine.request import SamplingParams
from dynamo_exp_amd.models.config import LayeredConfig, get_config
from dynamo_exp_amd.models.povurax import PovuraxForCausalLM
from dynamo_exp_amd.ops import mixers as mx
from dynamo_exp_amd.ops import recurrent as rc

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
CASES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


# ----------------------------------------------------------------- configurations
def par(H=4, G=2, d=12, dv=20, dims=8, base=100.0, scale=None, ls=0.7, Hs=6, P=10, N=14, groups=2, norm_groups=3, conv=3,
        rs=1.2):
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": scale or d ** -0.5}
    if dims:
        left["rot"] = {"base": base, "dims": dims}
    return {"type": "parallel", "mixer": {
        "left": left, "left_scale": ls, "right_scale": rs,
        "right": {"heads": Hs, "vdim": P, "state": N, "groups": groups, "norm_groups": norm_groups, "conv": conv}}}


def gla(H=3, d=10, dv=14, tau=8.0):
    return {"type": "gla", "mixer": {"heads": H, "dim": d, "vdim": dv, "tau": tau}}


def layer(mix, ff=40, limit=0.8):
    return {**mix, "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def again(layers, j):
    return {**copy.deepcopy(layers[j]), "weights_of": j}


def config(layers, width=72, vocab=97, eps=1e-5, embed_scale=3.0):
    return LayeredConfig(name="t", architecture="Povurax", vocab_size=vocab, hidden_size=width, layers=layers,
                         rms_norm_eps=eps, embedding_scale=embed_scale)


def mixed():
    ls = [layer(gla()), layer(par())]
    ls += [again(ls, 1), layer(gla(H=2, d=6, dv=22, tau=3.0), 0), again(ls, 0),
           layer(par(H=3, G=1, d=8, dv=6, dims=4, Hs=4, P=16, N=5, groups=1, norm_groups=1, conv=5), 0)]
    return config(ls + [again(ls, 3), again(ls, 5)])


CONFIGS = {
    # both mixers, both with and without a feed-forward, layers that run others' weights, sizes that differ per layer
    "mixed": mixed,
    # values a model may happen to make equal or one: one head, one channel, one state, one tap, scales and tau of one
    "ones": lambda: config([layer(par(H=1, G=1, d=8, dv=8, dims=8, scale=1.0, ls=1.0, Hs=1, P=1, N=1, groups=1, norm_groups=1,
                                      conv=1, rs=1.0)),
                            layer(gla(H=1, d=1, dv=1, tau=1.0)), layer(gla(H=1, d=8, dv=8, tau=1.0), 0),
                            layer(par(H=2, G=2, d=2, dv=4, dims=2, Hs=4, P=2, N=4, groups=4, norm_groups=8, conv=2))],
                           width=32, embed_scale=1.0),
    # nothing divides by 4 or 8 (scalar paths), odd head widths, no rotation
    "odd": lambda: config([layer(par(H=6, G=2, d=7, dv=9, dims=6, Hs=5, P=3, N=17, groups=5, norm_groups=5, conv=4), 10),
                           layer(gla(H=2, d=18, dv=5, tau=2.5), 10), layer(par(H=2, G=1, d=9, dv=5, dims=0, Hs=3, P=7, N=33,
                                                                                groups=1, norm_groups=7, conv=7), 10),
                           layer(gla(H=1, d=34, dv=3), 0)], width=102, vocab=101),
    # head widths the matrix-core kernels serve (bf16 on the GPU), scan widths of the unconditional kernels
    "tiles": lambda: config([layer(par(H=2, G=1, d=64, dv=128, dims=64, base=1e4, Hs=4, P=64, N=128, groups=2, norm_groups=2,
                                       conv=4), 64), layer(gla(H=2, d=64, dv=64, tau=16.0), 0),
                             layer(par(H=4, G=2, d=32, dv=32, dims=16, base=1e4, Hs=2, P=128, N=16, groups=1, norm_groups=1,
                                       conv=4), 64), layer(gla(H=1, d=128, dv=32, tau=4.0), 64)], width=64),
}


def cfg_dict(cfg: LayeredConfig) -> dict:
    return {"layers": cfg.layers, "norm": {"eps": cfg.rms_norm_eps}, "embedding": {"scale": cfg.embedding_scale}}


def weights(cfg, seed=0):
    return PovuraxForCausalLM(cfg, "cpu", torch.float32).random_state(seed)


def engine(cfg, sd, device, dtype, blocks=48, bs=8, seqs=4):
    model = PovuraxForCausalLM(cfg, device, DT[dtype]).load_state(sd)
    return LLMEngine(EngineConfig(model="t", device=device, dtype=dtype, block_size=bs, num_gpu_blocks=blocks,
                                  max_model_len=blocks * bs, max_num_seqs=seqs, enable_prefix_caching=False,
                                  use_cuda_graph=False, async_schedule=False), model_cfg=cfg, model=model)


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def close(got, want, dtype, what=""):
    """Logit rows agree: error relative to the rows' spread, after the mean is taken off."""
    got = got.detach().double().cpu()
    want = want.double()
    a, b = got - got.mean(-1, keepdim=True), want - want.mean(-1, keepdim=True)
    err = ((a - b) ** 2).mean(-1).sqrt() / b.pow(2).mean().sqrt()
    if dtype == "float32":
        assert float(err.max()) < 3e-4, f"{what}: error {float(err.max()):.3g} at row {int(err.argmax())}"
    else:
        assert float(err.median()) < 2e-2 and float((err > 6e-2).float().mean()) <= 0.05, \
            f"{what}: median error {float(err.median()):.3g}, max {float(err.max()):.3g}"


def run_cut(eng, rid, toks, cuts):
    """Feed `toks` in portions of the given sizes (the rest one by one); logits of all positions."""
    out, at = [], 0
    for n in list(cuts) + [1] * (len(toks) - sum(cuts)):
        got = eng.forced_step([(rid, toks[at:at + n], list(range(n)))], [rid] if at + n == len(toks) else [])
        out.append(got[rid])
        at += n
    return torch.cat(out, 0)


def step_meta(device, chunks, slots):
    """Rows of one step: chunks = [(first position, rows)] per sequence, in row order."""
    pos = torch.cat([torch.arange(p, p + n) for p, n in chunks]).to(device)
    row_seq = torch.cat([torch.full((n,), i, dtype=torch.int32) for i, (_, n) in enumerate(chunks)]).to(device)
    b = [0]
    for _, n in chunks:
        b.append(b[-1] + n)
    return pos, row_seq, torch.tensor(b, dtype=torch.int32, device=device), \
        torch.tensor(slots, dtype=torch.int32, device=device)


def interleave(portions, slots, device):
    """Steps of several sequences' portions side by side: (live sequences, cuts, step metadata)."""
    it, at = [list(p) for p in portions], [0] * len(portions)
    while any(it):
        live = [s for s in range(len(it)) if it[s]]
        cuts = [(at[s], it[s].pop(0)) for s in live]
        yield live, cuts, step_meta(device, cuts, [slots[s] for s in live])
        for s, (p, n) in zip(live, cuts):
            at[s] = p + n


def section(t, extra, device):
    """The rows of t as a column section of wider rows."""
    wide = torch.full((t.shape[0], t.shape[1] + extra), 7.0, dtype=t.dtype)
    wide[:, :t.shape[1]] = t
    return wide.to(device)[:, :t.shape[1]]


# ----------------------------------------------------------------- mechanisms alone
SCAN_T = 150
SCAN_PORTIONS = [[(150,), (150,)], [(19, 2, 1, 1, 9, 8, 1, 64, 45), (3, 30, 7, 1, 65, 16, 17, 11)]]


def check_scan(device, run, want, state):
    """run(live, cuts, meta) over whole sequences, then unequal portions, in slots that hold garbage."""
    for portions in SCAN_PORTIONS:
        got = [[], []]
        for live, cuts, meta in interleave(portions, [3, 1], device):
            o = run(live, cuts, meta)
            for i, s in enumerate(live):
                got[s].append(o[int(meta[2][i]):int(meta[2][i + 1])].cpu())
        for s in range(2):
            w, S = want[s]
            assert torch.allclose(torch.cat(got[s]).double(), w.reshape(SCAN_T, -1), atol=3e-4, rtol=1e-4)
            assert torch.allclose(state[3 if s == 0 else 1].cpu().double().transpose(1, 2), S, atol=3e-4, rtol=1e-4)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,N,P", [(4, 2, 14, 10), (1, 1, 1, 1), (2, 1, 128, 64), (4, 4, 16, 256), (3, 1, 33, 7),
                                     (8, 2, 64, 64), (2, 2, 256, 16), (6, 3, 24, 80), (2, 1, 200, 3), (2, 1, 300, 5)])
def test_ssd_scan_alone(device, dtype, H, G, N, P):
    """The state-space recurrence with its step sizes, shared B / C groups and skip, then a decode step
    with a padding row; x, B, C, dt are sections of wider rows."""
    torch.manual_seed(N)
    T, dt_ = SCAN_T, DT[dtype]
    x, B, C = torch.randn(2, T, H * P).to(dt_), torch.randn(2, T, G * N).to(dt_), torch.randn(2, T, G * N).to(dt_)
    dt = (torch.randn(2, T, H) * 2).to(dt_)
    bias, A_log, D = torch.randn(H) - 1, torch.rand(H) * 2, torch.randn(H)
    B, C = B * 0.5, (C.float() * N ** -0.5).to(dt_)  # (outputs stay O(1))
    want = [O.ssd_scan(x[s].double().view(T, H, P), B[s].double().view(T, G, N), C[s].double().view(T, G, N),
                       O.softplus(dt[s].double() + bias.double()), A_log.double(), D.double()) for s in range(2)]
    state = torch.randn(5, H, P, N, device=device)  # garbage: position 0 must reset it
    d = lambda t: t.to(device)  # noqa: E731
    rate = torch.exp(A_log)

    def run(live, cuts, meta):
        sel = lambda t: section(torch.cat([t[s, p:p + n] for s, (p, n) in zip(live, cuts)]), 8, device)  # noqa: E731
        return rc.ssd(sel(x), sel(B), sel(C), sel(dt), d(bias), d(rate), d(D), state, meta[0], meta[2], meta[3], H, G, N, P)

    check_scan(device, run, want, state)
    pos, slots = torch.tensor([T, T, 0], device=device), torch.tensor([3, 1, -1], dtype=torch.int32, device=device)
    before = state[[0, 2, 4]].clone()
    o = rc.ssd(d(x[0, :3]), d(B[0, :3]), d(C[0, :3]), d(dt[0, :3]), d(bias), d(rate), d(D), state, pos, None, slots, H, G, N,
               P)
    assert bool(torch.isfinite(o).all()) and float(o[2].abs().max()) == 0.0
    assert torch.equal(state[[0, 2, 4]], before)  # other slots are not touched


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,dk,dv,tau", [(3, 10, 14, 8.0), (1, 1, 1, 1.0), (2, 64, 64, 16.0), (2, 128, 32, 4.0), (1, 34, 3, 2.0),
                                         (1, 16, 256, 16.0), (2, 256, 32, 16.0), (1, 48, 40, 0.5), (2, 32, 128, 16.0),
                                         (1, 64, 64, 0.25), (1, 128, 64, 0.5), (1, 512, 2, 16.0)])
def test_gla_scan_alone(device, dtype, H, dk, dv, tau):
    """Gated linear attention: a decay per key channel, from hardly any to nearly total (logits far below
    zero, where the decay is a power of e / tau, and far above), then a decode step with a padding row."""
    torch.manual_seed(dk)
    T, dt_ = SCAN_T, DT[dtype]
    q, k, z = (torch.randn(2, T, H * dk).to(dt_) for _ in range(3))
    z = z * 3
    z[:, ::7] -= 40.0
    z[:, 3::7] += 30.0
    z[1, 20] = -300.0
    v, b = torch.randn(2, T, H * dv).to(dt_), torch.randn(H * dk)
    view = lambda t, w: t.double().view(T, H, w)  # noqa: E731
    want = [O.gla_scan(view(q[s], dk) * dk ** -0.5, view(k[s], dk), view(v[s], dv),
                       torch.exp(-O.softplus(-(z[s].double() + b.double())) / tau).view(T, H, dk)) for s in range(2)]
    state = torch.randn(5, H, dv, dk, device=device)
    d = lambda t: t.to(device)  # noqa: E731

    def run(live, cuts, meta):
        sel = lambda t: section(torch.cat([t[s, p:p + n] for s, (p, n) in zip(live, cuts)]), 8, device)  # noqa: E731
        return rc.gated_linear_attention(sel(q), sel(k), sel(v), sel(z), d(b), tau, dk ** -0.5, state, meta[0], meta[2],
                                         meta[3], H, dk, dv)

    check_scan(device, run, want, state)
    pos, slots = torch.tensor([T, T, 0], device=device), torch.tensor([3, 1, -1], dtype=torch.int32, device=device)
    before = state[[0, 2, 4]].clone()
    o = rc.gated_linear_attention(d(q[0, :3]), d(k[0, :3]), d(v[0, :3]), d(z[0, :3]), d(b), tau, 1.0, state, pos, None,
                                  slots, H, dk, dv)
    assert bool(torch.isfinite(o).all()) and float(o[2].abs().max()) == 0.0
    assert torch.equal(state[[0, 2, 4]], before)


@pytest.mark.parametrize("device", DEVICES)
def test_scans_decay_and_keep(device):
    """Crafted: one write, then reads through empty tokens, over a portion, a single token and a portion.
    Per-channel decay: channel 0 halves per token, channel 1 keeps everything (a decay on the value side
    instead would mix them).  State-space: the read-out falls by exp(-rate u) per token, and the skip adds
    D x at its own token only."""
    H, dk, dv, T = 1, 8, 8, 6
    steps = [(0, 2), (2, 1), (3, 3)]
    k, q, v, z = torch.zeros(T, dk), torch.zeros(T, dk), torch.zeros(T, dv), torch.zeros(T, dk)
    k[0, :2] = torch.tensor([1.0, 10.0])
    q[:, :2] = 1.0
    v[0] = 3.0
    z[:, 1] = 60.0  # sigmoid(0) = 1/2 on channel 0, 1 on channel 1
    state = torch.full((2, H, dv, dk), 7.0, device=device)
    got = []
    for p, n in steps:
        pos, _, seq_rows, slots = step_meta(device, [(p, n)], [1])
        got.append(rc.gated_linear_attention(*(t[p:p + n].to(device) for t in (q, k, v, z)), None, 1.0, 1.0, state, pos,
                                             seq_rows, slots, H, dk, dv).cpu())
    o = torch.cat(got)
    for t in range(T):
        assert torch.allclose(o[t], torch.full((dv,), 3.0 * 0.5 ** t + 30.0), atol=1e-4)
    x, dt = torch.zeros(T, dv), torch.zeros(T, H)
    x[0], x[4] = 2.0, 1.0
    B, C = torch.zeros(T, dk), torch.zeros(T, dk)
    B[0, 0], C[:, 0] = 4.0, 1.0
    dt[:] = math.log(math.e - 1.0)  # softplus = 1
    rate, D = torch.tensor([math.log(2.0)]), torch.tensor([0.25])
    got = []
    for p, n in steps:
        pos, _, seq_rows, slots = step_meta(device, [(p, n)], [1])
        got.append(rc.ssd(*(t[p:p + n].to(device) for t in (x, B, C, dt)), None, rate.to(device), D.to(device), state, pos,
                          seq_rows, slots, H, 1, dk, dv).cpu())
    o = torch.cat(got)
    for t in range(T):
        assert torch.allclose(o[t], torch.full((dv,), 8.0 * 0.5 ** t + 0.25 * float(x[t, 0])), atol=1e-5)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,d,dv,dims", [(4, 2, 12, 20, 8), (6, 2, 7, 9, 6), (1, 1, 2, 4, 2), (2, 1, 64, 128, 64), (3, 3, 9, 5, 0),
                                           (32, 8, 128, 128, 32), (5, 1, 16, 8, 10), (80, 16, 128, 24, 128), (3, 1, 6, 3, 4)])
def test_norm_rope_cache_alone(device, dtype, H, G, d, dv, dims):
    """One norm over all heads (not per head, not one for q and k together), rotation of interleaved pairs,
    cache rows of scattered slots, one row not cached; without norm weights too."""
    torch.manual_seed(d)
    T, eps = 9, 1e-5
    dt = DT[dtype]
    pos = torch.tensor([0, 1, 2, 17, 18, 400, 3, 3, 1000])
    slots = torch.tensor([5, 4, 30, 2, 1, 0, -1, 9, 8])
    nq, nk, nv = H * d, G * d, G * dv
    x = (torch.randn(T, nq + nk + nv + 8) * 3).to(dt)
    qw, kw = torch.randn(nq), torch.randn(nk)
    inv = rc.rotary_frequencies(dims, 1e4).to(device) if dims else None
    for with_norm in (True, False):
        xd = x.to(device).clone()
        kc = torch.full((32, nk), 9.0, device=device, dtype=dt)
        vc = torch.full((32, nv), 9.0, device=device, dtype=dt)
        mx.norm_rope_cache(xd, pos.to(device), slots.to(device), H, G, d, nv, qw.to(device) if with_norm else None,
                           kw.to(device) if with_norm else None, eps, inv, kc, vc)
        xf = x.double()
        q, k = xf[:, :nq], xf[:, nq:nq + nk]
        if with_norm:
            q, k = O.unit_rms(q, eps) * qw.double(), O.unit_rms(k, eps) * kw.double()
        q, k = O.rotate_pairs(q.view(T, H, d), pos, dims, 1e4), O.rotate_pairs(k.view(T, G, d), pos, dims, 1e4)
        tol = dict(atol=2e-3, rtol=1e-4) if dtype == "float32" else dict(atol=2e-2, rtol=1e-2)  # (angles up to 1000 in fp32)
        assert torch.allclose(xd[:, :nq].cpu().double(), q.reshape(T, -1), **tol)
        assert torch.equal(xd[:, nq:].cpu(), x[:, nq:])
        ok = slots >= 0
        assert torch.allclose(kc[slots[ok]].cpu().double(), k.reshape(T, -1)[ok], **tol)
        assert torch.equal(vc[slots[ok]].cpu(), x[ok, nq + nk:nq + nk + nv])
        untouched = torch.ones(32, dtype=torch.bool)
        untouched[slots[ok]] = False
        assert bool((kc.cpu()[untouched] == 9.0).all()) and bool((vc.cpu()[untouched] == 9.0).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps,C", [(4, 72), (1, 32), (5, 102), (2, 1), (8, 64), (2, 1040), (3, 24), (4, 30)])
def test_convolution_bias_silu_alone(device, taps, C):
    """The short convolution with bias and silu, two sequences in portions down to one row (shorter than the
    taps), slots reused with garbage in them, channels that are a section of wider rows."""
    torch.manual_seed(taps)
    T = 23
    x, w, b = torch.randn(2, T, C), torch.randn(C, taps), torch.randn(C)
    want = [O.silu(O.channel_conv(x[s].double(), w.double(), b.double())) for s in range(2)]
    tail = torch.randn(4, taps - 1, C, device=device)
    got = [[], []]
    for live, cuts, (pos, row_seq, seq_rows, slots) in interleave([[1, 1, 2, 8, 1, 9, 1], [1, 1, 19, 1, 1]], [2, 0], device):
        xs = section(torch.cat([x[s, p:p + n] for s, (p, n) in zip(live, cuts)]), 8, device)
        if all(n == 1 for _, n in cuts):  # a decode step: row i is sequence i
            row_seq = seq_rows = None
        y = rc.causal_conv(xs, w.t().contiguous().to(device), tail, pos, row_seq, seq_rows, slots, bias=b.to(device), act="silu")
        seq_rows = torch.tensor([0] + [n for _, n in cuts]).cumsum(0)
        for i, s in enumerate(live):
            got[s].append(y[int(seq_rows[i]):int(seq_rows[i + 1])].cpu())
    for s in range(2):
        assert torch.allclose(torch.cat(got[s]).double(), want[s], atol=2e-5)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,groups", [(60, 3), (8, 8), (16384, 2), (4104, 1), (21, 3), (1024, 8), (9000, 1), (640, 10)])
def test_gate_group_norm_alone(device, dtype, W, groups):
    """silu gate in front of the norm, every part by its own root mean square, into a column section."""
    torch.manual_seed(W)
    T, eps, dt = 5, 1e-5, DT[dtype]
    y, z, w = torch.randn(T, W) * 3, (torch.randn(T, W + 8) * 2).to(dt), torch.randn(W)
    y *= torch.logspace(-1, 1, groups).repeat_interleave(W // groups)  # parts of different size
    out = torch.full((T, W + 16), 9.0, dtype=dt, device=device)
    rc.gate_group_norm(y.to(device), z.to(device)[:, 8:], w.to(device), groups, eps, dt, out=out[:, 8:8 + W])
    want = O.gated_group_norm(y.double(), z[:, 8:].double(), w.double(), groups, eps)
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == "float32" else dict(atol=1e-2, rtol=1e-2)
    assert torch.allclose(out[:, 8:8 + W].cpu().double(), want, **tol)
    assert bool((out[:, :8] == 9.0).all()) and bool((out[:, 8 + W:] == 9.0).all())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,dv", [(3, 14), (2, 32), (5, 64), (3, 128), (2, 200), (7, 12), (1, 300), (3, 5)])
def test_head_norm_silu_gate_alone(device, dtype, H, dv):
    """The per-head unit norm with a weight shared by the heads, then the silu gate (behind the norm)."""
    torch.manual_seed(dv)
    T, eps, dt = 5, 1e-5, DT[dtype]
    o, z, w = torch.randn(T, H * dv) * 3, (torch.randn(T, H * dv + 8) * 2).to(dt), torch.randn(dv)
    got = rc.head_norm_gate(o.to(device), H, w.repeat(H).to(device), z.to(device)[:, 8:], eps, dt, gate_act="silu")
    want = (O.unit_rms(o.double().view(T, H, dv), eps) * w.double()).reshape(T, -1) * O.silu(z[:, 8:].double())
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == "float32" else dict(atol=1e-2, rtol=1e-2)
    assert torch.allclose(got.cpu().double(), want, **tol)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("F", [24, 21])
def test_gates_and_clamp_alone(device, F):
    """Output gate times a scale into one part of a wider row; the clamped gated unit beyond its limits."""
    torch.manual_seed(F)
    g, a = torch.randn(5, F + 3) * 2, torch.randn(5, F)
    out = torch.full((5, F + 4), 9.0, device=device)
    mx.act_mul(g.to(device)[:, 3:], a.to(device), "sigmoid", out=out[:, 4:], scale=0.3)
    want = 0.3 * a.double() * O.sigmoid(g[:, 3:].double())
    assert torch.allclose(out[:, 4:].cpu().double(), want, atol=1e-5) and bool((out[:, :4] == 9.0).all())
    gu = torch.randn(5, 2 * F) * 3
    got = mx.glu_act(gu.to(device), "swiglu_clamp", 1.25, O.FF_ALPHA)
    eye = torch.eye(F, dtype=torch.float64)
    want = torch.cat([O.clamped_ff(torch.cat([r[:F], r[F:]])[None].double(), torch.cat([eye, 0 * eye], 1),
                                   torch.cat([0 * eye, eye], 1), eye, 1.25) for r in gu])
    assert torch.allclose(got.cpu().double(), want, atol=2e-5)


# ----------------------------------------------------------------- crafted: one key stands out
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("d,dv,bs", [(32, 32, 16), (12, 20, 8), (64, 128, 8), (128, 128, 64), (64, 64, 128)])
def test_far_keys(device, dtype, d, dv, bs):
    """A cache of empty keys in which one matches the query strongly and carries a marked value: the first
    token, page borders, among hundreds, the query's own token; a key just behind the query is not seen.
    Prompt rows and decode rows (keys in parts) alike."""
    H, G, T = 2, 1, 330
    dt = DT[dtype]
    perm = torch.randperm(48, generator=torch.Generator().manual_seed(3)).to(torch.int32)
    table = perm[: -(-T // bs)][None].contiguous().to(device)
    j = torch.arange(T, device=device)
    slots = table[0].long()[j // bs] * bs + j % bs
    e0 = torch.zeros(d)
    e0[0] = 8.0
    q = e0.repeat(H)[None].to(device, dt)
    kc = torch.zeros(48 * bs, G * d, device=device, dtype=dt)
    vc = torch.zeros(48 * bs, G * dv, device=device, dtype=dt)
    for p in {T - 1, 150, T // bs * bs, T // bs * bs - 1, bs, 1, 0}:
        assert p < T
        for mark in {0, 1, p, p + 1, p - 1, bs - 1, bs, p // bs * bs, p // bs * bs - 1}:
            if not 0 <= mark < T:
                continue
            K, V = torch.zeros(T, d), torch.full((T, dv), -1.0)
            K[mark], V[mark] = e0, 1.0
            kc[slots], vc[slots] = K.to(device, dt), V.to(device, dt)
            hit = math.exp(16.0) if mark <= p else 0.0
            rest = p + 1 - (1 if mark <= p else 0)
            want = (hit - rest) / (hit + rest)
            pos = torch.tensor([p], device=device)
            for seq, parts in ((torch.zeros(1, dtype=torch.int32, device=device), 1), (None, 1), (None, 3)):
                tl = (torch.tensor([[0, 1]], dtype=torch.int32, device=device), 1) if seq is not None else (None, 0)
                got = mx.attention(q, kc, vc, pos, seq, table, bs, H, 1, H // G, d, dv, 0.25, "causal", 0, parts, False, *tl)
                err = float((got.float() - want).abs().max())
                assert err < (1e-4 if dtype == "float32" else 2e-2), (p, mark, seq is None, parts, err)


@pytest.mark.gpu
@pytest.mark.parametrize("d,n_qh,G,maps,bs", [(128, 8, 2, 1, 64), (64, 3, 1, 1, 128), (128, 16, 1, 1, 64), (64, 4, 2, 2, 64)])
@pytest.mark.parametrize("size", [0, 1, 64, 65, 100])
def test_decode_rows_over_whole_tile_pages(d, n_qh, G, maps, bs, size):
    """bf16 decode rows over pages of whole 64-key tiles (the streaming kernel): rows at tile and page edges
    and at position 0, keys in parts, windows that start inside a tile, pages whose unused rows hold NaN."""
    torch.manual_seed(d + size)
    ps = [0, 1, 63, 64, 127, 128, 299]
    n_kh, group, B = G * maps, n_qh // maps // G, len(ps)
    T, per = 300, -(-300 // bs)
    k, v = torch.randn(B, T, n_kh, d).bfloat16(), torch.randn(B, T, G, d).bfloat16()
    q = torch.randn(B, n_qh, d).bfloat16()
    table = torch.randperm(B * per, generator=torch.Generator().manual_seed(1)).to(torch.int32).view(B, per)
    kc = torch.full((B * per * bs, n_kh * d), float("nan"), dtype=torch.bfloat16)
    vc = torch.full((B * per * bs, G * d), float("nan"), dtype=torch.bfloat16)
    want = torch.zeros(B, n_qh, d, dtype=torch.float64)
    for b, p in enumerate(ps):
        j = torch.arange(p + 1)
        sl = table[b].long()[j // bs] * bs + j % bs
        kc[sl], vc[sl] = k[b, :p + 1].reshape(p + 1, -1), v[b, :p + 1].reshape(p + 1, -1)
        near = j[max(0, p - size + 1) if size else 0:]
        for h in range(n_qh):
            head, mp = h // maps, h % maps
            w = torch.softmax((k[b, near, head // group * maps + mp].double() @ q[b, h].double()) * 0.3, 0)
            want[b, h] = w @ v[b, near, head // group].double()
    pos = torch.tensor(ps).cuda()
    for parts in (1, 3):
        got = mx.attention(q.reshape(B, -1).cuda(), kc.cuda(), vc.cuda(), pos, None, table.cuda(), bs, n_qh, maps, group, d, d,
                           0.3, "window" if size else "causal", size, parts, True)
        assert float((got.cpu().double() - want).abs().max()) < 1e-3 * max(1.0, float(want.abs().max()))


@pytest.mark.gpu
@pytest.mark.parametrize("d,n_qh,G,bs", [(128, 8, 2, 64), (64, 4, 2, 128), (128, 12, 2, 64), (64, 16, 2, 64), (128, 3, 1, 64)])
@pytest.mark.parametrize("size", [0, 1, 64, 65, 100])
def test_prompt_rows_over_whole_tile_pages(d, n_qh, G, bs, size):
    """bf16 prompt rows over pages of whole 64-key tiles (the streaming kernel where heads pair up): portions
    that start at position 0, inside a cached prefix and at a tile's edge, one of two rows, beside a decode row;
    windows that start inside a tile, pages whose unused rows hold NaN."""
    torch.manual_seed(d + size)
    chunks = [(0, 150), (37, 263), (64, 2), (190, 130), (5, 1)]  # (first position, rows); the last a decode row
    group, B, T = n_qh // G, len(chunks), 330
    per = -(-T // bs)
    k, v = torch.randn(B, T, G, d).bfloat16(), torch.randn(B, T, G, d).bfloat16()
    table = torch.randperm(B * per, generator=torch.Generator().manual_seed(1)).to(torch.int32).view(B, per)
    kc = torch.full((B * per * bs, G * d), float("nan"), dtype=torch.bfloat16)
    vc = torch.full((B * per * bs, G * d), float("nan"), dtype=torch.bfloat16)
    q = torch.randn(sum(n for _, n in chunks), n_qh, d).bfloat16()
    want, tiles, r0 = torch.zeros(q.shape, dtype=torch.float64), [], 0
    for b, (p, n) in enumerate(chunks):
        j = torch.arange(p + n)
        sl = table[b].long()[j // bs] * bs + j % bs
        kc[sl], vc[sl] = k[b, :p + n].reshape(p + n, -1), v[b, :p + n].reshape(p + n, -1)
        dist = torch.arange(p, p + n)[:, None] - j[None, :]
        vis = (dist >= 0) & ((dist < size) if size else torch.ones_like(dist, dtype=torch.bool))
        for h in range(n_qh):
            sc = (q[r0:r0 + n, h].double() @ k[b, :p + n, h // group].double().T) * 0.2
            want[r0:r0 + n, h] = torch.softmax(sc.masked_fill(~vis, float("-inf")), -1) @ v[b, :p + n, h // group].double()
        if b < B - 1:
            tiles += mx.tile_list(r0, n)
        r0 += n
    pos, row_seq, _, _ = step_meta("cuda", chunks, [0] * B)
    tl = torch.tensor(tiles, dtype=torch.int32, device="cuda")
    err = []
    for fine in (False, True):
        got = mx.attention(q.reshape(r0, -1).cuda(), kc.cuda(), vc.cuda(), pos, row_seq, table.cuda(), bs, n_qh, 1, group, d, d,
                           0.2, "window" if size else "causal", size, 1, False, tl, r0 - 1, fine_weights=fine)
        diff = (got.cpu().double() - want).abs()
        assert float(diff.max()) < 2e-2 * max(1.0, float(want.abs().max()))
        err.append(float((diff / want.abs().clamp_min(0.05)).pow(2).mean().sqrt()))
    assert err[1] < 2.5e-3  # the result's own rounding to bf16, and no more
    assert size == 1 or err[0] > 1.1 * err[1]


# ----------------------------------------------------------------- whole model
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_layers(device, dtype, name):
    """A whole prompt in one step: logits at every position, and (float32) the residual after every layer."""
    cfg = CONFIGS[name]()
    sd = weights(cfg, 1)
    toks = tokens(75, cfg.vocab_size, 2)
    want, after = O.forward(cfg_dict(cfg), sd, toks)
    eng = engine(cfg, sd, device, dtype)
    if dtype == "float32":
        eng.model.trace_layers = []
    got = eng.forced_step([("a", toks, list(range(len(toks))))], ["a"])["a"]
    close(got, want, dtype, name)
    if dtype == "float32":
        assert len(eng.model.trace_layers) == len(cfg.layers)
        for i, (x, w) in enumerate(zip(eng.model.trace_layers, after)):
            assert float((x.cpu().double() - w).abs().max()) < 2e-3 * float(w.abs().max()), f"layer {i}"


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name,cuts", [("mixed", ()), ("mixed", (31, 2, 2, 17, 3)), ("ones", (2, 2, 2, 40)),
                                       ("odd", (50, 2)), ("tiles", (7, 64, 2)), ("tiles", ())])
def test_portions_and_decode(device, dtype, name, cuts):
    """Token-by-token decoding from the first token, and portions of several sizes down to two
    tokens followed by single tokens, against the whole-sequence oracle."""
    cfg = CONFIGS[name]()
    sd = weights(cfg, 4)
    toks = tokens(80, cfg.vocab_size, 5)
    want, _ = O.forward(cfg_dict(cfg), sd, toks)
    close(run_cut(engine(cfg, sd, device, dtype), "a", toks, cuts), want, dtype, f"{name} {cuts}")


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_mixed_batches_reuse(device, dtype, name):
    """Five unequal requests interleaved, portions beside single tokens, in a pool of pages and of
    state slots (three) that only fits them because both are given back and used again."""
    cfg = CONFIGS[name]()
    sd = weights(cfg, 5)
    reqs = {f"r{i}": tokens(n, cfg.vocab_size, 10 + i) for i, n in enumerate([70, 41, 90, 33, 58])}
    want = {k: O.forward(cfg_dict(cfg), sd, t)[0] for k, t in reqs.items()}
    eng = engine(cfg, sd, device, dtype, blocks=30, bs=8, seqs=3)
    plan = [[("r0", 9), ("r1", 2)], [("r0", 1), ("r1", 30), ("r2", 3)], [("r0", 40), ("r1", 1), ("r2", 1)],
            [("r0", 1), ("r1", 8), ("r2", 50)], [("r0", 19), ("r2", 1)], [("r2", 35), ("r3", 2)],
            [("r3", 31), ("r4", 2)], [("r4", 1)], [("r4", 55)]]
    at, got = {k: 0 for k in reqs}, {k: [] for k in reqs}
    for step in plan:
        entries, end = [], []
        for k, n in step:
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        out = eng.forced_step(entries, end)
        for k, _ in step:
            got[k].append(out[k])
    assert eng.kv.num_free_state() == 3 and eng.kv.num_free() == 30
    for k in reqs:
        assert at[k] == len(reqs[k])
        close(torch.cat(got[k]), want[k], dtype, f"{name} {k}")


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_decode_and_first_tokens(device, dtype):
    """146 consecutive decode steps after a two-token prompt, the first positions (fewer tokens than taps)
    among them; then a prompt as long as several scan blocks and attention tiles in one step."""
    cfg = CONFIGS["mixed"]()
    sd = weights(cfg, 6)
    toks = tokens(148, cfg.vocab_size, 7)
    want, _ = O.forward(cfg_dict(cfg), sd, toks)
    close(run_cut(engine(cfg, sd, device, dtype), "a", toks, (2,)), want, dtype, "long decode")


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("bs", [8, 64])
def test_long_prompt_portions(device, dtype, bs):
    """A prompt of several hundred tokens in portions that end inside and at the edges of the kernels' token
    blocks and tiles (63, 64, 65, 128 + 1, ...), beside a second sequence."""
    cfg = config([layer(par(H=4, G=2, d=64, dv=64, dims=32, base=1e4, Hs=2, P=64, N=64, groups=1, norm_groups=1, conv=4), 32),
                  layer(gla(H=1, d=64, dv=64, tau=16.0), 0)], width=32)
    sd = weights(cfg, 16)
    a, b = tokens(330, cfg.vocab_size, 17), tokens(200, cfg.vocab_size, 18)
    wa, wb = O.forward(cfg_dict(cfg), sd, a)[0], O.forward(cfg_dict(cfg), sd, b)[0]
    eng = engine(cfg, sd, device, dtype, blocks=640 // bs, bs=bs)
    ga, gb, pa, pb = [], [], 0, 0
    for na, nb in ((63, 64), (65, 1), (129, 127), (1, 2), (64, 6), (8, 0)):
        ent = [("a", a[pa:pa + na], list(range(na)))] + ([("b", b[pb:pb + nb], list(range(nb)))] if nb else [])
        out = eng.forced_step(ent, [k for k, done in (("a", pa + na == 330), ("b", nb and pb + nb == 200)) if done])
        ga.append(out["a"])
        if nb:
            gb.append(out["b"])
        pa, pb = pa + na, pb + nb
    close(torch.cat(ga), wa, dtype, "a")
    close(torch.cat(gb), wb, dtype, "b")


@pytest.mark.parametrize("device,dtype", CASES)
def test_crafted_weights_show_faults(device, dtype):
    """Weights made so that faults move the logits; the engine agrees with the oracle, and the oracle's own
    variants -- swapped halves' scales, a rotation by halves' worth of base, another tau, no skip, a decay
    rate slightly off, a clamp elsewhere, a shared layer's weights of its own, norms over other parts -- differ visibly."""
    ls = [layer(par(H=2, G=1, d=16, dv=16, dims=16, scale=1.0, Hs=4, P=8, N=16, groups=2, norm_groups=2, ls=0.6, rs=1.4)),
          layer(gla(H=2, d=16, dv=16, tau=2.0), 0)]
    cfg = config(ls + [again(ls, 0)], width=48, vocab=61)
    sd = weights(cfg, 8)
    sd["l0.mix.right.dt_bias"] = torch.full((4,), -1.0).bfloat16()
    toks = tokens(60, cfg.vocab_size, 9)
    want, _ = O.forward(cfg_dict(cfg), sd, toks)
    close(run_cut(engine(cfg, sd, device, dtype), "a", toks, (13, 2, 30)), want, dtype, "crafted")

    def differs(change):
        c, s2 = copy.deepcopy(cfg_dict(cfg)), dict(sd)
        change(c["layers"], s2)
        off = O.forward(c, s2, toks)[0]
        return float((off - want).abs().max()) > 0.02 * float(want.abs().max())

    def each(layers, *path):  # the dicts at mixer/path of both parallel layers
        for L in (layers[0], layers[2]):
            m = L["mixer"]
            for k in path:
                m = m[k]
            yield m

    assert differs(lambda c, s: [m.update(left_scale=1.4, right_scale=0.6) for m in each(c)])
    assert differs(lambda c, s: [m["rot"].update(base=50.0) for m in each(c, "left")])
    assert differs(lambda c, s: [m["rot"].update(dims=14) for m in each(c, "left")])
    assert differs(lambda c, s: [m.update(norm_groups=1) for m in each(c, "right")])
    assert differs(lambda c, s: c[1]["mixer"].update(tau=2.2))
    assert differs(lambda c, s: [L["mlp"].update(limit=1.0) for L in (c[0], c[2])])
    assert differs(lambda c, s: s.update({"l0.mix.right.D": sd["l0.mix.right.D"] * 0}))
    assert differs(lambda c, s: s.update({"l0.mix.right.A_log": sd["l0.mix.right.A_log"] + 0.2}))
    assert differs(lambda c, s: (c[2].pop("weights_of"),
                                 s.update({k.replace("l0.", "l2."): v.roll(1, 0) for k, v in sd.items() if k[:3] == "l0."})))


# ----------------------------------------------------------------- the engine's own entry point
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation(device, dtype, graphs):
    """add_request + step(): chunked prefill, continuous batching, state slots handed out and taken
    back by the scheduler, HIP-graph decode on the GPU; greedy tokens equal the oracle's."""
    if graphs and device == "cpu":
        pytest.skip("graphs are a GPU path")
    cfg = CONFIGS["tiles" if device == "cuda" else "mixed"]()
    sd = weights(cfg, 11)
    model = PovuraxForCausalLM(cfg, device, DT[dtype]).load_state(sd)
    eng = LLMEngine(EngineConfig(model="t", device=device, dtype=dtype, block_size=8, num_gpu_blocks=64,
                                 max_model_len=256, max_num_seqs=2, max_num_batched_tokens=24,
                                 use_cuda_graph=graphs, graph_sizes=(1, 2), async_schedule=False),
                    model_cfg=cfg, model=model)
    assert eng.cfg.enable_prefix_caching is False  # per-sequence state cannot be served from the prefix cache
    if graphs:
        eng.warmup()
    prompts = [tokens(37, cfg.vocab_size, 20), tokens(9, cfg.vocab_size, 21), tokens(50, cfg.vocab_size, 22)]
    n_new = 10
    for i, p in enumerate(prompts):
        eng.add_request(f"g{i}", p, SamplingParams(max_tokens=n_new, ignore_eos=True))
    done = {}
    for _ in range(400):
        for r in eng.step():
            if r.finished:
                done[r.request_id] = list(r.output)
        if not eng.has_unfinished():
            break
    assert len(done) == 3 and eng.kv.num_free_state() == 2
    for i, p in enumerate(prompts):
        out = done[f"g{i}"]
        assert len(out) == n_new
        # the oracle over the engine's own path: every token on it is the best of its row
        lg = O.forward(cfg_dict(cfg), sd, list(p) + out)[0][len(p) - 1:-1]
        for row, t in zip(lg, out):
            gap = float(row.max() - row[t])
            assert gap < (1e-3 if dtype == "float32" else 0.1 * float(row.std())), (i, gap)


@pytest.mark.parametrize("device,dtype", CASES)
def test_trace_replay_command(tmp_path, monkeypatch, capsys, device, dtype):
    """The replay command on a checkpoint directory: the class follows config.json, a portion beside
    a shorter one, a decode token beside a portion, a step in which nothing is wanted, a slot and
    pages used again; logits files against the oracle."""
    import io
    import json
    import sys

    import numpy as np
    from safetensors.torch import save_file

    from dynamo_exp_amd.cli import trace_run

    cfg = CONFIGS["mixed"]()
    sd = weights(cfg, 21)
    model_dir, out = tmp_path / "m", tmp_path / "out"
    cfg.write_hf_config(str(model_dir))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(model_dir / "model.safetensors"))
    a, b = tokens(40, cfg.vocab_size, 31), tokens(9, cfg.vocab_size, 32)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:25], "want": [0, 24]},
                                     {"id": "b", "tokens": b[:2], "want": [1]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[25:26], "want": [0]},
                                     {"id": "b", "tokens": b[2:], "want": [0, 6]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[26:], "want": []}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [8]}], "end": ["c"]}]
    monkeypatch.setattr(sys, "stdin", io.StringIO("\n".join(json.dumps(st) for st in steps) + "\n"))
    assert trace_run.main(["--model", str(model_dir), "--dtype", dtype, "--out", str(out), "--max-tokens", "128",
                           "--device", device]) == 0
    assert [ln for ln in capsys.readouterr().out.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    assert not (out / "2.f32").exists()
    wa, wb = O.forward(cfg_dict(cfg), sd, a)[0], O.forward(cfg_dict(cfg), sd, b)[0]
    got = {i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg.vocab_size)) for i in (0, 1, 3)}
    close(got[0], torch.cat([wa[[0, 24]], wb[[1]]]), dtype, "step 0")
    close(got[1], torch.cat([wa[[25]], wb[[2, 8]]]), dtype, "step 1")
    close(got[3], wb[[8]], dtype, "step 3")


def test_config_round_trip(tmp_path):
    """config.json keys -> LayeredConfig -> config.json; weight sharing; the preset builds and counts its weights."""
    cfg = CONFIGS["mixed"]()
    cfg.write_hf_config(str(tmp_path))
    back = get_config(str(tmp_path))
    assert back.architecture == "Povurax" and back.layers == cfg.layers and back.embedding_scale == cfg.embedding_scale
    assert back.weight_layers() == [0, 1, 1, 3, 0, 5, 3, 5]
    tiny = get_config("povurax-tiny")
    model = PovuraxForCausalLM(tiny, "cpu", torch.float32)
    sd = model.random_state(0)
    assert sum(v.numel() for v in sd.values()) == tiny.num_params()
    model.load_state(sd)
    assert model.layers[2] is model.layers[0] and model.layers[1] is not model.layers[3]
    kv = model.alloc_kv_caches(2, 4, torch.float32)  # shared weights, caches and states of their own
    assert kv[0][0].data_ptr() != kv[2][0].data_ptr() and kv[1][0].numel() == 0
    assert len(model.alloc_state(1)) == 2 * 3 + 2
    from dynamo_exp_amd.models.registry import build_model, supports_dtype

    assert supports_dtype("Povurax", "float32") and supports_dtype("Povurax", "bfloat16")
    assert isinstance(build_model(back, "cpu", dtype="float32"), PovuraxForCausalLM)
    for bad in ([{"type": "general_delta", "mixer": {"heads": 1, "dim": 8}, "mlp": None}],
                [{**layer(gla()), "weights_of": 0}], [layer(gla()), {**layer(gla(tau=2.0)), "weights_of": 0}]):
        with pytest.raises(ValueError):
            PovuraxForCausalLM(config(bad), "cpu", torch.float32)
