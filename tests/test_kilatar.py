"""Kilatar in the engine against the plain oracle (tests/kilatar_oracle.py).

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

import kilatar_oracle as O
from dynamo_exp_amd.engine.engine import EngineConfig, LLMEngine
from dynamo_exp_amd.engine.request import SamplingParams
from dynamo_exp_amd.models.config import LayeredConfig, get_config
from dynamo_exp_amd.models.kilatar import KilatarForCausalLM
from dynamo_exp_amd.ops import mixers as mx
from dynamo_exp_amd.ops import moe
from dynamo_exp_amd.ops import recurrent as rc

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
CASES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
SCALING = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 60}


# ----------------------------------------------------------------- configurations
def lat(H=3, d=12, dr=8, dv=10, r=24, dims=None, base=100.0, scale=None):
    return {"type": "latent_attention", "mixer": {
        "heads": H, "dim": d, "rot_dim": dr, "vdim": dv, "kv_rank": r, "scale": scale or (d + dr) ** -0.5,
        "rot": {"base": base, "dims": dr if dims is None else dims}}}


def ssm(H=6, P=10, N=14, groups=2, norm_groups=3, conv=3):
    return {"type": "mamba2", "mixer": {"heads": H, "vdim": P, "state": N, "groups": groups, "norm_groups": norm_groups,
                                        "conv": conv}}


def par(H=4, G=2, d=12, dv=20, dims=8, base=100.0, scaling=SCALING, chunk=24, scale=None, Hr=3, dk=10, dvr=14, decay=None):
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": scale or d ** -0.5}
    if dims:
        left["rot"] = {"base": base, "dims": dims, **({"scaling": dict(scaling)} if scaling else {})}
    if chunk:
        left["mask"] = {"size": chunk}
    return {"type": "parallel", "mixer": {"left": left, "right": {
        "heads": Hr, "dim": dk, "vdim": dvr, "decay": decay or [1.0 - 0.4 ** (h + 1) for h in range(Hr)]}}}


def dense(mix, ff=40):
    return {**mix, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def routed(mix, E=5, top=2, identity=2, ff=24, shared=28, scale=1.5):
    return {**mix, "mlp": {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None,
                           "router": {"experts": E, "top": top, "identity": identity, "scale": scale}}}


def config(layers, width=72, vocab=97, eps=1e-5, loop=None):
    return LayeredConfig(name="t", architecture="Kilatar", vocab_size=vocab, hidden_size=width, layers=layers,
                         rms_norm_eps=eps, loop=loop)


def span(start, stop, times):
    return {"start": start, "stop": stop, "times": times}


CONFIGS = {
    # every mixer with every kind of feed-forward or none, a loop in the middle, sizes that differ per layer
    "mixed": lambda: config([dense(lat()), routed(par()), dense(ssm(), 0), routed(lat(H=2, d=6, dr=4, dv=22, r=16), E=7, top=3,
                             identity=1, shared=0), dense(par(H=3, G=1, d=8, dv=6, dims=4, scaling=None, chunk=7, Hr=2, dk=6,
                                                              dvr=22)), routed(ssm(H=4, P=16, N=5, groups=1, norm_groups=1,
                                                                                   conv=5), identity=0)],
                            loop=span(1, 4, 2)),
    # values a model may happen to make equal or one: one head, channel, state, tap, expert; a loop of one pass
    "ones": lambda: config([routed(par(H=1, G=1, d=8, dv=8, dims=8, chunk=1, scale=1.0, Hr=1, dk=1, dvr=1, decay=[0.5]), E=1,
                                   top=1, identity=0, ff=8, shared=0, scale=1.0),
                            dense(ssm(H=1, P=1, N=1, groups=1, norm_groups=1, conv=1)),
                            dense(lat(H=1, d=2, dr=2, dv=2, r=4, scale=1.0)),
                            routed(ssm(H=4, P=2, N=4, groups=4, norm_groups=8, conv=2), E=2, top=3, identity=1, ff=8, shared=8,
                                   scale=0.5)], width=32, loop=span(0, 4, 1)),
    # nothing divides by 4 or 8 (scalar paths), odd head widths, no rotation, no chunks; the whole stack three times
    "odd": lambda: config([routed(par(H=6, G=2, d=7, dv=9, dims=6, chunk=31, Hr=2, dk=18, dvr=5), E=3, top=1, identity=3, ff=11,
                                  shared=9), dense(lat(H=5, d=3, dr=5, dv=7, r=9, dims=4), 13),
                           routed(ssm(H=5, P=3, N=17, groups=5, norm_groups=5, conv=4), E=3, identity=1, ff=7, shared=0),
                           dense(par(H=2, G=1, d=9, dv=5, dims=0, chunk=0, Hr=1, dk=34, dvr=3), 10)], width=101, vocab=103,
                          loop=span(0, 4, 3)),
    # widths the matrix-core kernels serve (bf16 on the GPU), scan widths of the unconditional and chunked kernels;
    # chunks that end inside and at tiles; a loop at the end
    "tiles": lambda: config([routed(par(H=4, G=2, d=64, dv=64, dims=64, base=1e4, chunk=64, Hr=2, dk=64, dvr=64), E=4, ff=64,
                                    shared=64), dense(lat(H=4, d=32, dr=32, dv=48, r=64, base=1e4), 64),
                             routed(ssm(H=4, P=64, N=128, groups=2, norm_groups=2, conv=4), E=4, ff=64, shared=64),
                             dense(par(H=2, G=1, d=32, dv=64, dims=16, base=1e4, chunk=50, Hr=1, dk=128, dvr=32))], width=64,
                            loop=span(2, 4, 2)),
}


def cfg_dict(cfg: LayeredConfig) -> dict:
    return {"layers": cfg.layers, "norm": {"eps": cfg.rms_norm_eps}, "loop": cfg.loop}


def weights(cfg, seed=0):
    """Random weights; routers decisive enough that bfloat16 rounding rarely changes a choice that matters."""
    sd = KilatarForCausalLM(cfg, "cpu", torch.float32).random_state(seed)
    return {k: v * 3 if k.endswith("mlp.router") else v for k, v in sd.items()}


def engine(cfg, sd, device, dtype, blocks=48, bs=8, seqs=4):
    model = KilatarForCausalLM(cfg, device, DT[dtype]).load_state(sd)
    return LLMEngine(EngineConfig(model="t", device=device, dtype=dtype, block_size=bs, num_gpu_blocks=blocks,
                                  max_model_len=blocks * bs, max_num_seqs=seqs, enable_prefix_caching=False,
                                  use_cuda_graph=False, async_schedule=False), model_cfg=cfg, model=model)


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def close(got, want, dtype, what=""):
    """Logit rows agree: error relative to the rows' spread, after the mean is taken off.  bfloat16: the median
    row, and most rows (a close call of a router may go the other way)."""
    got = got.detach().double().cpu()
    want = want.double()
    a, b = got - got.mean(-1, keepdim=True), want - want.mean(-1, keepdim=True)
    err = ((a - b) ** 2).mean(-1).sqrt() / b.pow(2).mean().sqrt()
    if dtype == "float32":
        assert float(err.max()) < 3e-4, f"{what}: error {float(err.max()):.3g} at row {int(err.argmax())}"
    else:
        assert float(err.median()) < 3e-2 and float((err > 8e-2).float().mean()) <= 0.1, \
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


def section(t, extra, device):
    """The rows of t as a column section of wider rows."""
    wide = torch.full((t.shape[0], t.shape[1] + extra), 7.0, dtype=t.dtype)
    wide[:, :t.shape[1]] = t
    return wide.to(device)[:, :t.shape[1]]


def tol(dtype, f=1e-4, b=1e-2):
    return dict(atol=f, rtol=f) if dtype == "float32" else dict(atol=b, rtol=b)


# ----------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W", [72, 21, 2051, 8200])
def test_embedding_norm_alone(device, W):
    torch.manual_seed(W)
    table, w, ids = torch.randn(11, W) * 3, torch.randn(W), torch.tensor([3, 0, 10, 3])
    got = mx.embed_streams(ids.to(device), table.to(device), 1, norm_w=w.to(device), eps=1e-3).cpu().double()
    assert torch.allclose(got[:, 0], O.unit_rms(table[ids].double(), 1e-3) * w.double(), atol=2e-5, rtol=1e-5)
    plain = mx.embed_streams(ids.to(device), table.to(device), 2).cpu()
    assert torch.equal(plain[:, 0], table[ids]) and torch.equal(plain[:, 1], table[ids])


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W", [72, 21, 2051, 8200])
def test_residual_step_addends_alone(device, dtype, W):
    """Two addends that enter with unit RMS, a constant row, experts' weighted sum with identity outputs, the
    re-entering fp32 addend, the norm behind them; all of it on a list of rows with the residual left alone."""
    torch.manual_seed(W)
    T, top, E, eps, dt = 6, 3, 4, 1e-3, DT[dtype]
    X, e = torch.randn(T, W), torch.randn(T, W)
    a, c, d, y, h = (torch.randn(n, W).to(dt) for n in (T, T, T, T * top, T))
    cw, dw, bias, nw = (torch.randn(W) for _ in range(4))
    w, idx = torch.rand(T, top), torch.randint(0, E + 2, (T, top), dtype=torch.int32)
    idx[0] = torch.tensor([E, 1, E + 1])
    ys = y.double().view(T, top, W).clone()
    y = y.view(T, top, W)
    y[idx >= E] = float("nan")  # an identity output's slot holds nothing
    y = y.view(T * top, W)
    ys = torch.where((idx >= E)[:, :, None], h.double()[:, None, :], ys)
    m = (ys * w.double()[:, :, None]).sum(1)
    dev = lambda t: t.to(device)  # noqa: E731
    for part in ("all", "d", "experts", "e", "bias"):
        kw, want = {}, X.double()
        if part in ("all", "d"):
            kw.update(a=dev(a), c=dev(c), c_w=dev(cw), d=dev(section(d, 5, "cpu")), d_w=dev(dw))
            want = want + a.double() + O.unit_rms(c.double(), eps) * cw.double() + O.unit_rms(d.double(), eps) * dw.double()
        if part in ("all", "bias"):
            kw.update(bias=dev(bias))
            want = want + bias.double()
        if part in ("all", "e"):
            kw.update(e=dev(e))
            want = want + e.double()
        if part in ("all", "experts"):
            kw.update(experts=(dev(y), dev(w), dev(idx), E, dev(h)))
            want = want + m
        nrm = O.unit_rms(want, eps) * nw.double()
        for rows in (torch.tensor([5, 0, 0, 3]), None):
            Xd = X.clone().to(device)
            got, xc = mx.residual_step(Xd, eps=eps, norm="rms", norm_w=dev(nw), out_dtype=dt, want_cast=True,
                                       rows=dev(rows) if rows is not None else None, **kw)
            pick = slice(None) if rows is None else rows
            assert torch.allclose(got.cpu().double(), nrm[pick], **tol(dtype, 1e-4, 2e-2)), (part, rows)
            assert torch.allclose(xc.cpu().double(), want[pick], **tol(dtype, 1e-4, 2e-2))
            assert torch.allclose(Xd.cpu().double(), want if rows is None else X.double(), atol=1e-4, rtol=1e-5)
    got = mx.residual_step(X.clone().to(device), eps=eps, norm="rms", norm_w=dev(nw), out_dtype=dt,
                           experts=(dev(torch.nan_to_num(y)), dev(w), None, E, None))[0]
    want = X.double() + (torch.nan_to_num(y).double().view(T, top, W) * w.double()[:, :, None]).sum(1)
    assert torch.allclose(got.cpu().double(), O.unit_rms(want, eps) * nw.double(), **tol(dtype, 1e-4, 2e-2))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("W,E,top,identity,gates", [(72, 5, 2, 2, 1), (33, 1, 1, 0, 0), (21, 3, 4, 3, 1), (256, 30, 8, 2, 2),
                                                    (130, 64, 6, 5, 1), (8, 700, 3, 1, 1), (2056, 9, 2, 2, 1)])
@pytest.mark.parametrize("T", [1, 17, 300, 1100])
def test_router_alone(device, dtype, W, E, top, identity, gates, T):
    """Logits in fp32, softmax over all outputs, choice with the correction, weights without it, divided by their
    sum, scaled; gates of the same pass; token counts on all of the kernels' shapes."""
    torch.manual_seed(W + E)
    n, dt = E + identity, DT[dtype]
    h, w, corr = torch.randn(T, W).to(dt), torch.randn(n + gates, W) * W ** -0.5 * 2, torch.randn(n) * 0.2
    for c in (corr, None):
        idx, wt, gt = moe.router(section(h, 8, device), w.to(device), n, c.to(device) if c is not None else None, top,
                                 score="softmax", renorm=True, scale=1.7)
        z = h.double() @ w.double().T
        assert (gt is None) == (gates == 0)
        if gates:
            assert torch.allclose(gt.cpu().double(), O.sigmoid(z[:, n:]), atol=1e-5)
        cc = c.double() if c is not None else torch.zeros(n, dtype=torch.float64)
        for t in list(range(min(T, 20))) + ([T - 1] if T > 20 else []):
            order, want = O.route(z[t, :n], cc, top, 1.7)
            s = torch.softmax(z[t, :n], -1) + cc
            srt = s.sort(descending=True).values
            if top < n and float(srt[top - 1] - srt[top]) < 1e-6:
                continue  # a tie within fp32 rounding
            got = dict(zip(idx[t].tolist(), wt[t].double().tolist()))
            assert sorted(got) == sorted(order), (t, idx[t], order)
            for e, v in zip(order, want.tolist()):
                assert abs(got[e] - v) < 2e-5
    zs = (h.double() @ w[:n].double().T).float().contiguous()
    i2, w2 = moe.route(zs.to(device), corr.to(device), top, score="softmax", renorm=True, scale=1.7)
    order, want = O.route(zs[0].double(), corr.double(), top, 1.7)
    assert sorted(i2[0].tolist()) == sorted(order) and abs(float(w2[0].sum()) - 1.7) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
def test_router_correction_decides_and_identity_wins(device):
    """A correction that lifts a low-scored output into the choice without touching its weight; tokens whose
    choices are all identity outputs; every token on one expert."""
    E, ident, top, T, W = 4, 2, 2, 9, 16
    w = torch.zeros(E + ident, W)
    for e in range(E + ident):
        w[e, e] = 1.0
    h = torch.zeros(T, W)
    h[:, :6] = torch.tensor([3.0, 2.0, 0.0, -1.0, 1.0, -2.0])
    corr = torch.zeros(E + ident)
    corr[5] = 2.0  # softmax score 0.0045: chosen for its correction, weighed without it
    idx, wt, _ = moe.router(h.to(device), w.to(device), E + ident, corr.to(device), top, score="softmax", renorm=True)
    s = torch.softmax(torch.tensor([3.0, 2.0, 0.0, -1.0, 1.0, -2.0]).double(), 0)
    assert idx.cpu().tolist() == [[5, 0]] * T
    assert torch.allclose(wt[3].cpu().double(), s[[5, 0]] / s[[5, 0]].sum(), atol=1e-6)
    corr[4] = 3.0
    idx, _, _ = moe.router(h.to(device), w.to(device), E + ident, corr.to(device), top, score="softmax", renorm=True)
    assert idx.cpu().tolist() == [[4, 5]] * T
    order, off = moe.plan(idx, E)  # nobody is chosen
    assert off.cpu().tolist() == [0] * (E + 1)
    x = torch.randn(T, W, device=device)
    we = torch.randn(E, 24, W, device=device)
    assert moe.grouped_gemm(x, we, order, off, top, gather=True, scatter=False).shape == (T * top, 24)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("T,E,top,identity,W,ff,shared", [(1, 3, 2, 1, 24, 8, 12), (50, 5, 3, 4, 40, 24, 0), (300, 6, 2, 2, 64, 64, 64),
                                                         (70, 1, 1, 1, 33, 7, 5)])
def test_routed_experts_alone(device, dtype, T, E, top, identity, W, ff, shared):
    """Routed, identity and shared experts together: the layer's pieces against the oracle's token by token sum."""
    L = routed(ssm(H=1, P=W, N=2, groups=1, norm_groups=1, conv=1), E=E, top=top, identity=identity, ff=ff, shared=shared)
    cfg = config([L], width=W)
    sd = weights(cfg, T)
    model = KilatarForCausalLM(cfg, device, DT[dtype]).load_state(sd)
    lw = model.layers[0]
    torch.manual_seed(T)
    h = torch.randn(T, W).to(DT[dtype])
    hd = h.to(device)
    idx, w, gates = moe.router(hd, lw["router"], lw["n_route"], lw["correction"], top, score="softmax", renorm=True, scale=1.5)
    y = torch.zeros(T, W, device=device)
    mx.residual_step(y, experts=model._experts(lw, hd, idx, w), out_dtype=DT[dtype])
    p = {k[len("l0.mlp."):]: v.double() for k, v in sd.items() if k.startswith("l0.mlp.")}
    want = O.moe_ff(h.double(), p, {**L["mlp"], "shared": None})
    assert torch.allclose(y.cpu().double(), want, **tol(dtype, 1e-4, 4e-2))
    if shared:
        gu = hd @ torch.cat([sd["l0.mlp.shared.gate"], sd["l0.mlp.shared.up"]]).to(device, DT[dtype]).t()
        act = mx.glu_act(gu, "silu", row_scale=gates.view(T))
        got = act @ sd["l0.mlp.shared.down"].to(device, DT[dtype]).t()
        ws = O.expert(h.double(), p, "shared.") * O.sigmoid(h.double() @ p["shared.sg"].T)
        assert torch.allclose(got.cpu().double(), ws, **tol(dtype, 1e-4, 4e-2))


@pytest.mark.gpu
@pytest.mark.parametrize("counts,K,N", [((0, 1, 16, 17, 5), 64, 32), ((3, 0, 2), 320, 96), ((40, 65, 2, 0, 31), 128, 192),
                                        ((130, 1, 64, 33, 12, 90), 704, 64), ((7,), 4096, 256)])
def test_few_rows_per_expert_stream_the_weights(monkeypatch, counts, K, N):
    """The weight-streaming grouped GEMM (bf16, few rows per expert): experts without rows, with one, and with more
    than one pass holds; widths that leave some of the waves without a piece; gathered rows in, scattered rows
    out; the SwiGLU epilogue; choices without an expert among the slots."""
    torch.manual_seed(K)
    monkeypatch.setattr(moe, "STREAM_ROWS", 1 << 20)
    monkeypatch.setattr(moe, "STREAM_TILES", 1 << 20)
    E, top = len(counts), 2
    flat = torch.cat([torch.full((c,), e) for e, c in enumerate(counts)] + [torch.full((4 + sum(counts) % 2,), E)])
    idx = flat[torch.randperm(flat.numel())].view(-1, top).to(torch.int32)
    T = idx.shape[0]
    order, offsets = moe.plan(idx.cuda(), E)
    n, o = int(offsets[-1]), order.cpu().long()
    assert n == sum(counts) and offsets.cpu().tolist() == [0] + torch.tensor(counts).cumsum(0).tolist()
    e_of = idx.reshape(-1).long()[o[:n]]
    a, w = torch.randn(T, K).bfloat16(), (torch.randn(E, N, K) * K ** -0.5).bfloat16()
    ac, wc = a.cuda(), w.cuda()
    assert moe.stream_gemm_ok(ac, wc, T * top)
    want = torch.stack([w[e].double() @ a[s // top].double() for e, s in zip(e_of.tolist(), o[:n].tolist())])
    got = moe.grouped_gemm(ac, wc, order, offsets, top, gather=True, scatter=False)[:n].cpu().double()
    assert float((got - want).abs().max()) < 3e-2
    b = torch.randn(T * top, K + 8).bfloat16()[:, :K]
    want = torch.stack([w[e].double() @ b[r].double() for r, e in enumerate(e_of.tolist())])
    got = moe.grouped_gemm(b.cuda(), wc, order, offsets, top, gather=False, scatter=True).cpu().double()
    assert float((got[o[:n]] - want).abs().max()) < 3e-2
    if N % 256 == 0 and K % 128 == 0:
        want = torch.stack([w[e].double() @ a[s // top].double() for e, s in zip(e_of.tolist(), o[:n].tolist())])
        got = moe.grouped_gemm(ac, moe.interleave_glu(wc), order, offsets, top, gather=True, scatter=False, glu=True)
        want = O.silu(want[:, :N // 2]) * want[:, N // 2:]
        assert float((got[:n].cpu().double() - want).abs().max()) < 3e-2


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("F,dv", [(24, 8), (21, 7), (1028, 4), (30, 10)])
def test_gated_units_alone(device, dtype, F, dv):
    """gelu (tanh form) with biases on both halves, a scale per row, a head-major second factor; into a section."""
    torch.manual_seed(F)
    T, dt = 5, DT[dtype]
    gu, gb, ub, rs = (torch.randn(T, 2 * F) * 2).to(dt), torch.randn(F), torch.randn(F), torch.rand(T)
    dev = lambda t: t.to(device)  # noqa: E731
    got = mx.glu_act(dev(gu), "gelu_tanh", gate_b=dev(gb), up_b=dev(ub), row_scale=dev(rs))
    g, u = gu[:, :F].double() + gb.double(), gu[:, F:].double() + ub.double()
    assert torch.allclose(got.cpu().double(), O.gelu_tanh(g) * u * rs.double()[:, None], **tol(dtype, 2e-5, 2e-2))
    if F == 24:  # many rows: a workgroup takes several
        gu = (torch.randn(2051, 2 * F) * 2).to(dt)
        got = mx.glu_act(dev(gu), "gelu_tanh", gate_b=dev(gb), up_b=dev(ub), row_scale=dev(rs.repeat(411)[:2051].contiguous()))
        g, u = gu[:, :F].double() + gb.double(), gu[:, F:].double() + ub.double()
        want = O.gelu_tanh(g) * u * rs.repeat(411)[:2051].double()[:, None]
        assert torch.allclose(got.cpu().double(), want, **tol(dtype, 2e-5, 2e-2))
        gu = gu[:T]
    H = F // dv
    up = torch.randn(H, T, dv).to(dt)
    out = torch.full((T, F + 4), 9.0, device=device, dtype=dt)
    mx.act_mul(dev(gu)[:, F:], dev(up), "sigmoid", out=out[:, 4:])
    want = O.sigmoid(gu[:, F:].double()) * up.double().transpose(0, 1).reshape(T, F)
    assert torch.allclose(out[:, 4:].cpu().double(), want, **tol(dtype, 2e-5, 2e-2)) and bool((out[:, :4] == 9.0).all())


def test_scaled_frequencies():
    """All three bands of the scaling, their edges, and none."""
    for dims, base, sc in ((40, 200000.0, {"factor": 6.0, "low": 1.0, "high": 5.0, "original": 700}), (8, 100.0, SCALING),
                           (2, 10.0, None), (64, 1e4, {"factor": 2.0, "low": 2.0, "high": 3.0, "original": 100})):
        rot = {"dims": dims, "base": base, **({"scaling": sc} if sc else {})}
        want = torch.tensor(O.frequencies(rot), dtype=torch.float64)
        assert torch.allclose(rc.rotary_frequencies(dims, base, sc).double(), want, rtol=1e-6)
    f = torch.tensor(O.frequencies({"dims": 40, "base": 200000.0, "scaling": {"factor": 6.0, "low": 1.0, "high": 5.0,
                                                                               "original": 700}}))
    plain = torch.tensor(O.frequencies({"dims": 40, "base": 200000.0}))
    assert float((f / plain).max()) == 1.0 and abs(float((f / plain).min()) - 1 / 6) < 1e-6
    assert bool(((f / plain > 0.17) & (f / plain < 0.99)).any())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,G,d,dv,dims,n_act", [(4, 2, 12, 20, 8, 34), (6, 2, 7, 9, 6, 41), (1, 1, 2, 4, 2, 3), (2, 1, 64, 128, 64, 320),
                                                 (3, 3, 9, 5, 0, 7), (32, 8, 128, 128, 128, 4096)])
def test_rotary_cache_and_second_section_alone(device, dtype, H, G, d, dv, dims, n_act):
    """Rotation without a norm, cache write at scattered slots, silu on a later section and nothing else."""
    torch.manual_seed(d)
    T, dt = 6, DT[dtype]
    nq, nk, nv = H * d, G * d, G * dv
    x = torch.randn(T, nq + nk + nv + n_act + 11).to(dt)
    pos = torch.tensor([0, 1, 5, 130, 131, 999])
    slots = torch.tensor([3, 0, -1, 17, 9, 30])
    inv = rc.rotary_frequencies(dims, 1e4, {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 60}).to(device) if dims else None
    xd = x.clone().to(device)
    kc = torch.full((32, nk), 9.0, device=device, dtype=dt)
    vc = torch.full((32, nv), 9.0, device=device, dtype=dt)
    a0 = nq + nk + nv
    mx.norm_rope_cache(xd, pos.to(device), slots.to(device), H, G, d, nv, None, None, 0.0, inv, kc, vc, silu=(a0, n_act))
    rot = {"dims": dims, "base": 1e4, "scaling": SCALING}
    q, k = (O.rotate_pairs(t, pos, rot) if dims else t for t in (x[:, :nq].double().view(T, H, d),
                                                                 x[:, nq:nq + nk].double().view(T, G, d)))
    tl = dict(atol=2e-3, rtol=1e-4) if dtype == "float32" else dict(atol=2e-2, rtol=1e-2)  # (angles up to 1000 in fp32)
    assert torch.allclose(xd[:, :nq].cpu().double(), q.reshape(T, -1), **tl)
    assert torch.equal(xd[:, nq:a0].cpu(), x[:, nq:a0]) and torch.equal(xd[:, a0 + n_act:].cpu(), x[:, a0 + n_act:])
    assert torch.allclose(xd[:, a0:a0 + n_act].cpu().double(), O.silu(x[:, a0:a0 + n_act].double()), **tol(dtype, 1e-5, 1e-2))
    ok = slots >= 0
    assert torch.allclose(kc[slots[ok]].cpu().double(), k.reshape(T, -1)[ok], **tl)
    assert torch.equal(vc[slots[ok]].cpu(), x[ok, nq + nk:a0])
    untouched = torch.ones(32, dtype=torch.bool)
    untouched[slots[ok]] = False
    assert bool((kc.cpu()[untouched] == 9.0).all()) and bool((vc.cpu()[untouched] == 9.0).all())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,d,dr,r,dims", [(3, 12, 8, 24, 8), (2, 5, 6, 7, 4), (4, 32, 32, 64, 32), (1, 8, 8, 8, 0), (8, 64, 64, 192, 64),
                                           (2, 16, 16, 32, 6)])
def test_latent_rope_interleaved_alone(device, dtype, H, d, dr, r, dims):
    """Latent norm, neighbouring pairs rotated (all of a part or its head), cache row, assembled queries."""
    torch.manual_seed(r)
    T, eps, dt = 5, 1e-3, DT[dtype]
    qa, q, kv, cn = torch.randn(H, T, r).to(dt), torch.randn(T, H * (d + dr)).to(dt), torch.randn(T, r + dr).to(dt), torch.randn(r)
    pos, slots = torch.tensor([0, 1, 7, 64, 300]), torch.tensor([4, -1, 2, 0, 6])
    rot = {"dims": dims, "base": 1e4}
    inv = rc.rotary_frequencies(dims, 1e4).to(device) if dims else None
    cache = torch.full((8, r + dr), 9.0, dtype=dt, device=device)
    got = rc.latent_rope(qa.to(device), section(q, 8, device), d + dr, d, section(kv, 16, device), r, dr, cn.to(device), eps, inv,
                         1.0, pos.to(device), slots.to(device), cache, interleaved=True)
    qr = O.rotate_pairs(q.double().view(T, H, d + dr)[..., d:], pos, rot)
    want = torch.cat([qa.double().transpose(0, 1), qr], -1).reshape(T, -1)
    assert torch.allclose(got.cpu().double(), want, **tol(dtype, 1e-4, 2e-2))
    row = torch.cat([O.unit_rms(kv[:, :r].double(), eps) * cn.double(), O.rotate_pairs(kv[:, None, r:].double(), pos, rot)[:, 0]], -1)
    ok = slots >= 0
    assert torch.allclose(cache[slots[ok]].cpu().double(), row[ok], **tol(dtype, 1e-4, 2e-2))
    assert bool((cache[[1, 3, 5, 7]] == 9.0).all())


SCAN_T = 150


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,dk,dv", [(3, 10, 14), (1, 1, 1), (2, 64, 64), (4, 128, 128), (1, 34, 3), (2, 32, 80)])
def test_lightning_scan_alone(device, dtype, H, dk, dv):
    """S <- decay S + k v^T, o = S^T q with decays from a half to none, whole and in unequal portions of two
    sequences side by side, in slots that hold garbage."""
    torch.manual_seed(dk)
    dt = DT[dtype]
    q, k, v = (torch.randn(2, SCAN_T, H * n).to(dt) for n in (dk, dk, dv))
    decay = torch.tensor([0.5, 1.0, 0.9, 0.99][:H])
    want = [O.lightning_scan(q[s].double().view(SCAN_T, H, dk), k[s].double().view(SCAN_T, H, dk),
                             v[s].double().view(SCAN_T, H, dv), decay.double().tolist()) for s in range(2)]
    for portions in [[(150,), (150,)], [(19, 2, 1, 1, 9, 8, 1, 64, 45), (3, 30, 7, 1, 65, 16, 17, 11)]]:
        state = torch.randn(4, H, dv, dk, device=device)
        it, at, got = [list(p) for p in portions], [0, 0], [[], []]
        while any(it):
            live = [s for s in range(2) if it[s]]
            cuts = [(at[s], it[s].pop(0)) for s in live]
            pos, _, seq_rows, slots = step_meta(device, cuts, [(3, 1)[s] for s in live])
            qs, ks, vs = (section(torch.cat([t[s, p:p + n] for s, (p, n) in zip(live, cuts)]), 8, device) for t in (q, k, v))
            o = rc.retention(qs, ks, vs, decay.to(device), 1.0, state, pos, seq_rows, slots, H, dk, dv)
            for i, (s, (p, n)) in enumerate(zip(live, cuts)):
                got[s].append(o[int(seq_rows[i]):int(seq_rows[i + 1])].cpu())
                at[s] = p + n
        for s in range(2):
            w, S = want[s]
            scale = float(w.abs().max())
            assert float((torch.cat(got[s]).double() - w.reshape(SCAN_T, -1)).abs().max()) < 1e-4 * max(1.0, scale)
            assert float((state[3 - 2 * s].cpu().double().transpose(1, 2) - S).abs().max()) < 1e-4 * max(1.0, float(S.abs().max()))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,dv", [(3, 14), (1, 1), (5, 64), (32, 128), (7, 9), (72, 128), (27, 19)])
def test_norm_over_all_heads_and_gate_alone(device, dtype, H, dv):
    torch.manual_seed(dv)
    T, eps, dt = 5, 1e-3, DT[dtype]
    o, z, w = torch.randn(T, H * dv) * 3, (torch.randn(T, H * dv + 8) * 2).to(dt), torch.randn(H * dv)
    got = rc.head_norm_gate(o.to(device), 1, w.to(device), z.to(device)[:, 8:], eps, dt)
    want = O.unit_rms(o.double(), eps) * w.double() * O.sigmoid(z[:, 8:].double())
    assert torch.allclose(got.cpu().double(), want, **tol(dtype))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H,P,N,groups,norm_groups,conv", [(6, 10, 14, 2, 3, 3), (1, 1, 1, 1, 1, 1), (4, 64, 64, 1, 4, 4), (5, 3, 17, 5, 5, 6)])
def test_mamba2_mixer_alone(device, dtype, H, P, N, groups, norm_groups, conv):
    """The whole mixer of one layer (convolution, step sizes, scan, gate, norm in parts, output projection)."""
    cfg = config([dense(ssm(H, P, N, groups, norm_groups, conv), 0)], width=40)
    sd = weights(cfg, 3)
    model = KilatarForCausalLM(cfg, device, DT[dtype]).load_state(sd)
    L, T = model.layers[0], 37
    h = torch.randn(T, 40, generator=torch.Generator().manual_seed(1)).to(DT[dtype])
    state = [s.normal_() for s in model.alloc_state(2)]
    want = O.mamba2(h.double(), {k[len("l0.mix."):]: v.double() for k, v in sd.items() if k.startswith("l0.mix.")},
                    L["m"], cfg.rms_norm_eps)
    got, at = [], 0
    for n in (1, 2, 20, 1, 13):
        pos, row_seq, seq_rows, slots = step_meta(device, [(at, n)], [1])
        meta = type("M", (), dict(positions=pos, is_prefill=True, row_seq=row_seq, seq_rows=seq_rows, state_slots=slots))()
        o = torch.empty(n, H * P, dtype=DT[dtype], device=device)
        model._mamba2(L, h[at:at + n].to(device) @ L["w_in"].t(), o, meta, *state)
        got.append((o @ L["w_out"].t()).cpu())
        at += n
    assert torch.allclose(torch.cat(got).double(), want, **tol(dtype, 2e-4, 6e-2))


# ----------------------------------------------------------------- attention: masks, widths, one key that stands out
def dense_rows(q, k, v, ps, scale, chunk):
    """q [n, H, d] at positions ps, k / v [T, H, .] per query head -> [n, H, dv]."""
    T = k.shape[0]
    vis = O.visible(T, chunk)[ps]
    return torch.stack([torch.softmax((q[:, h] @ k[:, h].T * scale).masked_fill(~vis, float("-inf")), -1) @ v[:, h]
                        for h in range(q.shape[1])], 1)


CHUNK_DIMS = [(64, 64, 4, 2, 64), (128, 128, 8, 2, 64), (64, 64, 3, 3, 64), (32, 64, 4, 2, 16), (12, 20, 4, 1, 8), (128, 128, 12, 2, 128)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("d,dv,H,G,bs", CHUNK_DIMS)
@pytest.mark.parametrize("chunk", [1, 50, 64, 100])
def test_chunk_mask_alone(device, dtype, d, dv, H, G, bs, chunk):
    """Prompt portions that start before, at and behind chunk edges and span several, beside decode rows at a
    chunk's first and last position, keys in parts; unused rows of the pages hold NaN."""
    torch.manual_seed(d + chunk)
    dt = DT[dtype]
    chunks = [(0, 150), (37, 173), (chunk, 2), (max(0, chunk - 1), 130), (2 * chunk, 1), (2 * chunk - 1, 1), (209, 1)]
    n_dec, B, T = 3, len(chunks), 230
    per = -(-T // bs)
    k, v = torch.randn(B, T, G, d).to(dt), torch.randn(B, T, G, dv).to(dt)
    table = torch.randperm(B * per, generator=torch.Generator().manual_seed(1)).to(torch.int32).view(B, per)
    kc = torch.full((B * per * bs, G * d), float("nan"), dtype=dt)
    vc = torch.full((B * per * bs, G * dv), float("nan"), dtype=dt)
    q = torch.randn(sum(n for _, n in chunks), H, d).to(dt)
    want, tiles, r0 = torch.zeros(q.shape[0], H, dv, dtype=torch.float64), [], 0
    for b, (p, n) in enumerate(chunks):
        j = torch.arange(p + n)
        sl = table[b].long()[j // bs] * bs + j % bs
        kc[sl], vc[sl] = k[b, :p + n].reshape(p + n, -1), v[b, :p + n].reshape(p + n, -1)
        kh, vh = (t[b, :p + n].double().repeat_interleave(H // G, 1) for t in (k, v))
        want[r0:r0 + n] = dense_rows(q[r0:r0 + n].double(), kh, vh, torch.arange(p, p + n), 0.2, chunk)
        if b < B - n_dec:
            tiles += mx.tile_list(r0, n)
        r0 += n
    pos, row_seq, _, _ = step_meta(device, chunks, [0] * B)
    tl = torch.tensor(tiles, dtype=torch.int32, device=device)
    for parts in (1, 3):
        got = mx.attention(q.reshape(r0, -1).to(device), kc.to(device), vc.to(device), pos, row_seq, table.to(device), bs, H, 1,
                           H // G, d, dv, 0.2, "chunk", chunk, parts, False, tl, r0 - n_dec)
        diff = (got.cpu().double() - want).abs()
        assert float(diff.max()) < (2e-4 if dtype == "float32" else 3e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("r,dr,H", [(64, 32, 3), (64, 32, 20), (128, 32, 4), (128, 64, 8), (192, 64, 4), (24, 8, 3)])
def test_latent_widths_alone(device, dtype, r, dr, H):
    """One [latent | key part] row as key and value of all heads: prompt portions and decode rows of every width
    the matrix-core kernels have for it, and one they have not."""
    torch.manual_seed(r)
    dt, bs, d = DT[dtype], 64, r + dr
    chunks, T = [(0, 140), (70, 66), (129, 1), (64, 1)], 140
    B, per = len(chunks), -(-T // 64)
    rows = torch.randn(B, T, d).to(dt)
    table = torch.randperm(B * per, generator=torch.Generator().manual_seed(1)).to(torch.int32).view(B, per)
    cache = torch.full((B * per * bs, d), float("nan"), dtype=dt)
    q = torch.randn(sum(n for _, n in chunks), H, d).to(dt)
    want, r0 = torch.zeros(q.shape[0], H, r, dtype=torch.float64), 0
    for b, (p, n) in enumerate(chunks):
        j = torch.arange(p + n)
        cache[table[b].long()[j // bs] * bs + j % bs] = rows[b, :p + n]
        kh = rows[b, :p + n].double()[:, None, :].expand(-1, H, -1)
        want[r0:r0 + n] = dense_rows(q[r0:r0 + n].double(), kh, kh[..., :r], torch.arange(p, p + n), 0.1, 0)
        r0 += n
    pos, row_seq, _, _ = step_meta(device, chunks, [0] * B)
    tl = torch.tensor(mx.tile_list(0, 140) + mx.tile_list(140, 66), dtype=torch.int32, device=device)
    c = cache.to(device)
    for parts in (1, 2):
        got = mx.attention(q.reshape(r0, -1).to(device), c, c, pos, row_seq, table.to(device), bs, H, 1, H, d, r, 0.1, "causal", 0,
                           parts, False, tl, r0 - 2)
        diff = (got.cpu().double() - want).abs()
        assert float(diff.max()) < (2e-4 if dtype == "float32" else 3e-2) * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("d,dv,bs", [(32, 32, 16), (12, 20, 8), (64, 64, 64), (128, 128, 64), (96, 64, 64)])
@pytest.mark.parametrize("chunk", [0, 40, 64, 96])
def test_far_keys_and_chunk_edges(device, dtype, d, dv, bs, chunk):
    """A cache of empty keys in which one matches the query strongly and carries a marked value: a chunk's first
    key and the last one before it, page borders, the sequence's first token, the query's own and the one behind
    it.  Prompt rows and decode rows (keys in parts) alike."""
    H, T = 2, 330
    dt = DT[dtype]
    perm = torch.randperm(48, generator=torch.Generator().manual_seed(3)).to(torch.int32)
    table = perm[: -(-T // bs)][None].contiguous().to(device)
    j = torch.arange(T, device=device)
    slots = table[0].long()[j // bs] * bs + j % bs
    e0 = torch.zeros(d)
    e0[0] = 8.0
    q = e0.repeat(H)[None].to(device, dt)
    kc = torch.zeros(48 * bs, d, device=device, dtype=dt)
    vc = torch.zeros(48 * bs, dv, device=device, dtype=dt)
    c = chunk or T + 1
    for p in {T - 1, 150, min(c, 299), min(2 * c - 1, T - 1), min(3 * c, 320), 0}:
        lo = p // c * c
        for mark in {0, 1, p, p + 1, p - 1, lo, lo - 1, lo + 1, p // bs * bs, p // bs * bs - 1}:
            if not 0 <= mark < T:
                continue
            K, V = torch.zeros(T, d), torch.full((T, dv), -1.0)
            K[mark], V[mark] = e0, 1.0
            kc[slots], vc[slots] = K.to(device, dt), V.to(device, dt)
            seen = lo <= mark <= p
            hit, rest = math.exp(16.0) if seen else 0.0, p - lo + (0 if seen else 1)
            want = (hit - rest) / (hit + rest)
            pos = torch.tensor([p], device=device)
            for seq, parts in ((torch.zeros(1, dtype=torch.int32, device=device), 1), (None, 1), (None, 3)):
                tl = (torch.tensor([[0, 1]], dtype=torch.int32, device=device), 1) if seq is not None else (None, 0)
                got = mx.attention(q, kc, vc, pos, seq, table, bs, H, 1, H, d, dv, 0.25, "chunk" if chunk else "causal", chunk,
                                   parts, False, *tl)
                err = float((got.float() - want).abs().max())
                assert err < (1e-4 if dtype == "float32" else 2e-2), (p, mark, seq is None, parts, err)


# ----------------------------------------------------------------- whole model
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_layers(device, dtype, name):
    """A whole prompt in one step: logits at every position, and (float32) the residual after every layer run."""
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
        assert len(eng.model.trace_layers) == len(cfg.layer_runs()) == len(after)
        for i, (x, w) in enumerate(zip(eng.model.trace_layers, after)):
            assert float((x.cpu().double() - w).abs().max()) < 1e-3 * float(w.abs().max()), f"layer run {i}"
        eng.model.trace_layers = None  # (with the residual steps joined across layers)
        close(eng.forced_step([("b", toks, list(range(len(toks))))], ["b"])["b"], want, dtype, name)


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


@pytest.mark.parametrize("device", DEVICES)
def test_batch_and_cuts_change_nothing(device):
    """The same request alone in one step, in portions, and in portions beside others and in other pages and
    slots: equal logits beyond float32 rounding."""
    cfg = CONFIGS["mixed"]()
    sd = weights(cfg, 12)
    a, b = tokens(70, cfg.vocab_size, 13), tokens(64, cfg.vocab_size, 14)
    one = run_cut(engine(cfg, sd, device, "float32"), "a", a, (70,)).double().cpu()
    eng, got, p = engine(cfg, sd, device, "float32", blocks=24, bs=8, seqs=2), [], 0
    eng.forced_step([("b", b[:33], [])], [])
    for i, n in enumerate((2, 24, 1, 2, 30, 1, 10)):
        ent = [("a", a[p:p + n], list(range(n)))] + ([("b", b[33 + 6 * i:39 + 6 * i], [])] if i < 5 else [])
        got.append(eng.forced_step(ent, ["b"] if i == 4 else [])["a"])
        p += n
    assert float((torch.cat(got).double().cpu() - one).abs().max()) < 1e-4 * float(one.abs().max())


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_decode_and_first_tokens(device, dtype):
    """146 consecutive decode steps after a two-token prompt: the first positions (fewer tokens than taps), chunk
    edges passed while decoding."""
    cfg = CONFIGS["mixed"]()
    sd = weights(cfg, 6)
    toks = tokens(148, cfg.vocab_size, 7)
    want, _ = O.forward(cfg_dict(cfg), sd, toks)
    close(run_cut(engine(cfg, sd, device, dtype), "a", toks, (2,)), want, dtype, "long decode")


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("bs", [8, 64])
def test_long_prompt_portions(device, dtype, bs):
    """A prompt of several hundred tokens in portions that end inside and at the edges of the kernels' token
    blocks, tiles and the chunks (63, 64, 65, 128 + 1, ...), beside a second sequence."""
    cfg = config([routed(par(H=4, G=2, d=64, dv=64, dims=32, base=1e4, chunk=96, Hr=2, dk=64, dvr=64), E=4, ff=32, shared=32),
                  dense(lat(H=4, d=16, dr=32, dv=16, r=64, base=1e4), 32),
                  dense(ssm(H=2, P=64, N=64, groups=1, norm_groups=1, conv=4), 32)], width=32, loop=span(0, 2, 2))
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
    variants -- another chunk or rotation, a plain sum of the two sides, no shared expert, another router scale,
    no correction, one pass fewer, no re-entering embedding, ... -- differ visibly."""
    cfg = config([routed(par(H=2, G=1, d=16, dv=16, dims=16, chunk=20, scale=1.0, Hr=2, dk=16, dvr=16), shared=24),
                  dense(lat(H=2, d=8, dr=16, dv=16, r=24, scale=1.0)),
                  dense(ssm(H=4, P=8, N=16, groups=2, norm_groups=2))], width=48, vocab=61, loop=span(0, 2, 2))
    sd = weights(cfg, 8)
    sd["l2.mix.dt_bias"] = torch.full((4,), -1.0).bfloat16()
    sd["l0.mlp.correction"] = torch.tensor([0.0, 0.6, 0.0, 0.0, 0.0, 0.3, 0.0]).bfloat16()
    toks = tokens(60, cfg.vocab_size, 9)
    base = cfg_dict(cfg)
    want, _ = O.forward(base, sd, toks)
    close(run_cut(engine(cfg, sd, device, dtype), "a", toks, (13, 2, 30)), want, dtype, "crafted")

    def differs(change):
        c, s2 = copy.deepcopy(base), dict(sd)
        change(c, s2)
        off = O.forward(c, s2, toks)[0]
        return float((off - want).abs().max()) > 0.02 * float(want.abs().max())

    def mixer(c, i, *path):
        m = c["layers"][i]["mixer"]
        for k in path:
            m = m[k]
        return m

    assert differs(lambda c, s: mixer(c, 0, "left", "mask").update(size=21))
    assert differs(lambda c, s: mixer(c, 0, "left", "rot").pop("scaling"))
    assert differs(lambda c, s: mixer(c, 0, "left", "rot").update(dims=14))
    assert differs(lambda c, s: mixer(c, 0, "right").update(decay=[0.5, 0.8]))
    assert differs(lambda c, s: s.update({"l0.mix.left.out": sd["l0.mix.left.out"] * 2}))
    assert differs(lambda c, s: mixer(c, 1, "rot").update(base=50.0))
    assert differs(lambda c, s: mixer(c, 1).update(scale=0.7))
    assert differs(lambda c, s: s.update({"l1.mix.g": sd["l1.mix.g"] * 0}))
    assert differs(lambda c, s: mixer(c, 2).update(norm_groups=1))
    assert differs(lambda c, s: s.update({"l2.mix.D": sd["l2.mix.D"] * 0}))
    assert differs(lambda c, s: s.update({"l2.mix.A_log": sd["l2.mix.A_log"] + 0.3}))
    assert differs(lambda c, s: s.update({"l2.mix.conv.b": sd["l2.mix.conv.b"] * 0}))
    for b in ("gate.b", "up.b", "down.b"):
        assert differs(lambda c, s: s.update({"l1.mlp." + b: sd["l1.mlp." + b] * 0}))
    assert differs(lambda c, s: c["layers"][0]["mlp"].update(shared=None))
    assert differs(lambda c, s: s.update({"l0.mlp.shared.sg": sd["l0.mlp.shared.sg"] * 0}))
    assert differs(lambda c, s: c["layers"][0]["mlp"]["router"].update(scale=1.0))
    assert differs(lambda c, s: s.update({"l0.mlp.correction": sd["l0.mlp.correction"] * 0}))
    assert differs(lambda c, s: c["loop"].update(times=1))
    assert differs(lambda c, s: s.update({"embed.norm": sd["embed.norm"] * 1.5}))
    real = O.layer_order
    O.layer_order = lambda c: [(i, False) for i, _ in real(c)]
    try:
        assert differs(lambda c, s: None)  # the embedding output does not come back
    finally:
        O.layer_order = real


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
    model = KilatarForCausalLM(cfg, device, DT[dtype]).load_state(sd)
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
            assert gap < (1e-3 if dtype == "float32" else 0.15 * float(row.std())), (i, gap)


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
    close(torch.cat([got[0], got[1], got[3]]), torch.cat([wa[[0, 24]], wb[[1]], wa[[25]], wb[[2, 8]], wb[[8]]]), dtype, "replay")


def test_config_round_trip(tmp_path):
    """config.json keys -> LayeredConfig -> config.json; the loop's runs; the presets build and count their weights."""
    cfg = CONFIGS["mixed"]()
    cfg.write_hf_config(str(tmp_path))
    back = get_config(str(tmp_path))
    assert back.architecture == "Kilatar" and back.layers == cfg.layers and back.loop == cfg.loop
    assert back.layer_runs() == [0, 1, 2, 3, 1, 2, 3, 4, 5] and back.loop_reentries() == [4]
    assert config(cfg.layers).loop_reentries() == [] and config(cfg.layers, loop=span(0, 6, 1)).loop_reentries() == []
    assert config(cfg.layers, loop=span(2, 2, 3)).layer_runs() == list(range(6))
    assert config(cfg.layers, loop=span(2, 2, 3)).loop_reentries() == []
    assert config(cfg.layers, loop=span(4, 6, 3)).loop_reentries() == [6, 8]
    tiny = get_config("kilatar-tiny")
    model = KilatarForCausalLM(tiny, "cpu", torch.float32)
    sd = model.random_state(0)
    assert sum(v.numel() for v in sd.values()) == tiny.num_params()
    model.load_state(sd)
    kv = model.alloc_kv_caches(2, 4, torch.float32)  # a cache and a state per run: layers 0, 1, 2, 1, 2, 3, 4
    assert len(kv) == 7 and kv[1][0] is kv[1][1] and kv[1][0].data_ptr() != kv[3][0].data_ptr()
    assert kv[2][0].numel() == 0 and kv[0][0].data_ptr() != kv[0][1].data_ptr()
    assert len(model.alloc_state(1)) == 2 + 2 * 2
    from dynamo_exp_amd.models.registry import build_model, supports_dtype

    assert supports_dtype("Kilatar", "float32") and supports_dtype("Kilatar", "bfloat16")
    assert isinstance(build_model(back, "cpu", dtype="float32"), KilatarForCausalLM)
    for bad in ([{"type": "gla", "mixer": {"heads": 1, "dim": 8}, "mlp": None}], [dense(par(H=3, G=2))],
                [dense(par(Hr=2, decay=[0.5]))], [dense(lat(dr=4, dims=6))], [dense(ssm(H=3, groups=2))]):
        with pytest.raises(ValueError):
            KilatarForCausalLM(config(bad), "cpu", torch.float32)
