"""Kilatar: a layer-listed hybrid decoder for the MI355X engine: latent
attention, Mamba-2 and layers in which chunked softmax attention and lightning
attention (linear attention with a fixed decay per head) run side by side, all
in parallel with a dense or routed feed-forward that reads the same normed
input; a span of layers may run several times in a row (`loop`), each pass with
a cache and state of its own and, from the second on, with the embedding output
added in front.

x <- x + (mixer(h) + ff(h)), h = rms(x) w: one norm and one residual step per
layer.  Everything that reads h is one projection (the mixer's sections, then
the gate and up rows of the dense or shared feed-forward), and where nothing
stands between the mixer's output projection and the sum, the feed-forward's
down projection shares its GEMM: [o | act] @ [Wo | Wdown]^T is the sum of both.
Per layer run, T rows of one engine step (prompt chunks and decode tokens of
different sequences; state per sequence in the slot the engine assigned):

  latent_attention
    p  = h @ [Wq | Wdkv | Wg | Wgate | Wup]^T              hipBLASLt
    qa = q_unrotated @ Wuk (per head)                      batched GEMM: the key up-projection folded into the query
    q' = latent_rope(qa, q, p_dkv)                         HIP  latent norm, interleaved rotary, cache row [latent | key part]
    a  = attention(q', cache, cache)                       HIP  one key/value head shared by all query heads
    o  = sigmoid(p_g) (a @ Wuv per head)                   batched GEMM + HIP act_mul (reads the heads as they lie)
  mamba2
    p  = h @ [Wz | Wx | WB | WC | Wgate | Wup | Wdt]^T
    c  = causal_conv(p_xBC, bias, silu)                    HIP  short convolution over time, tail state per slot
    s  = ssd(c_x, c_B, c_C, p_dt; S)                       HIP  S <- exp(-rate u) S + u B x^T, y = S^T C + D x, fp32
    o  = gate_group_norm(s, p_z)                           HIP
  parallel
    p  = h @ [Wq Wk Wv | Wq Wk Wv Wg (right) | Wgate | Wup]^T
         norm_rope_cache(p)                                HIP  left: rotary, K / V into the pages; right: silu on q, k, v
    yl = attention(q, K, V; chunk mask) @ Wo^T             HIP + hipBLASLt
    yr = head_norm_gate(retention(q, k, v; S)) @ Wo^T      HIP  S <- decay S + k v^T, o = S^T q, fp32; norm over all heads
  feed-forward
    dense: act = gelu(p_gate + b) (p_up + b)               HIP act_mul
    moe:   choice, weights, shared gate = router(h)        HIP  fp32 logits, softmax, correction, choice: one kernel
           plan -> grouped GEMMs (SwiGLU in the epilogue)  HIP
           shared act = silu(p_gate) p_up sigmoid(h.w_sg)  HIP act_mul
  residual
    X += a + rms(yl) wl/2 + rms(yr) wr/2 + bias + sum_k w_k y_k (+ embedding output);  h = rms(X) w
                                                           HIP residual_step: one pass, identity outputs read h

Positions and angles, scores and weights, norms, router, residual, decays, step
sizes and the recurrent states are fp32; projections, the convolution and
activations are bf16 (dtype=bfloat16) or everything is fp32 (dtype=float32).
"""
from __future__ import annotations

import torch

from ..ops import mixers as mx
from ..ops import moe
from ..ops import recurrent as rc
from .config import LayeredConfig
from .layered import IN_PAD, StatefulLayeredModel
from .llama import AttnMeta, TPGroup

MIXERS = ("latent_attention", "mamba2", "parallel")


class KilatarForCausalLM(StatefulLayeredModel):
    LINEARS = ("w_in", "w_out", "w_lo", "w_ro", "w_down")

    def __init__(self, cfg: LayeredConfig, device: torch.device | str = "cuda", dtype=torch.bfloat16,
                 tp: TPGroup | None = None):
        super().__init__(cfg, device, dtype, tp)
        if cfg.streams:
            raise ValueError("Kilatar has no parallel residual streams")
        for i, L in enumerate(cfg.layers):
            m, mlp = L["mixer"], L.get("mlp")
            if L["type"] not in MIXERS:
                raise ValueError(f"unknown mixer type {L['type']!r}")
            if mlp and mlp.get("kind") not in ("dense", "moe"):
                raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
            if L["type"] == "parallel":
                a, b = m["left"], m["right"]
                if a["heads"] % a["kv_heads"]:
                    raise ValueError(f"layer {i}: {a['heads']} heads over {a['kv_heads']} key/value heads")
                if len(b["decay"]) != b["heads"]:
                    raise ValueError(f"layer {i}: {len(b['decay'])} decays for {b['heads']} heads")
            elif L["type"] == "mamba2" and (m["heads"] % m["groups"] or (m["heads"] * m["vdim"]) % m["norm_groups"]):
                raise ValueError(f"layer {i}: state-space heads or channels do not divide into their groups")
            rot, width = (m["left"].get("rot"), m["left"]["dim"]) if L["type"] == "parallel" else \
                (m.get("rot"), m.get("rot_dim", 0))
            if int((rot or {}).get("dims") or 0) > width:
                raise ValueError(f"layer {i}: {rot['dims']} rotated dimensions in a part of {width}")
        self.runs = cfg.layer_runs()
        self.reentry = set(cfg.loop_reentries())
        # per layer run, the index of its convolution tail and of its running matrices in the state list
        self._state_index: list[tuple[int | None, int | None]] = []
        self.state_shapes()

    # ------------------------------------------------------------------ paged caches and state slots
    def cache_widths(self) -> list[tuple[int, int] | None]:
        out: list[tuple[int, int] | None] = []
        for li in self.runs:
            L = self.cfg.layers[li]
            m = L["mixer"]
            if L["type"] == "latent_attention":
                out.append((m["kv_rank"] + m["rot_dim"], 0))
            elif L["type"] == "parallel":
                a = m["left"]
                out.append((a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]))
            else:
                out.append(None)
        return out

    @staticmethod
    def _conv_channels(m: dict) -> int:
        return m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]

    def state_shapes(self) -> list[tuple[tuple, torch.dtype]]:
        """Per layer run: the running matrices (fp32, column by column), and in
        front of a Mamba-2 layer's the last taps - 1 projected rows before the
        short convolution."""
        out, index = [], []
        for li in self.runs:
            L = self.cfg.layers[li]
            m, ci, ri = L["mixer"], None, None
            if L["type"] == "mamba2":
                ci = len(out)
                out.append(((int(m["conv"]) - 1, self._conv_channels(m)), self.dtype))
                ri = len(out)
                out.append(((m["heads"], m["vdim"], m["state"]), torch.float32))
            elif L["type"] == "parallel":
                b = m["right"]
                ri = len(out)
                out.append(((b["heads"], b["vdim"], b["dim"]), torch.float32))
            index.append((ci, ri))
        self._state_index = index
        return out

    # ------------------------------------------------------------------ weights
    def random_state(self, seed: int = 0) -> dict[str, torch.Tensor]:
        """Random weights in the checkpoint's naming and dtypes (bf16), scaled
        so activations stay O(1)."""
        cfg = self.cfg
        g = torch.Generator().manual_seed(seed)
        W = cfg.hidden_size

        def rnd(*shape, std):
            return (torch.randn(*shape, generator=g) * std).to(torch.bfloat16)

        def lin(rows, cols):
            return rnd(rows, cols, std=cols ** -0.5)

        def near(n, mean=1.0, std=0.1):
            return (mean + torch.randn(n, generator=g) * std).to(torch.bfloat16)

        def uni(n, lo, hi):
            return (lo + (hi - lo) * torch.rand(n, generator=g)).to(torch.bfloat16)

        sd = {"embed": rnd(cfg.vocab_size, W, std=1.0), "embed.norm": near(W), "final.norm": near(W),
              "head": lin(cfg.vocab_size, W)}
        for i, L in enumerate(cfg.layers):
            m, p, q, mlp = L["mixer"], f"l{i}.mix.", f"l{i}.mlp.", L.get("mlp")
            sd[f"l{i}.norm1"] = near(W)
            if L["type"] == "latent_attention":
                H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
                sd[p + "q"], sd[p + "dkv"], sd[p + "dkv.norm"] = lin(H * (d + dr), W), lin(r + dr, W), near(r)
                sd[p + "uk"], sd[p + "uv"] = lin(H * d, r), lin(H * dv, r)
                sd[p + "g"], sd[p + "o"] = lin(H * dv, W), lin(W, H * dv)
            elif L["type"] == "mamba2":
                Hs, inner, C, taps = m["heads"], m["heads"] * m["vdim"], self._conv_channels(m), int(m["conv"])
                sd[p + "in"] = lin(inner + C + Hs, W)
                sd[p + "conv"], sd[p + "conv.b"] = rnd(C, taps, std=taps ** -0.5), rnd(C, std=0.1)
                sd[p + "dt_bias"], sd[p + "A_log"] = uni(Hs, -4.0, -1.0), uni(Hs, 0.0, 2.5)
                sd[p + "D"], sd[p + "norm"], sd[p + "o"] = near(Hs, std=0.2), near(inner), lin(W, inner)
            else:
                a, b = m["left"], m["right"]
                H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
                for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                    sd[p + "left." + n] = lin(rows, W)
                sd[p + "left.o"], sd[p + "left.out"] = lin(W, H * dv), near(W, 0.7)
                H, d, dv = b["heads"], b["dim"], b["vdim"]
                for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                    sd[p + "right." + n] = lin(rows, W)
                sd[p + "right.norm"], sd[p + "right.o"], sd[p + "right.out"] = near(H * dv), lin(W, H * dv), near(W, 0.7)
            if not mlp:
                continue
            if mlp["kind"] == "dense":
                F = mlp["ff"]
                for n, rows, cols in (("gate", F, W), ("up", F, W), ("down", W, F)):
                    sd[q + n], sd[q + n + ".b"] = lin(rows, cols), rnd(rows, std=0.1)
                continue
            r, F = mlp["router"], mlp["expert"]["ff"]
            n_out = r["experts"] + int(r.get("identity") or 0)
            sd[q + "router"], sd[q + "correction"] = lin(n_out, W), rnd(n_out, std=0.05)
            for e in range(r["experts"]):
                for n, rows, cols in (("gate", F, W), ("up", F, W), ("down", W, F)):
                    sd[f"{q}e{e}.{n}"] = lin(rows, cols)
            if mlp.get("shared"):
                F = mlp["shared"]["ff"]
                for n, rows, cols in (("gate", F, W), ("up", F, W), ("down", W, F), ("sg", 1, W)):
                    sd[f"{q}shared.{n}"] = lin(rows, cols)
        return sd

    def load_state(self, sd: dict[str, torch.Tensor]) -> "KilatarForCausalLM":
        """Build the run-time weights from a checkpoint-named state dict: fused
        projection matrices in the activation dtype; norms, biases, router and
        shared gate, convolution taps, decays and rotary frequencies in fp32."""
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def act(*ts, pad: int = 0, dim: int = 0):  # (fused) projection weight; pad: zero rows up to a multiple of it
            t = torch.cat(ts, dim) if len(ts) > 1 else ts[0]
            if pad and t.shape[0] % pad:
                t = torch.cat([t, t.new_zeros((pad - t.shape[0] % pad, t.shape[1]))], 0)
            return t.to(dev, dt).contiguous()

        def f32(t):
            return t.to(dev, torch.float32).contiguous()

        def freq(rot):
            return rc.rotary_frequencies(int(rot["dims"]), float(rot["base"]), rot.get("scaling")).to(dev) \
                if rot and int(rot.get("dims") or 0) >= 2 else None

        self.layers = []
        for i, L in enumerate(cfg.layers):
            m, p, q, mlp = L["mixer"], f"l{i}.mix.", f"l{i}.mlp.", L.get("mlp")
            out = dict(m=m, type=L["type"], mlp=mlp, norm1=f32(sd[f"l{i}.norm1"]))
            # rows of the fused projection behind the mixer's: gate and up of the dense or shared feed-forward
            ff = q if mlp and mlp["kind"] == "dense" else q + "shared." if mlp and mlp.get("shared") else None
            glu = [sd[ff + "gate"], sd[ff + "up"]] if ff else []
            out["ff"] = int(glu[0].shape[0]) if ff else 0
            down = [sd[ff + "down"]] if ff else []
            if L["type"] == "latent_attention":
                H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
                if sd[p + "dkv"].shape[0] != r + dr or sd[p + "q"].shape[0] != H * (d + dr):
                    raise ValueError(f"{p}: projection rows do not fit kv_rank, rot_dim, heads and dim")
                out.update(w_in=act(sd[p + "q"], sd[p + "dkv"], sd[p + "g"], *glu, pad=IN_PAD), cn=f32(sd[p + "dkv.norm"]),
                           uk=act(sd[p + "uk"]).view(H, d, r),
                           uv=act(sd[p + "uv"]).view(H, dv, r).transpose(1, 2).contiguous(), inv_freq=freq(m.get("rot")),
                           w_out=act(sd[p + "o"], *down, dim=1))
            elif L["type"] == "mamba2":
                inner, C = m["heads"] * m["vdim"], self._conv_channels(m)
                w = sd[p + "in"]
                if w.shape[0] != inner + C + m["heads"] or sd[p + "conv"].shape != (C, int(m["conv"])):
                    raise ValueError(f"{p}: projection rows or convolution taps do not fit the config")
                out.update(w_in=act(w[:inner + C], *glu, w[inner + C:], pad=IN_PAD),  # the narrow step sizes last
                           # tap-major [taps, C]: a run of neighbouring channels shares one load in the kernel
                           conv_w=f32(sd[p + "conv"].t()), conv_b=f32(sd[p + "conv.b"]), dt_bias=f32(sd[p + "dt_bias"]),
                           rate=torch.exp(sd[p + "A_log"].double()).to(dev, torch.float32), skip=f32(sd[p + "D"]),
                           gn=f32(sd[p + "norm"]), w_out=act(sd[p + "o"], *down, dim=1))
            else:
                a, b = p + "left.", p + "right."
                out.update(w_in=act(sd[a + "q"], sd[a + "k"], sd[a + "v"], sd[b + "q"], sd[b + "k"], sd[b + "v"], sd[b + "g"],
                                    *glu, pad=IN_PAD), inv_freq=freq(m["left"].get("rot")),
                           decay=torch.tensor([float(x) for x in m["right"]["decay"]], dtype=torch.float32, device=dev),
                           hn=f32(sd[b + "norm"]), w_lo=act(sd[a + "o"]), w_ro=act(sd[b + "o"]),
                           # half the sum of the two sides: the halves ride in the norms' weights
                           lw=f32(0.5 * sd[a + "out"].float()), rw=f32(0.5 * sd[b + "out"].float()),
                           w_down=act(*down) if down else None)
            if mlp and mlp["kind"] == "dense":
                out.update(gate_b=f32(sd[q + "gate.b"]), up_b=f32(sd[q + "up.b"]), down_b=f32(sd[q + "down.b"]))
            elif mlp:
                E = mlp["router"]["experts"]
                w_egu = torch.stack([torch.cat([sd[f"{q}e{e}.gate"], sd[f"{q}e{e}.up"]], 0)
                                     for e in range(E)]).to(dev, dt).contiguous()
                # where the 256-tile GEMM serves the shape, gate and up rows are interleaved
                # for its SwiGLU epilogue and the [rows, 2 ff] intermediate is never written
                fused = moe.tile_gemm_ok(torch.empty((1, w_egu.shape[2]), device=dev, dtype=dt), w_egu) and \
                    (w_egu.shape[1] // 2) % moe.GLU_BLOCK == 0
                corr = sd.get(q + "correction")
                router = sd[q + "router"]
                if router.shape[0] != E + int(mlp["router"].get("identity") or 0):
                    raise ValueError(f"{q}router: {router.shape[0]} outputs for {E} experts and the identity outputs")
                out.update(n_route=int(router.shape[0]), correction=f32(corr) if corr is not None else None,
                           # the shared expert's gate is one more row of the router's pass over h
                           router=f32(torch.cat([router, sd[q + "shared.sg"]], 0) if ff else router),
                           w_egu=moe.interleave_glu(w_egu) if fused else w_egu, egu_fused=fused,
                           w_edown=torch.stack([sd[f"{q}e{e}.down"] for e in range(E)]).to(dev, dt).contiguous())
            self.layers.append(out)
        self.embed = act(sd["embed"])
        self.embed_w = f32(sd["embed.norm"])
        self.head = act(sd["head"])
        self.final_w = f32(sd["final.norm"])
        return self

    # ------------------------------------------------------------------ mixers
    def _latent(self, L: dict, p: torch.Tensor, o: torch.Tensor, meta: AttnMeta, cache, seq, tables):
        """Gated heads into o; p = [q | dkv | g | ...]."""
        m, T = L["m"], p.shape[0]
        H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        nq = H * (d + dr)
        q = p[:, :nq]  # per head [dim unrotated | rot_dim rotated]
        # fold the key up-projection into the query: the cached latent is the one key/value head of every query head
        qa = torch.bmm(q.unflatten(1, (H, d + dr))[:, :, :d].transpose(0, 1), L["uk"])
        ql = rc.latent_rope(qa, q, d + dr, d, p[:, nq:nq + r + dr], r, dr, L["cn"], self.cfg.rms_norm_eps, L["inv_freq"], 1.0,
                            meta.positions, meta.slot_mapping, cache, interleaved=True)
        tl = (meta.row_tiles, meta.num_prefill_tokens) if meta.is_prefill else (None, 0)
        a = mx.attention(ql, cache, cache, meta.positions, seq, tables, meta.block_size, H, 1, H, r + dr, r, m["scale"],
                         "causal", 0, self._parts(T, H, H, 0, meta, latent=True), False, *tl)
        up = torch.bmm(a.view(T, H, r).transpose(0, 1), L["uv"])  # [H, T, dv]
        g0 = nq + r + dr
        mx.act_mul(p[:, g0:g0 + H * dv], up, "sigmoid", out=o)

    def _mamba2(self, L: dict, p: torch.Tensor, o: torch.Tensor, meta: AttnMeta, tail, state):
        """Gated, normed channels into o; p = [z | x | B | C | gate | up | dt]."""
        m = L["m"]
        Hs, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
        inner, C = Hs * P, self._conv_channels(m)
        t0 = inner + C + 2 * L["ff"]
        xbc = rc.causal_conv(p[:, inner:inner + C], L["conv_w"], tail, meta.positions,
                             meta.row_seq if meta.is_prefill else None, meta.seq_rows, meta.state_slots, bias=L["conv_b"],
                             act="silu")
        y = rc.ssd(xbc[:, :inner], xbc[:, inner:inner + G * N], xbc[:, inner + G * N:], p[:, t0:t0 + Hs], L["dt_bias"],
                   L["rate"], L["skip"], state, meta.positions, meta.seq_rows, meta.state_slots, Hs, G, N, P)
        rc.gate_group_norm(y, p[:, :inner], L["gn"], m["norm_groups"], self.cfg.rms_norm_eps, self.dtype, out=o)

    def _parallel(self, L: dict, p: torch.Tensor, meta: AttnMeta, kc, vc, state, seq, tables) -> dict:
        """The two sides' outputs as the residual step's normed addends; p = [q k v | q k v g | ...]."""
        m, T = L["m"], p.shape[0]
        a, b = m["left"], m["right"]
        H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        Hr, dk, dvr = b["heads"], b["dim"], b["vdim"]
        r0 = H * d + G * (d + dv)
        n, nv = Hr * dk, Hr * dvr
        mx.norm_rope_cache(p, meta.positions, meta.slot_mapping, H, G, d, G * dv, None, None, 0.0, L["inv_freq"], kc, vc,
                           silu=(r0, 2 * n + nv))
        size = int((a.get("mask") or {}).get("size") or 0)
        tl = (meta.row_tiles, meta.num_prefill_tokens) if meta.is_prefill else (None, 0)
        y = mx.attention(p, kc, vc, meta.positions, seq, tables, meta.block_size, H, 1, H // G, d, dv, a["scale"],
                         "chunk" if size else "causal", size, self._parts(T, H, H // G, size, meta), False, *tl)
        o = rc.retention(p[:, r0:r0 + n], p[:, r0 + n:r0 + 2 * n], p[:, r0 + 2 * n:r0 + 2 * n + nv], L["decay"], 1.0, state,
                         meta.positions, meta.seq_rows, meta.state_slots, Hr, dk, dvr)
        g0 = r0 + 2 * n + nv
        o = rc.head_norm_gate(o, 1, L["hn"], p[:, g0:g0 + nv], self.cfg.rms_norm_eps, self.dtype)  # all heads together
        return dict(c=self._mm(y.view(T, H * dv), L["w_lo"]), c_w=L["lw"], d=self._mm(o, L["w_ro"]), d_w=L["rw"])

    # ------------------------------------------------------------------ feed-forward
    def _experts(self, L: dict, h: torch.Tensor, idx, w) -> tuple:
        """The routed experts' outputs in slot order, as the residual step takes them."""
        r = L["mlp"]["router"]
        order, offsets = moe.plan(idx, r["experts"])
        g = moe.grouped_gemm(h, L["w_egu"], order, offsets, r["top"], gather=True, scatter=False, glu=L["egu_fused"])
        act = g if L["egu_fused"] else mx.glu_act(g, "silu")
        y = moe.grouped_gemm(act, L["w_edown"], order, offsets, r["top"], gather=False, scatter=True)
        return y, w, idx if L["n_route"] > r["experts"] else None, r["experts"], h

    def _layer(self, L: dict, h: torch.Tensor, meta: AttnMeta, kc, vc, ci, ri, seq, tables) -> dict:
        """One layer's addends to the residual (arguments of residual_step)."""
        m, mlp, F, T = L["m"], L["mlp"], L["ff"], h.shape[0]
        p = self._mm(h, L["w_in"])
        add: dict = {}
        row_scale = None
        if mlp and mlp["kind"] == "moe":
            r = mlp["router"]
            idx, w, gates = moe.router(h, L["router"], L["n_route"], L["correction"], r["top"], score="softmax",
                                       renorm=True, scale=float(r["scale"]))
            row_scale = gates.view(T) if gates is not None else None
            add["experts"] = self._experts(L, h, idx, w)
        elif mlp:
            add["bias"] = L["down_b"]

        def glu(f0: int, out=None):  # the dense or shared feed-forward up to its down projection
            g, u = p[:, f0:f0 + F], p[:, f0 + F:f0 + 2 * F]
            if mlp["kind"] == "dense":
                return mx.act_mul(g, u, "gelu_tanh", out=out, gate_b=L["gate_b"], up_b=L["up_b"])
            return mx.act_mul(g, u, "silu", out=out, row_scale=row_scale)

        if L["type"] == "parallel":
            a, b = m["left"], m["right"]
            f0 = a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"]) + 2 * b["heads"] * (b["dim"] + b["vdim"])
            add.update(self._parallel(L, p, meta, kc, vc, meta.state[ri], seq, tables))
            if F:
                add["b"] = self._mm(glu(f0), L["w_down"])
            return add
        nv = m["heads"] * m["vdim"]
        o = torch.empty((T, nv + F), dtype=h.dtype, device=h.device)  # [mixer | feed-forward], one output projection
        if L["type"] == "latent_attention":
            f0 = m["heads"] * (m["dim"] + m["rot_dim"]) + m["kv_rank"] + m["rot_dim"] + nv
            self._latent(L, p, o[:, :nv], meta, kc, seq, tables)
        else:
            f0 = nv + self._conv_channels(m)
            self._mamba2(L, p, o[:, :nv], meta, meta.state[ci], meta.state[ri])
        if F:
            glu(f0, o[:, nv:])
        add["a"] = self._mm(o, L["w_out"])
        return add

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, meta: AttnMeta, kv_caches: list[tuple]) -> torch.Tensor:
        """Final-normed hidden rows at meta.logits_idx (or all rows)."""
        cfg = self.cfg
        if meta.state is None or meta.state_slots is None:
            raise ValueError("Kilatar needs the step's state slots (a runner with state support)")
        rs = dict(eps=cfg.rms_norm_eps, out_dtype=self.dtype)
        X0 = mx.embed_streams(input_ids, self.embed, 1, norm_w=self.embed_w, eps=cfg.rms_norm_eps)
        X0 = X0.view(X0.shape[0], X0.shape[2])
        X = X0.clone() if self.reentry else X0
        if meta.is_prefill:  # rows of several sequences: per-row sequence ids + one table
            seq, tables = meta.row_seq, meta.row_tables
        else:  # decode: row i is sequence i
            seq, tables = None, meta.block_tables
        pend: dict = {}
        for run, li in enumerate(self.runs):
            L = self.layers[li]
            if run in self.reentry:
                pend["e"] = X0  # a further pass: the embedding output joins once more
            h, _ = mx.residual_step(X, norm="rms", norm_w=L["norm1"], **pend, **rs)
            pend = self._layer(L, h, meta, *kv_caches[run], *self._state_index[run], seq, tables)
            if self.layer_hook is not None and meta.is_prefill:
                self.layer_hook(run)
            if self.trace_layers is not None:
                mx.residual_step(X, **pend, **rs)
                pend = {}
                self.trace_layers.append(X.clone())
        pick = meta.logits_idx
        if pick is not None and pick.numel() == 0:
            return torch.empty((0, cfg.hidden_size), device=X.device, dtype=self.dtype)
        # the last layer's addends and the final norm, on the chosen rows only
        return mx.residual_step(X, norm="rms", norm_w=self.final_w, rows=pick, **pend, **rs)[0]
