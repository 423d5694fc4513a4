"""Povurax: a layer-listed hybrid decoder for the MI355X engine: layers in which
softmax attention and a state-space (Mamba-2) mixer read the same input side by
side, and gated linear attention layers, with norms on the sublayers' outputs
only and layers that share another layer's weights.

A checkpoint lists its layers; an entry with `weights_of` runs another layer's
weights with a cache and state of its own.  Sublayers read the residual as it
is, and what they return is normed into it: x <- x + rms(sub(x)) * w.  Per
layer, T rows of one engine step (prompt chunks and decode tokens of different
sequences; state per sequence in the slot the engine assigned), h the residual
in the activation dtype:

  parallel
    p  = h @ [Wq | Wk | Wv | Wg | Win]^T                hipBLASLt, one fused projection for both halves
         norm_rope_cache(p_q, p_k, p_v)                 HIP  one RMS norm over all heads of q (of k), rotary
                                                             (interleaved pairs), K / V into the paged caches
    a  = attention(q, K, V)                             HIP  tile kernel (prompt chunks) / grouped decode / row kernel
    c  = causal_conv(p_x|B|C, bias, silu)               HIP  short causal convolution over time, tail state per slot
    s  = ssd(c_x, c_B, c_C, p_dt; S)                    HIP  S <- exp(-rate u) S + u B x^T, y = S^T C + D x, fp32
    o  = [left_scale a sigmoid(p_g) |                   HIP  act_mul, gate_group_norm: both write their part of
          right_scale groupnorm(s silu(p_z)) w]              the one row that the output projection reads
    y  = o @ [Wo_left | Wo_right]^T                     hipBLASLt: both output projections and their sum in one GEMM
  gla
    p  = h @ [Wq | Wk | Wv | Wg | Wa1]^T;  z = p_a1 @ Wa2^T
    o  = gated_linear_attention(q, k, v, z; S)          HIP  S <- diag(sigmoid(z + b)^(1/tau)) S + k v^T, fp32
    y  = head_norm_gate(o, w, silu(p_g)) @ Wo^T         HIP + hipBLASLt
  both
    X += rms(y) w1; h = cast(X)                         HIP  residual_step
    X += rms(ff(h)) w2; h' = cast(X)                    hipBLASLt + HIP glu_act (clamped unit) + residual_step

Norms, the residual, scores and weights, decays, step sizes and the recurrent
states are fp32; projections, the convolution and activations are bf16
(dtype=bfloat16) or everything is fp32 (dtype=float32).
"""
from __future__ import annotations

import torch

from ..ops import mixers as mx
from ..ops import recurrent as rc
from .config import LayeredConfig
from .layered import IN_PAD, StatefulLayeredModel
from .llama import AttnMeta, TPGroup

MIXERS = ("parallel", "gla")
FF_ALPHA = 1.702  # the feed-forward's gate is g * sigmoid(FF_ALPHA * g)


class PovuraxForCausalLM(StatefulLayeredModel):
    LINEARS = ("w_in", "w_a2", "w_o", "w_gu", "w_down")

    def __init__(self, cfg: LayeredConfig, device: torch.device | str = "cuda", dtype=torch.bfloat16,
                 tp: TPGroup | None = None):
        super().__init__(cfg, device, dtype, tp)
        if cfg.loop or cfg.streams:
            raise ValueError("Povurax has neither a layer loop nor parallel residual streams")
        self.src = cfg.weight_layers()  # the layer whose tensors each layer runs
        for i, L in enumerate(cfg.layers):
            m, S = L["mixer"], cfg.layers[self.src[i]]
            if L["type"] not in MIXERS:
                raise ValueError(f"unknown mixer type {L['type']!r}")
            if L.get("mlp") and L["mlp"].get("kind") != "dense":
                raise ValueError(f"unknown feed-forward kind {L['mlp'].get('kind')!r}")
            if (S["type"], S["mixer"], S.get("mlp")) != (L["type"], m, L.get("mlp")):
                raise ValueError(f"layer {i} differs from layer {self.src[i]}, whose weights it uses")
            if L["type"] != "parallel":
                continue
            a, b = m["left"], m["right"]
            if a["heads"] % a["kv_heads"]:
                raise ValueError(f"layer {i}: {a['heads']} heads over {a['kv_heads']} key/value heads")
            if int((a.get("rot") or {}).get("dims", 0)) > a["dim"]:
                raise ValueError(f"layer {i}: {a['rot']['dims']} rotated dimensions in a head of {a['dim']}")
            if b["heads"] % b["groups"] or (b["heads"] * b["vdim"]) % b["norm_groups"]:
                raise ValueError(f"layer {i}: state-space heads or channels do not divide into their groups")
        # per layer, the index of its convolution tail and of its running matrices in the state list
        self._state_index: list[tuple[int | None, int]] = []
        self.state_shapes()

    # ------------------------------------------------------------------ paged caches and state slots
    def cache_widths(self) -> list[tuple[int, int] | None]:
        """(K row width, V row width) of every layer with attention, whoever's weights it runs."""
        out = []
        for L in self.cfg.layers:
            a = L["mixer"].get("left") if L["type"] == "parallel" else None
            out.append((a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]) if a else None)
        return out

    @staticmethod
    def _conv_channels(b: dict) -> int:
        return b["heads"] * b["vdim"] + 2 * b["groups"] * b["state"]

    def state_shapes(self) -> list[tuple[tuple, torch.dtype]]:
        """Shape (without the slot dimension) and dtype of every per-sequence
        state tensor: a layer's running matrices (fp32, column by column), and in
        front of them a parallel layer's last taps - 1 projected rows before the
        short convolution."""
        out, index = [], []
        for L in self.cfg.layers:
            m = L["mixer"]
            if L["type"] == "parallel":
                b = m["right"]
                index.append((len(out), len(out) + 1))
                out.append(((int(b["conv"]) - 1, self._conv_channels(b)), self.dtype))
                out.append(((b["heads"], b["vdim"], b["state"]), torch.float32))
            else:
                index.append((None, len(out)))
                out.append(((m["heads"], m["vdim"], m["dim"]), torch.float32))
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

        def uni(n, lo, hi):
            return (lo + (hi - lo) * torch.rand(n, generator=g)).to(torch.bfloat16)

        sd = {"embed": rnd(cfg.vocab_size, W, std=1.0 / max(cfg.embedding_scale, 1e-6)), "final.norm": 1 + rnd(W, std=0.1),
              "head": rnd(cfg.vocab_size, W, std=W ** -0.5)}
        for i, L in enumerate(cfg.layers):
            if self.src[i] != i:
                continue
            m, p, q = L["mixer"], f"l{i}.mix.", f"l{i}."
            sd[q + "norm1"] = 0.5 + rnd(W, std=0.1)
            if L["type"] == "parallel":
                a, b, l, r = m["left"], m["right"], p + "left.", p + "right."
                H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
                for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv), ("g", H * dv)):
                    sd[l + n] = rnd(rows, W, std=W ** -0.5)
                sd[l + "q.norm"], sd[l + "k.norm"] = 1 + rnd(H * d, std=0.1), 1 + rnd(G * d, std=0.1)
                sd[l + "o"] = rnd(W, H * dv, std=(H * dv) ** -0.5)
                Hs, inner, C, taps = b["heads"], b["heads"] * b["vdim"], self._conv_channels(b), int(b["conv"])
                sd[r + "in"] = rnd(inner + C + Hs, W, std=W ** -0.5)
                sd[r + "conv"], sd[r + "conv.b"] = rnd(C, taps, std=taps ** -0.5), rnd(C, std=0.1)
                sd[r + "dt_bias"] = uni(Hs, -4.0, -1.0)
                sd[r + "A_log"], sd[r + "D"] = uni(Hs, 0.0, 2.5), 1 + rnd(Hs, std=0.2)
                sd[r + "norm"] = 1 + rnd(inner, std=0.1)
                sd[r + "o"] = rnd(W, inner, std=inner ** -0.5)
            else:
                H, d, dv = m["heads"], m["dim"], m["vdim"]
                lo = int(m.get("decay_rank") or min(16, W))
                for n, rows in (("q", H * d), ("k", H * d), ("v", H * dv), ("g", H * dv)):
                    sd[p + n] = rnd(rows, W, std=W ** -0.5)
                sd[p + "o"] = rnd(W, H * dv, std=(H * dv) ** -0.5)
                sd[p + "norm"] = 1 + rnd(dv, std=0.1)
                sd[p + "a1"], sd[p + "a2"] = rnd(lo, W, std=W ** -0.5), rnd(H * d, lo, std=lo ** -0.5)
                sd[p + "a2.b"] = rnd(H * d, std=1.0) + 1.0
            if L.get("mlp"):
                F = L["mlp"]["ff"]
                sd[q + "norm2"] = 0.5 + rnd(W, std=0.1)
                sd[q + "mlp.gate"], sd[q + "mlp.up"] = rnd(F, W, std=W ** -0.5), rnd(F, W, std=W ** -0.5)
                sd[q + "mlp.down"] = rnd(W, F, std=F ** -0.5)
        return sd

    def load_state(self, sd: dict[str, torch.Tensor]) -> "PovuraxForCausalLM":
        """Build the run-time weights from a checkpoint-named state dict: fused
        projection matrices in the activation dtype; norms, biases, convolution
        taps, state-space rates and rotary frequencies in fp32.  A layer that runs
        another layer's weights holds the same dict."""
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def act(*names, pad: int = 0, dim: int = 0):  # (fused) projection weight; pad: zero rows up to a multiple of it
            t = torch.cat([sd[n] for n in names], dim) if len(names) > 1 else sd[names[0]]
            if pad and t.shape[0] % pad:
                t = torch.cat([t, t.new_zeros((pad - t.shape[0] % pad, t.shape[1]))], 0)
            return t.to(dev, dt).contiguous()

        def f32(t):
            return t.to(dev, torch.float32).contiguous()

        def parallel(m: dict, p: str) -> dict:
            a, b, l, r = m["left"], m["right"], p + "left.", p + "right."
            rows = b["heads"] * b["vdim"] + self._conv_channels(b) + b["heads"]
            if sd[r + "in"].shape[0] != rows or sd[r + "conv"].shape != (self._conv_channels(b), int(b["conv"])):
                raise ValueError(f"{r}: projection rows or convolution taps do not fit the config")
            rot = a.get("rot")
            return dict(
                w_in=act(l + "q", l + "k", l + "v", l + "g", r + "in", pad=IN_PAD),
                qn=f32(sd[l + "q.norm"]), kn=f32(sd[l + "k.norm"]),
                inv_freq=rc.rotary_frequencies(int(rot["dims"]), float(rot["base"])).to(dev)
                if rot and int(rot.get("dims") or 0) >= 2 else None,
                # tap-major [taps, C]: a run of neighbouring channels shares one load in the kernel
                conv_w=f32(sd[r + "conv"].t()), conv_b=f32(sd[r + "conv.b"]), dt_bias=f32(sd[r + "dt_bias"]),
                rate=torch.exp(sd[r + "A_log"].double()).to(dev, torch.float32), skip=f32(sd[r + "D"]),
                # the halves' scales enter where their rows are formed in fp32, in front of the common output projection
                gn=f32(sd[r + "norm"].float() * float(m["right_scale"])), left_scale=float(m["left_scale"]),
                w_o=act(l + "o", r + "o", dim=1))

        def gla(m: dict, p: str) -> dict:
            return dict(w_in=act(p + "q", p + "k", p + "v", p + "g", p + "a1", pad=IN_PAD), w_a2=act(p + "a2"),
                        lora=int(sd[p + "a1"].shape[0]), a_b=f32(sd[p + "a2.b"]),
                        hnorm=f32(sd[p + "norm"].float().repeat(m["heads"])), w_o=act(p + "o"))

        own = {}
        for i, L in enumerate(cfg.layers):
            if self.src[i] != i:
                continue
            p, q, mlp = f"l{i}.mix.", f"l{i}.", L.get("mlp")
            out = dict(m=L["mixer"], type=L["type"], mlp=mlp, norm1=f32(sd[q + "norm1"]))
            out.update(parallel(L["mixer"], p) if L["type"] == "parallel" else gla(L["mixer"], p))
            if mlp:
                out.update(norm2=f32(sd[q + "norm2"]), w_gu=act(q + "mlp.gate", q + "mlp.up"), w_down=act(q + "mlp.down"))
            own[i] = out
        self.layers = [own[j] for j in self.src]
        self.embed = act("embed")
        self.head = act("head")
        self.final_w = f32(sd["final.norm"])
        return self

    # ------------------------------------------------------------------ forward
    def _parallel(self, L: dict, h: torch.Tensor, meta: AttnMeta, kc, vc, tail, state, seq, tables, bs: int):
        m, T, eps = L["m"], h.shape[0], self.cfg.rms_norm_eps
        a, b = m["left"], m["right"]
        H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        Hs, P, N, Gs = b["heads"], b["vdim"], b["state"], b["groups"]
        nv, inner, C = H * dv, Hs * P, self._conv_channels(b)
        g0 = H * d + G * (d + dv)
        z0 = g0 + nv
        c0 = z0 + inner
        p = self._mm(h, L["w_in"])  # [q | k | v | g || z | x | B | C | dt]
        o = torch.empty((T, nv + inner), dtype=h.dtype, device=h.device)
        # left: attention
        mx.norm_rope_cache(p, meta.positions, meta.slot_mapping, H, G, d, G * dv, L["qn"], L["kn"], eps, L["inv_freq"],
                           kc, vc)
        tl = (meta.row_tiles, meta.num_prefill_tokens) if meta.is_prefill else (None, 0)
        y = mx.attention(p, kc, vc, meta.positions, seq, tables, bs, H, 1, H // G, d, dv, a["scale"], "causal", 0,
                         self._parts(T, H, H // G, 0, meta), False, *tl, fine_weights=True)
        mx.act_mul(p[:, g0:z0], y.view(T, nv), "sigmoid", out=o[:, :nv], scale=L["left_scale"])
        # right: state-space mixer
        xbc = rc.causal_conv(p[:, c0:c0 + C], L["conv_w"], tail, meta.positions, meta.row_seq if meta.is_prefill else None,
                             meta.seq_rows, meta.state_slots, bias=L["conv_b"], act="silu")
        y = rc.ssd(xbc[:, :inner], xbc[:, inner:inner + Gs * N], xbc[:, inner + Gs * N:], p[:, c0 + C:c0 + C + Hs],
                   L["dt_bias"], L["rate"], L["skip"], state, meta.positions, meta.seq_rows, meta.state_slots, Hs, Gs, N, P)
        rc.gate_group_norm(y, p[:, z0:c0], L["gn"], b["norm_groups"], eps, self.dtype, out=o[:, nv:])
        return self._mm(o, L["w_o"])

    def _gla(self, L: dict, h: torch.Tensor, meta: AttnMeta, state: torch.Tensor):
        m = L["m"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        n, nv = H * d, H * dv
        p = self._mm(h, L["w_in"])  # [q | k | v | g | a1]
        g0 = 2 * n + nv
        z = self._mm(p[:, g0 + nv:g0 + nv + L["lora"]], L["w_a2"])
        o = rc.gated_linear_attention(p[:, :n], p[:, n:2 * n], p[:, 2 * n:g0], z, L["a_b"], float(m["tau"]), d ** -0.5, state,
                                      meta.positions, meta.seq_rows, meta.state_slots, H, d, dv)
        o = rc.head_norm_gate(o, H, L["hnorm"], p[:, g0:g0 + nv], self.cfg.rms_norm_eps, self.dtype, gate_act="silu")
        return self._mm(o, L["w_o"])

    def forward(self, input_ids: torch.Tensor, meta: AttnMeta, kv_caches: list[tuple]) -> torch.Tensor:
        """Final-normed hidden rows at meta.logits_idx (or all rows)."""
        cfg, dt = self.cfg, self.dtype
        if meta.state is None or meta.state_slots is None:
            raise ValueError("Povurax needs the step's state slots (a runner with state support)")
        X = mx.embed_streams(input_ids, self.embed, 1, scale=cfg.embedding_scale)
        X = X.view(X.shape[0], X.shape[2])
        if meta.is_prefill:  # rows of several sequences: per-row sequence ids + one table
            seq, tables = meta.row_seq, meta.row_tables
        else:  # decode: row i is sequence i
            seq, tables = None, meta.block_tables
        rs = dict(eps=cfg.rms_norm_eps, out_dtype=dt)
        cast = dt != torch.float32  # in float32 the sublayers read the residual itself

        def join(y=None, w=None):  # X += rms(y) w; the residual as the next sublayer reads it
            if y is None and not cast:
                return X
            h = mx.residual_step(X, c=y, c_w=w, want_cast=cast, **rs)[1]
            return X if h is None else h

        h = join()
        last, pend = len(self.layers) - 1, {}
        for i, L in enumerate(self.layers):
            ci, ri = self._state_index[i]
            kc, vc = kv_caches[i]
            if L["type"] == "parallel":
                y = self._parallel(L, h, meta, kc, vc, meta.state[ci], meta.state[ri], seq, tables, meta.block_size)
            else:
                y = self._gla(L, h, meta, meta.state[ri])
            if self.layer_hook is not None and meta.is_prefill:
                self.layer_hook(i)
            w = L["norm1"]
            if L["mlp"]:
                h = join(y, w)
                gu = self._mm(h, L["w_gu"])
                y = self._mm(mx.glu_act(gu, "swiglu_clamp", float(L["mlp"]["limit"]), FF_ALPHA), L["w_down"])
                w = L["norm2"]
            if i < last or self.trace_layers is not None:
                h = join(y, w)
                if self.trace_layers is not None:
                    self.trace_layers.append(X.clone())
            else:
                pend = dict(c=y, c_w=w)  # the last addend joins the residual on the chosen rows, with the final norm
        pick = meta.logits_idx
        if pick is not None:
            if pick.numel() == 0:
                return torch.empty((0, cfg.hidden_size), device=X.device, dtype=dt)
            X = X.index_select(0, pick)
            if pend:
                pend["c"] = pend["c"].index_select(0, pick)
        return mx.residual_step(X, norm="rms", norm_w=self.final_w, **pend, **rs)[0]
