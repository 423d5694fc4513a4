"""What the layer-listed model classes with recurrent state share: the engine's
hooks, decode-size GEMM selection, weight and state accounting, checkpoint
reading, the vocabulary projection.  A class adds its layers: load_state,
random_state, cache_widths, state_shapes, forward."""
from __future__ import annotations

import glob
import math
import os

import torch

from .config import LayeredConfig
from .gemm_tuning import planned_mm, tune_small_m
from .llama import AttnMeta, TPGroup

#: fused in-projections that end in a narrow section (a step size or a gate per head) are padded with zero
#: rows to a multiple of this, the GEMM kernels' column tile
IN_PAD = 64


class StatefulLayeredModel:
    #: the runner builds per-row sequence ids and one block table over all rows of a step
    unified_rows = True
    #: the runner allocates per-sequence state (alloc_state) and names every sequence's slot
    state_slots = True
    #: dense projections of a layer, by the name of their weight
    LINEARS: tuple[str, ...] = ()

    def __init__(self, cfg: LayeredConfig, device: torch.device | str = "cuda", dtype=torch.bfloat16,
                 tp: TPGroup | None = None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp = tp or TPGroup()
        if self.tp.size != 1:
            raise ValueError(f"{cfg.architecture} runs on one GPU per engine (tensor parallel size 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {dtype}")
        self.layers: list[dict] = []
        self.embed = self.head = self.final_w = None
        self.fp8 = False
        self.kv_scales = (1.0, 1.0)
        self.kv_amax = None
        self.layer_hook = None
        self.gemm_plan: dict = {}
        self.gemm_tuned: set = set()
        # debugging: when a list, forward() appends the residual after every layer
        self.trace_layers: list | None = None

    # ------------------------------------------------------------------ engine hooks (no-ops here)
    def enable_fused_mlp(self) -> bool:
        return False

    def fold_norms(self) -> bool:
        return False

    def tune_prefill_gemms(self, max_tokens, **kw) -> list:
        return []

    def quantize_fp8(self):
        raise ValueError(f"fp8 linears are not available for {self.cfg.architecture}")

    # ------------------------------------------------------------------ GEMMs
    def _own_layers(self) -> list[dict]:
        """Every set of layer weights once, however many layers run it."""
        return list({id(L): L for L in self.layers}.values())

    def tune_gemms(self, sizes, **kw) -> list:
        """Decode batch sizes: the hand-written small-M GEMMs where they beat the
        library (bf16 on the GPU; models/gemm_tuning.py)."""
        if self.device.type != "cuda" or self.dtype != torch.bfloat16 or not self.layers:
            return []
        groups: dict = {}  # layers of different mixers have projections of different shapes
        for n in self.LINEARS:
            for L in self._own_layers():
                if L.get(n) is not None:
                    groups.setdefault((n, tuple(L[n].shape)), []).append(L[n])
        return tune_small_m(list(groups.values()), sizes, self.gemm_plan, self.gemm_tuned, **kw)

    def _mm(self, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        return planned_mm(self.gemm_plan, x, w)

    @torch.no_grad()
    def warmup_linears(self, tokens: int) -> None:
        seen = set()
        for L in self._own_layers():
            for name in self.LINEARS:
                w = L.get(name)
                if w is None or tuple(w.shape) in seen:
                    continue
                seen.add(tuple(w.shape))
                torch.matmul(torch.zeros(tokens, w.shape[1], device=self.device, dtype=self.dtype), w.t())

    def weight_bytes(self) -> int:
        ts = [t for L in self._own_layers() for t in L.values() if isinstance(t, torch.Tensor)]
        ts += [t for t in (self.embed, self.head) if t is not None]
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------------------------ paged caches and state slots
    def cache_widths(self) -> list[tuple[int, int] | None]:
        """(K row width, V row width) of every layer run's paged cache; V width
        0: the K rows are the values too; None: no cache."""
        raise NotImplementedError

    def state_shapes(self) -> list[tuple[tuple, torch.dtype]]:
        """Shape (without the slot dimension) and dtype of every per-sequence state tensor."""
        raise NotImplementedError

    def kv_bytes_per_block(self, block_size: int, dtype: torch.dtype) -> int:
        es = torch.empty((), dtype=dtype).element_size()
        return sum((w[0] + w[1]) * block_size * es for w in self.cache_widths() if w)

    def alloc_kv_caches(self, num_blocks: int, block_size: int, dtype: torch.dtype) -> list[tuple]:
        """One (K, V) pair per layer run, token-major [num_blocks * block_size,
        width], indexed by the engine's one block table; the pair is the same
        tensor twice where the keys' rows are the values too, and empty where a
        layer caches nothing."""
        if dtype != self.dtype:
            raise ValueError(f"the cache holds the model's activation dtype {self.dtype}, not {dtype}")
        out: list[tuple] = []
        for w in self.cache_widths():
            n = num_blocks * block_size if w else 0
            k = torch.zeros((n, w[0] if w else 0), dtype=dtype, device=self.device)
            out.append((k, torch.zeros((n, w[1]), dtype=dtype, device=self.device) if w and w[1] else k))
        return out

    def state_bytes_per_slot(self) -> int:
        return sum(math.prod(s) * torch.empty((), dtype=dt).element_size() for s, dt in self.state_shapes())

    def alloc_state(self, num_slots: int) -> list[torch.Tensor]:
        return [torch.zeros((num_slots, *s), dtype=dt, device=self.device) for s, dt in self.state_shapes()]

    # ------------------------------------------------------------------ weights
    def random_state(self, seed: int = 0) -> dict[str, torch.Tensor]:
        raise NotImplementedError

    def load_state(self, sd: dict[str, torch.Tensor]) -> "StatefulLayeredModel":
        raise NotImplementedError

    def random_init(self, seed: int = 0) -> "StatefulLayeredModel":
        return self.load_state(self.random_state(seed))

    def load_safetensors(self, path: str) -> "StatefulLayeredModel":
        from safetensors import safe_open

        files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
        if not files:
            raise FileNotFoundError(f"no safetensors in {path}")
        tensors = {}
        for f in files:
            with safe_open(f, framework="pt", device="cpu") as sf:
                for k in sf.keys():
                    tensors[k] = sf.get_tensor(k)
        return self.load_state(tensors)

    # ------------------------------------------------------------------ forward
    def _parts(self, rows: int, n_qh: int, group: int, visible: int, meta: AttnMeta, latent: bool = False) -> int:
        """Key partitions of the step's decode rows (rows that are no prompt-chunk
        tiles): n_qh query heads, `group` per key/value head; visible: the most
        keys a row sees (0: its whole context); latent: one shared row that is key
        and value (a workgroup per 32 heads instead of a wave)."""
        from ..ops import mixers as mx

        vis = meta.max_ctx if meta.max_ctx else self.cfg.max_position_embeddings
        if visible:
            vis = min(vis, visible)
        grouped = self.dtype == torch.bfloat16 and self.device.type == "cuda"
        if meta.is_prefill and grouped:
            rows -= meta.num_prefill_tokens
        units = n_qh if not grouped else max(1, n_qh // group) * (-(-group // 32))
        target = mx.ROW_TARGET_WAVES if not grouped else mx.LATENT_TARGET_GROUPS if latent else mx.GROUP_TARGET_WAVES
        return mx.row_attention_parts(max(rows, 1), units, vis, target)

    def compute_logits(self, hidden: torch.Tensor, fp32: bool = False) -> torch.Tensor:
        """Logits of final-normed rows; fp32: the products of the bf16 operands
        accumulated and returned in fp32 (scoring), in vocabulary slices so no
        fp32 copy of the head persists."""
        if not fp32 or hidden.dtype == torch.float32:
            return torch.matmul(hidden, self.head.t())
        hf = hidden.float()
        V = self.head.shape[0]
        out = torch.empty((hidden.shape[0], V), dtype=torch.float32, device=hidden.device)
        for v0 in range(0, V, 16384):
            torch.matmul(hf, self.head[v0:v0 + 16384].float().t(), out=out[:, v0:v0 + 16384])
        return out

    def sample_sharded(self, *a, **kw):
        raise RuntimeError(f"vocab-sharded sampling needs tensor parallelism, which {self.cfg.architecture} does not use")
