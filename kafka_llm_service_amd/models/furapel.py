"""Furapel: a decoder of parallel layers with element-wise tanh norms, a run of layers that is looped over with shared
weights, and softmax attention, windowed latent attention and matrix-memory mixers beside routed squared-relu experts.

Layer (two norms of the same residual, one add):

    x <- x + mixer(norm1(x)) + experts(norm2(x))        norm(x) = tanh(alpha x) * w + b    (element-wise, alpha a scalar)

Loop. Layers ``loop.start`` .. ``loop.stop`` - 1 run ``loop.times`` times in a row with the same tensors. In front of
every pass x <- W_in [x | x0], x0 being the (scaled) embedding rows. Every pass has a cache and a state of its own.

Mixers
  attention         grouped-query softmax attention; rotation of dimension i with i + rot.dims / 2 on the first rot.dims
                    dimensions of every q and k head (frequencies blended by rot.scaling); every head's output times
                    sigmoid of one number, W_g h, before W_o.
  latent_attention  one RMS-normed latent row c (kv_rank) per token is cached; keys and values per head are W_uk c and
                    W_uv c, no positions, a sliding window (row i sees keys j with 0 <= i - j < mask.size). The engine
                    attends in the latent space (q_lat = W_uk^T q per head, scores q_lat . c, output W_uv (sum p c)).
  mlstm             per head a matrix memory S (dim x vdim), a normaliser n and a running maximum m that starts at 0,
                    with capped exponential input and sigmoid forget gates; the read-out S^T q / (max(|n . q|, e^-m) +
                    1e-6) is unit-RMS-normed per head, weighted, gated by sigmoid(W_g h) and projected.
Experts           router logits in fp32, softmax over all of them, the ``top`` largest chosen and weighted by their
                  scores as they are; expert = W_down relu(W_up h)^2.

How the engine runs it. A layer's projections of norm1(x) are one GEMM. The add to the residual, both norms of the next
layer and, in front of a pass, the residual's copy into the loop product's input are one element-wise kernel, which also
sums a split-K projection's slabs and, in long steps, gathers every token's expert rows. The head gates are applied by the
attention kernels as they write their output. The squared relu is part of the expert products. Long portions run the
matrix memory in chunks of matrix products.

Per sequence the engine keeps, for every layer RUN (a looped layer counts once per pass), pages (keys and page-wise
transposed values, or latent rows; page ids shared by all runs) or a slot of matrix-memory state (S, n, m). The residual,
norms, rotation, scores, softmax, router, gates of the recurrence and states are fp32, as is the loop product's result;
projections run in the model dtype (bf16, or fp32 throughout).

Steps are planned as segments (``SegMeta``, models/budurax.py): one run of consecutive rows per sequence, a decoded
token being a run of one, so prompt portions and single tokens go through the same layers.
"""
from __future__ import annotations

import json
import math
from dataclasses import dataclass, field
from pathlib import Path

import torch
import torch.nn.functional as F

from kafka_llm_service_amd import ops
from kafka_llm_service_amd.models.budurax import SegMeta, rotary_table
from kafka_llm_service_amd.ops import hybrid as hops

PAGE = 16


@dataclass
class FurapelConfig:
    name: str = "furapel"
    arch: str = "furapel"
    vocab_size: int = 0
    hidden_size: int = 0
    layers: list = field(default_factory=list)   # config.json's entries: {"type", "mixer": {...}, "mlp": {...}|None}
    norm_eps: float = 1e-6                       # of the latent and per-head RMS norms (the tanh norms have none)
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    loop: dict | None = None                     # {"start", "stop", "times"}; None = every layer once
    max_position_embeddings: int = 1 << 20
    bos_token_id: int = 0
    eos_token_ids: list = field(default_factory=list)
    tie_word_embeddings: bool = False
    num_experts: int = 0

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_dict(c: dict, name: str = "furapel") -> "FurapelConfig":
        lp = c.get("loop") or None
        return FurapelConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]),
                             layers=list(c["layers"]), norm_eps=float(c["norm"]["eps"]),
                             embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                             logit_scale=float(c.get("logit_scale", 1.0)),
                             loop={k: int(lp[k]) for k in ("start", "stop", "times")} if lp else None)

    @staticmethod
    def from_json(path: str | Path) -> "FurapelConfig":
        path = Path(path)
        return FurapelConfig.from_dict(json.loads(path.read_text()), name=path.parent.name)

    def to_dict(self) -> dict:
        d = {"architecture": "Furapel", "vocab": self.vocab_size, "width": self.hidden_size, "layers": self.layers,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embed_scale}, "logit_scale": self.logit_scale}
        if self.loop:
            d["loop"] = dict(self.loop)
        return d

    def runs(self) -> list[tuple[int, bool]]:
        """The layer runs in order: (layer, whether a pass of the loop starts right before it)."""
        n, lp = len(self.layers), self.loop
        if not lp:
            return [(i, False) for i in range(n)]
        a, b, k = lp["start"], lp["stop"], lp["times"]
        if not (0 <= a < b <= n and k >= 1):
            raise ValueError(f"loop over layers {a} .. {b - 1} of {n}, {k} times")
        return [(i, False) for i in range(a)] + [(i, i == a) for _ in range(k) for i in range(a, b)] + \
            [(i, False) for i in range(b, n)]

    def num_params(self) -> int:
        return sum(math.prod(s) for s in tensor_shapes(self).values())


def _moe_sizes(mlp: dict) -> tuple[int, int, int]:
    if mlp.get("kind", "moe") != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")
    return int(mlp["router"]["experts"]), int(mlp["router"]["top"]), int(mlp["expert"]["ff"])


def tensor_shapes(cfg: FurapelConfig) -> dict[str, tuple]:
    """Checkpoint tensor names -> shapes of a model with this config."""
    d, V = cfg.hidden_size, cfg.vocab_size
    s: dict[str, tuple] = {"embed": (V, d)}

    def norm(name):
        s[name], s[name + ".b"], s[name + ".alpha"] = (d,), (d,), ()

    if cfg.loop:
        s["loop.in"] = (d, 2 * d)
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.", L["mixer"]
        q = p + "mix."
        norm(p + "norm1")
        if L["type"] == "attention":
            H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
            s[q + "q"], s[q + "k"], s[q + "v"], s[q + "g"] = (H * D, d), (G * D, d), (G * Dv, d), (H, d)
            s[q + "o"] = (d, H * Dv)
        elif L["type"] == "latent_attention":
            H, D, Dv, R = (int(m[k]) for k in ("heads", "dim", "vdim", "kv_rank"))
            s[q + "q"], s[q + "dkv"], s[q + "dkv.norm"] = (H * D, d), (R, d), (R,)
            s[q + "uk"], s[q + "uv"], s[q + "o"] = (H * D, R), (H * Dv, R), (d, H * Dv)
        elif L["type"] == "mlstm":
            H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
            s[q + "q"], s[q + "k"] = (H * D, d), (H * D, d)
            s[q + "v"], s[q + "g"] = (H * Dv, d), (H * Dv, d)
            s[q + "o"], s[q + "norm"] = (d, H * Dv), (H * Dv,)
            for n in ("i", "f"):
                s[q + n], s[q + n + ".b"] = (H, d), (H,)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
        if L.get("mlp"):
            E, _, ff = _moe_sizes(L["mlp"])
            norm(p + "norm2")
            for e in range(E):
                s[f"{p}mlp.e{e}.up"], s[f"{p}mlp.e{e}.down"] = (ff, d), (d, ff)
            s[p + "mlp.router"] = (E, d)
    norm("final.norm")
    s["head"] = (V, d)
    return s


def random_tensors(cfg: FurapelConfig, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
    """Seeded bf16 weights with the value ranges each kind of tensor needs (norm weights around one, a loop product that
    keeps the residual's size, forget gates that mostly keep), drawn on ``device``."""
    g = torch.Generator(device=device).manual_seed(seed)

    def rn(shape):
        return torch.randn(shape, generator=g, device=device)

    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.1 * rn(shape)
        elif leaf == "alpha":
            t = 0.7 + 0.1 * rn(shape)
        elif name.endswith("f.b"):
            t = 2.0 + 3.0 * torch.rand(shape, generator=g, device=device)
        elif leaf == "b":
            t = 0.1 * rn(shape)
        elif leaf == "embed":
            t = rn(shape) / max(cfg.embed_scale, 1e-6)
        elif leaf == "router":
            t = rn(shape) * 2.0 / math.sqrt(shape[-1])
        else:
            t = rn(shape) / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out


class LayerState:
    """Per layer run a dict of state tensors, one row per state slot: ``S``, ``n``, ``m`` of an mlstm run (fp32), empty
    for the others."""

    def __init__(self):
        self.layers: list[dict] = []

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for st in self.layers for t in st.values())


class _Layer:
    pass


class FurapelLM:
    plan = "segments"  # the model runner plans its steps as SegMeta runs (engine/model_runner.py)

    def __init__(self, cfg: FurapelConfig, device, dtype=torch.bfloat16, tp: int = 1, tp_rank: int = 0,
                 max_positions: int | None = None):
        if tp != 1:
            raise ValueError("Furapel runs unsharded (tp = 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Furapel runs in bfloat16 or float32")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp, self.tp_rank, self.ep, self.ep_rank = 1, 0, 1, 0
        self.dp_attention = False
        self.stream = self.tiled_only = False
        self.stream_max_m = 0
        self.max_positions = int(max_positions or 8192)
        self.layers: list[_Layer] = []
        self.runs: list[tuple[int, bool]] = []
        self.attn_tile_tokens: list[int] = []
        self._rot: dict = {}

    # engine hooks shared with the other model classes ---------------------------------------------------------------
    STREAMED = ("w_in", "o")

    def _streamable(self, w) -> bool:
        return w is not None and w.dtype == torch.bfloat16 and w.is_cuda and \
            ops.stream_plan(1, w.shape[0], w.shape[1]) is not None

    def _experts_streamable(self, lw) -> bool:
        return bool(lw.E) and hops.moe_grouped_ok(torch.empty(1, lw.w_up.shape[2], dtype=lw.w_up.dtype,
                                                              device=self.device), lw.w_up, lw.w_down, glu=False) and \
            ops.stream_moe_supported(lw.w_up.shape[1], lw.w_up.shape[2]) and \
            ops.stream_moe_supported(lw.w_down.shape[1], lw.w_down.shape[2])

    def stream_weight_bytes(self) -> int:
        ws = [getattr(lw, n, None) for lw in self.layers for n in self.STREAMED] + [self.head, self.loop_in]
        return sum(w.numel() * w.element_size() for w in ws if self._streamable(w))

    def enable_stream_weights(self, tiled_only: bool = False) -> int:
        """Wave-tiled copies of the projections (ops.tile_weight) and of the experts (ops.tile_experts) so that
        decode-sized steps (<= ops.STREAM_MAX_M rows; experts: <= hops.MOE_STREAM_MAX_T) run them on the framework's
        weight-streaming MFMA kernels; prefill-sized steps and shapes the kernels do not take stay on hipBLASLt and
        the expert-sorted GEMMs. bf16 only. Returns the added bytes."""
        added = 0
        for lw in self.layers:
            for n in self.STREAMED:
                w = getattr(lw, n, None)
                if self._streamable(w):
                    setattr(lw, n + "_t", ops.tile_weight(w))
                    added += w.numel() * w.element_size()
            if self._experts_streamable(lw):
                lw.w_up_t, lw.w_down_t = ops.tile_experts(lw.w_up), ops.tile_experts(lw.w_down)
                added += (lw.w_up.numel() + lw.w_down.numel()) * lw.w_up.element_size()
        for n in ("head", "loop_in"):
            w = getattr(self, n)
            if self._streamable(w):
                setattr(self, n + "_t", ops.tile_weight(w))
                added += w.numel() * w.element_size()
        self.stream = added > 0
        self.stream_max_m = ops.STREAM_MAX_M
        return added

    def _lin(self, x, w, wt=None, slabs: bool = False):
        """x @ w^T: the weight-streaming kernel for decode-sized steps when the weight has a tiled copy, else
        hipBLASLt. ``slabs``: the caller takes the split-K slabs [S, T, N] as they are."""
        M = x.shape[0]
        if self.stream and wt is not None and 0 < M <= self.stream_max_m and \
                ops.stream_plan(M, w.shape[0], w.shape[1]) is not None:
            y = ops.linear_stream(x, wt)
            return ops.slab_reduce(y) if ops.is_slab(y) and not slabs else y
        return F.linear(x, w)

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self._tensors)

    # weights --------------------------------------------------------------------------------------------------
    def load_tensors(self, W: dict[str, torch.Tensor]) -> "FurapelLM":
        """Checkpoint tensors (any float dtype) -> device tensors: projections that read the same input fused into
        one GEMM weight in the model dtype (rows padded to a multiple of 32), per-head up-projections reshaped for the
        batched latent products, experts stacked; the tanh norms, gate biases and the router fp32, the embedding scale
        folded into an fp32 copy of the table."""
        cfg, dev, dt = self.cfg, self.device, self.dtype
        self.runs = cfg.runs()
        for k, shp in tensor_shapes(cfg).items():
            if k not in W:
                raise KeyError(f"checkpoint lacks tensor {k!r}")
            if tuple(W[k].shape) != tuple(shp):
                raise ValueError(f"tensor {k!r}: shape {tuple(W[k].shape)}, config says {tuple(shp)}")
        self._tensors = []

        def keep(t):
            t = t.contiguous()
            self._tensors.append(t)
            return t

        def act(name):  # model dtype
            return keep(W[name].to(device=dev, dtype=dt))

        def f32(name):
            return keep(W[name].to(device=dev, dtype=torch.float32))

        def fused(names, dtype=dt, multiple=1):
            ws = [W[n].to(device=dev, dtype=dtype) for n in names]
            pad = -sum(w.shape[0] for w in ws) % multiple
            if pad:
                ws.append(torch.zeros(pad, *ws[0].shape[1:], dtype=dtype, device=dev))
            return keep(torch.cat(ws, 0))

        def norm(name):
            return hops.TanhNorm(float(W[name + ".alpha"].float()), f32(name), f32(name + ".b"))

        self.embed = keep(W["embed"].to(device=dev, dtype=torch.float32) * float(cfg.embed_scale))
        self.final_norm = norm("final.norm")
        self.loop_in = act("loop.in") if cfg.loop else None
        # the sampler reads logits rows in 8-element vectors: the head is padded with zero rows to a multiple of 8
        # and the extra columns are cut off as a view
        self.head = fused(["head"], multiple=8)
        self.layers = []
        tiles = set()
        for i, L in enumerate(cfg.layers):
            p, m = f"l{i}.", L["mixer"]
            q = p + "mix."
            lw = _Layer()
            lw.type, lw.m = L["type"], m
            lw.norm1, lw.o = norm(p + "norm1"), act(q + "o")
            mask = m.get("mask") or {}
            lw.window = int(mask["size"]) if mask.get("size") is not None else 0   # 0 = every earlier position
            if mask.get("size") is not None and lw.window < 1:
                raise ValueError(f"layer {i}: mask.size must be at least 1")
            if lw.type == "attention":
                H, G, D = (int(m[k]) for k in ("heads", "kv_heads", "dim"))
                if G < 1 or H % G:
                    raise ValueError(f"layer {i}: {H} query heads over {G} key/value heads")
                lw.w_in = fused([q + n for n in ("q", "k", "v", "g")], multiple=32)
                lw.scale = float(m["scale"])
                rot = m.get("rot") or None
                lw.rot_dims = int(rot["dims"]) if rot else 0
                if lw.rot_dims > D or lw.rot_dims % 2:
                    raise ValueError(f"layer {i}: rot.dims must be even and at most the head size")
                lw.cos_sin = self._rot_table(rot) if lw.rot_dims else None
                tiles.add(hops.sig_tile_tokens(H, G))
            elif lw.type == "latent_attention":
                H, D, Dv, R = (int(m[k]) for k in ("heads", "dim", "vdim", "kv_rank"))
                lw.w_in = fused([q + "q", q + "dkv"], multiple=32)                  # row = [q heads | latent]
                lw.dkv_norm = act(q + "dkv.norm")
                lw.uk_h = act(q + "uk").view(H, D, R)                              # q_lat = q @ uk_h  (per head)
                lw.uv_ht = keep(W[q + "uv"].to(device=dev, dtype=dt).view(H, Dv, R).transpose(1, 2))
                lw.scale = float(m["scale"])
                tiles.add(hops.tile_tokens(H))
            else:
                lw.w_in = fused([q + n for n in ("q", "k", "v", "g")], multiple=32)
                lw.gate_w = fused([q + "i", q + "f"])
                lw.gate_b = fused([q + "i.b", q + "f.b"], torch.float32)
                lw.mnorm = act(q + "norm")
                lw.cap = float(m["gate_cap"])
                if not lw.cap > 0:
                    raise ValueError(f"layer {i}: gate_cap must be positive")
            lw.E = 0
            if L.get("mlp"):
                lw.E, lw.top, lw.ff = _moe_sizes(L["mlp"])
                if not 1 <= lw.top <= lw.E:
                    raise ValueError(f"layer {i}: top {lw.top} of {lw.E} experts")
                lw.norm2, lw.router = norm(p + "norm2"), f32(p + "mlp.router")
                low = lw.router.to(dt)                                              # where it is exact: one kernel
                lw.router_a = keep(low) if dt != torch.float32 and torch.equal(low.float(), lw.router) else None
                lw.w_up = keep(torch.stack([W[f"{p}mlp.e{e}.up"] for e in range(lw.E)]).to(device=dev, dtype=dt))
                lw.w_down = keep(torch.stack([W[f"{p}mlp.e{e}.down"] for e in range(lw.E)]).to(device=dev, dtype=dt))
            self.layers.append(lw)
        # tile sizes (tokens) the step plan must carry for the matrix-core attention kernels
        self.attn_tile_tokens = sorted(tiles)
        return self

    def _rot_table(self, rot: dict) -> torch.Tensor:
        """fp32 [positions, dims]: cos | sin of fp32 position x fp32 frequency, one table per rotation."""
        key = json.dumps(rot, sort_keys=True)
        if key not in self._rot:
            self._rot[key] = rotary_table(self.max_positions, rot, self.device)
        return self._rot[key]

    # caches ---------------------------------------------------------------------------------------------------
    def page_bytes(self) -> int:
        """Bytes of one 16-token page over every layer run."""
        es = torch.empty(0, dtype=self.dtype).element_size()
        n = 0
        for i, _ in self.cfg.runs():
            L = self.cfg.layers[i]
            m = L["mixer"]
            if L["type"] == "attention":
                n += int(m["kv_heads"]) * (int(m["dim"]) + int(m["vdim"]))
            elif L["type"] == "latent_attention":
                # (the latent is kept twice where the matrix-core kernel runs: row-major and page-wise transposed)
                n += 2 * int(m["kv_rank"])
        return PAGE * n * es or 1

    def alloc_cache(self, num_blocks: int, num_slots: int):
        """Per layer run: (keys [blocks, 16, G dim], values [blocks, G vdim, 16]), or the latent pool [blocks, 16,
        kv_rank], or None; and the slot state S [slots, heads, dim, vdim], n, m, fp32. Zeroed once: a masked key's row
        is never used, but fresh memory must not hold NaN patterns for the debug checks."""
        dev, dt = self.device, self.dtype
        pages, state = [], LayerState()
        self.pages_t = []  # page-wise transposed latent copies [blocks, kv_rank, 16] for the matrix-core kernel
        for i, _ in self.runs:
            lw = self.layers[i]
            m, st, pt = lw.m, {}, None
            if lw.type == "attention":
                G, D, Dv = (int(m[k]) for k in ("kv_heads", "dim", "vdim"))
                pages.append((torch.zeros(num_blocks, PAGE, G * D, dtype=dt, device=dev),
                              torch.zeros(num_blocks, G * Dv, PAGE, dtype=dt, device=dev)))
            elif lw.type == "latent_attention":
                R = int(m["kv_rank"])
                pages.append(torch.zeros(num_blocks, PAGE, R, dtype=dt, device=dev))
                if hops.latent_mfma_ok(pages[-1], R, 0):
                    pt = torch.zeros(num_blocks, R, PAGE, dtype=dt, device=dev)
            else:
                H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
                pages.append(None)
                st["S"] = torch.zeros(num_slots, H, D, Dv, dtype=torch.float32, device=dev)
                st["n"] = torch.zeros(num_slots, H, D, dtype=torch.float32, device=dev)
                st["m"] = torch.zeros(num_slots, H, dtype=torch.float32, device=dev)
            self.pages_t.append(pt)
            state.layers.append(st)
        return pages, state

    # one step ---------------------------------------------------------------------------------------------------
    def forward(self, inp, pages: list, state: LayerState, gather: bool = True,
                layers_out: list | None = None) -> torch.Tensor:
        """Logits fp32 [n, V] for ``inp.logit_rows``. ``layers_out``: a list that receives the residual stream after
        every layer run (fp32 [T, d] copies; debugging and the per-layer tests)."""
        cfg, dt, dev = self.cfg, self.dtype, self.device
        m: SegMeta = inp.attn
        T, d = inp.tokens.shape[0], cfg.hidden_size
        x = F.embedding(inp.tokens, self.embed)       # fp32 [T, d] residual (the table holds the scale)
        h1, h2 = (torch.empty(T, d, dtype=dt, device=dev) for _ in range(2))
        both = None                                   # the loop product's input [residual | embedding rows]
        if self.loop_in is not None:
            both = torch.empty(T, 2 * d, dtype=dt, device=dev)
            both[:, d:] = x

        def outputs(r):
            """What the element-wise pass in front of run r leaves: the norms of its layer, or - where a pass of the
            loop starts - the residual's copy for the loop product."""
            if r == len(self.runs):
                return {}
            i, enters = self.runs[r]
            return {"copy": both[:, :d]} if enters else norms(self.layers[i])

        def norms(lw):
            return {"norms": [lw.norm1] + ([lw.norm2] if lw.E else []), "outs": [h1] + ([h2] if lw.E else [])}

        if self.runs:
            hops.add_tanh_norm(x, **outputs(0))
        for r, (i, enters) in enumerate(self.runs):
            lw, st = self.layers[i], state.layers[r]
            if enters:
                y = self._loop_product(both)
                hops.add_tanh_norm(x, y, assign=True, **norms(lw))
            if lw.type == "attention":
                y = self._attention(r, lw, h1, inp, m, pages)
            elif lw.type == "latent_attention":
                y = self._latent_attention(r, lw, h1, inp, m, pages)
            else:
                y = self._mlstm(lw, h1, m, st)
            ye = self._experts(lw, h2) if lw.E else None
            hops.add_tanh_norm(x, y, ye, **outputs(r + 1))
            if layers_out is not None:
                layers_out.append(x.clone())
        xs = x.index_select(0, inp.logit_rows)
        hf = torch.empty(xs.shape[0], d, dtype=dt, device=dev)
        hops.add_tanh_norm(xs, norms=[self.final_norm], outs=[hf])
        logits = self._lin(hf, self.head, getattr(self, "head_t", None)).float()
        if cfg.logit_scale != 1.0:
            logits.mul_(cfg.logit_scale)
        return logits[:, :cfg.vocab_size]   # (a view: the padded row stride is what the sampler reads)

    def _loop_product(self, both):
        """W_in [x | x0] with an fp32 result (or fp32 slabs of it): the residual is not rounded."""
        wt = getattr(self, "loop_in_t", None)
        if self.stream and wt is not None and 0 < both.shape[0] <= self.stream_max_m:
            y = self._lin(both, self.loop_in, wt, slabs=True)
            if ops.is_slab(y):
                return y
        return hops.linear_f32(both, self.loop_in)

    def _attention(self, r: int, lw, h, inp, m: SegMeta, pages: list) -> torch.Tensor:
        mm = lw.m
        H, G, D, Dv = (int(mm[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        T, dt, dev = h.shape[0], self.dtype, self.device
        proj = self._lin(h, lw.w_in, getattr(lw, "w_in_t", None))                 # [q | k | v | head gates]
        k_cache, v_cache_t = pages[r]
        q = torch.empty(T, H * D, dtype=dt, device=dev)
        hops.rope_kv_store(proj, H, G, D, Dv, inp.positions, lw.cos_sin, lw.rot_dims, False, None, k_cache, v_cache_t,
                           inp.slot_mapping, q)
        ao = torch.empty(T, H * Dv, dtype=dt, device=dev)
        hops.window_attn(q, k_cache, v_cache_t, m.block_tables, m.tok_seg, inp.positions, H, G, lw.scale, lw.window,
                         None, ao, m.tiles.get(hops.sig_tile_tokens(H, G)), m.max_keys, gate=proj,
                         gate_off=H * D + G * D + G * Dv, kinds=m.tile_kinds(hops.sig_tile_tokens(H, G)))
        return self._lin(ao, lw.o, getattr(lw, "o_t", None), slabs=True)

    def _latent_attention(self, r: int, lw, h, inp, m: SegMeta, pages: list) -> torch.Tensor:
        mm = lw.m
        H, D, Dv, R = (int(mm[k]) for k in ("heads", "dim", "vdim", "kv_rank"))
        T, dt, dev = h.shape[0], self.dtype, self.device
        qd = self._lin(h, lw.w_in, getattr(lw, "w_in_t", None))                    # [q heads | latent]
        cache, cache_t = pages[r], self.pages_t[r]
        q_rot = torch.empty(T, H, 0, dtype=dt, device=dev)                         # (no rotated part in this family)
        hops.latent_prep(qd, H, D, 0, R, H * D, lw.dkv_norm, self.cfg.norm_eps, inp.positions, None, 0, cache,
                         inp.slot_mapping, q_rot, cache_t)
        q_u = qd[:, :H * D].view(T, H, D).transpose(0, 1)                          # [H, T, dim] (strided view)
        q_lat = torch.bmm(q_u, lw.uk_h)                                            # [H, T, R]
        o_lat = torch.empty(H, T, R, dtype=dt, device=dev)
        hops.latent_attn(q_lat, q_rot, cache, m.block_tables, m.tok_seg, m.seg, inp.positions, lw.scale, o_lat,
                         cache_t, m.tiles.get(hops.tile_tokens(H)), m.max_keys, window=lw.window)
        ao = torch.empty(T, H * Dv, dtype=dt, device=dev)
        torch.bmm(o_lat, lw.uv_ht, out=ao.view(T, H, Dv).transpose(0, 1))          # head h -> its vdim columns
        return self._lin(ao, lw.o, getattr(lw, "o_t", None), slabs=True)

    def _mlstm(self, lw, h, m: SegMeta, st: dict) -> torch.Tensor:
        H, D, Dv = (int(lw.m[k]) for k in ("heads", "dim", "vdim"))
        T, dt, dev = h.shape[0], self.dtype, self.device
        proj = self._lin(h, lw.w_in, getattr(lw, "w_in_t", None))                 # [q | k | v | output gate]
        gates = hops.linear_f32(h, lw.gate_w, lw.gate_b)                           # fp32 [T, 2 H]: input | forget
        o = torch.empty(T, H * Dv, dtype=torch.float32, device=dev)
        chunks, short = m.chunks(hops.MLSTM_CHUNK, hops.MLSTM_CHUNK_MIN)
        hops.mlstm_scan(proj, gates, H, D, Dv, lw.cap, m.tok_seg, m.seg, st["S"], st["n"], st["m"], o, chunks, short)
        on = torch.empty(T, H * Dv, dtype=dt, device=dev)
        hops.head_norm_gate(o, lw.mnorm, proj, 2 * H * D + H * Dv, H, self.cfg.norm_eps, on)
        return self._lin(on, lw.o, getattr(lw, "o_t", None), slabs=True)

    def _experts(self, lw, h):
        """The routed experts' weighted sum, fp32 [T, d], or of a long step its rows (``hops.ExpertRows``)."""
        tw, te, _ = hops.moe_router_grouped(h, lw.router, None, lw.top, 1, 1, norm=False, w_act=lw.router_a)
        T, up_t, down_t = h.shape[0], getattr(lw, "w_up_t", None), getattr(lw, "w_down_t", None)
        if up_t is not None and hops.moe_wide(T, lw.top, lw.E):
            return hops.moe_expert_rows(h, up_t, down_t, tw, te, lw.E)
        out = torch.empty(T, self.cfg.hidden_size, dtype=torch.float32, device=self.device)
        hops.moe_experts(h, lw.w_up, lw.w_down, tw, te, out, up_t, down_t, act="relu2")
        return out


def load_checkpoint(model: FurapelLM, path: str | Path) -> FurapelLM:
    """``path``: a folder holding model.safetensors (or any *.safetensors), or such a file."""
    from safetensors import safe_open

    path = Path(path)
    files = sorted(path.glob("*.safetensors")) if path.is_dir() else [path]
    W = {}
    for f in files:
        with safe_open(str(f), framework="pt", device="cpu") as h:
            for k in h.keys():
                W[k] = h.get_tensor(k)
    return model.load_tensors(W)


def save_checkpoint(cfg: FurapelConfig, W: dict[str, torch.Tensor], folder: str | Path) -> None:
    from safetensors.torch import save_file

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    save_file({k: v.contiguous() for k, v in W.items()}, str(folder / "model.safetensors"))
    (folder / "config.json").write_text(json.dumps(cfg.to_dict(), indent=1))
