"""Rogosun: a decoder of linear-attention layers and parallel layers (softmax attention beside the gated delta rule) with
norms on the sublayers' outputs only.

Residual. The sublayers read the residual x itself; what they give is normed before it is added:

    x <- x + rms_norm(mixer(x)) * w1        x <- x + rms_norm(ff(x)) * w2

Mixers
  gla         gated linear attention: per head a matrix state S (dim x vdim) with a decay per key channel,
              a = sigmoid(W_a2 W_a1 h + b)^(1 / tau), S <- diag(a) S + k v^T, read-out S^T q dim^(-1/2); the read-out is
              RMS-normed per head (one weight vector for all heads), times silu(W_g h), then W_o.
  parallel    two mixers read the same input, result = left_scale * left + right_scale * right.
              left: grouped-query softmax attention whose values are the keys as projected (there is no value
              projection); RMS norm of every q and k head, then rotation of dimension i with i + rot.dims / 2 on the
              first rot.dims dimensions (frequencies divided by rot.scaling.factor); a further score of 0 without a
              value joins the softmax denominator.
              right: gated delta rule. q, k, v pass a short causal per-channel convolution and silu; q and k become unit
              vectors per head; beta = sigmoid(W_b h) per head; a decay per head and key channel
              a = exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)); S <- diag(a) S, u = beta (v - S^T k),
              S <- S + k u^T, read-out S^T q dim^(-1/2), RMS-normed per head, times sigmoid(W_g2 W_g1 h), then W_o.
Feed-forward  dense: W_down relu(W_up h)^2; or routed experts W_down (silu(W_gate h) * W_up h): sigmoid scores from fp32
              logits, the ``top`` largest within the ``groups.keep`` groups of neighbours with the largest sum of their
              two largest scores, weighted by the scores themselves times ``scale``, plus a shared expert of the same
              form for every row.

How the engine runs it. The projections of a layer that read x are one GEMM (sections padded to 8 columns); the two
low-rank second factors of a delta mixer (decay and output gate) are one product with a block-diagonal weight; the two
output projections of a parallel layer are one product over [left heads | right heads]. The zero score of the softmax is
the windowed-attention kernels' sink logit 0. The norm and the add to the residual are one kernel that also sums a
split-K projection's slabs and leaves x in the model dtype for the next sublayer. Long portions run both recurrences in
chunks of matrix products (``ops.hybrid.lin_scan``), short ones token by token.

Per sequence the engine keeps pages (keys, normed and rotated, and page-wise transposed raw keys as values, of every
parallel layer; page ids shared by all layers) and one state slot (the matrix states, fp32; the last conv inputs). The
residual, norms, rotation, scores, softmax, router, decays, step sizes and states are fp32; projections run in the model
dtype (bf16, or fp32 throughout).

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
class RogosunConfig:
    name: str = "rogosun"
    arch: str = "rogosun"
    vocab_size: int = 0
    hidden_size: int = 0
    layers: list = field(default_factory=list)   # config.json's entries: {"type", "mixer": {...}, "mlp": {...}|None}
    norm_eps: float = 1e-5
    max_position_embeddings: int = 1 << 20
    bos_token_id: int = 0
    eos_token_ids: list = field(default_factory=list)
    tie_word_embeddings: bool = False
    num_experts: int = 0

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @staticmethod
    def from_dict(c: dict, name: str = "rogosun") -> "RogosunConfig":
        return RogosunConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]),
                             layers=list(c["layers"]), norm_eps=float(c["norm"]["eps"]))

    @staticmethod
    def from_json(path: str | Path) -> "RogosunConfig":
        path = Path(path)
        return RogosunConfig.from_dict(json.loads(path.read_text()), name=path.parent.name)

    def to_dict(self) -> dict:
        return {"architecture": "Rogosun", "vocab": self.vocab_size, "width": self.hidden_size, "layers": self.layers,
                "norm": {"eps": self.norm_eps}}

    def num_params(self) -> int:
        return sum(math.prod(s) for s in tensor_shapes(self, ranks=_RANKS).values())


# ranks of the low-rank factors of models that have no checkpoint (a checkpoint's tensors bring their own)
_RANKS = {"gla.a": 16, "right.a": 64, "right.g": 64}


def _moe_sizes(mlp: dict) -> dict:
    """Sizes and constants of a routed feed-forward entry."""
    r = mlp["router"]
    gr = r.get("groups") or {}
    sh = mlp.get("shared") or None
    return {"E": int(r["experts"]), "top": int(r["top"]), "ff": int(mlp["expert"]["ff"]),
            "groups": int(gr.get("count", 1)), "keep": int(gr.get("keep", 1)), "scale": float(r.get("scale", 1.0)),
            "shared_ff": int(sh["ff"]) if sh else 0}


def tensor_shapes(cfg: RogosunConfig, W: dict | None = None, ranks: dict | None = None) -> dict[str, tuple]:
    """Checkpoint tensor names -> shapes of a model with this config. The ranks of the low-rank factors are not in the
    config: they are taken from the tensors ``W``, or from ``ranks``."""
    d, V = cfg.hidden_size, cfg.vocab_size

    def rank(kind: str, name: str) -> int:
        if W is not None:
            if name not in W:
                raise KeyError(f"checkpoint lacks tensor {name!r}")
            return int(W[name].shape[0])
        return ranks[kind]

    s: dict[str, tuple] = {"embed": (V, d)}
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.", L["mixer"]
        s[p + "norm1"] = (d,)
        if L["type"] == "gla":
            H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
            q = p + "mix."
            s[q + "q"], s[q + "k"], s[q + "v"], s[q + "g"] = (H * D, d), (H * D, d), (H * Dv, d), (H * Dv, d)
            s[q + "o"], s[q + "norm"] = (d, H * Dv), (Dv,)
            ra = rank("gla.a", q + "a1")
            s[q + "a1"], s[q + "a2"], s[q + "a2.b"] = (ra, d), (H * D, ra), (H * D,)
        elif L["type"] == "parallel":
            a, b = m["left"], m["right"]
            H, G, D = (int(a[k]) for k in ("heads", "kv_heads", "dim"))
            q = p + "mix.left."
            s[q + "q"], s[q + "k"], s[q + "q.norm"], s[q + "k.norm"] = (H * D, d), (G * D, d), (D,), (D,)
            s[q + "o"] = (d, H * D)
            H, G, D, Dv, taps = (int(b[k]) for k in ("heads", "kv_heads", "dim", "vdim", "conv"))
            q = p + "mix.right."
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                s[q + n], s[q + n + ".conv"] = (rows, d), (rows, taps)
            ra, rg = rank("right.a", q + "a1"), rank("right.g", q + "g1")
            s[q + "b"], s[q + "A_log"], s[q + "norm"] = (H, d), (H,), (Dv,)
            s[q + "a1"], s[q + "a2"], s[q + "dt_bias"] = (ra, d), (H * D, ra), (H * D,)
            s[q + "g1"], s[q + "g2"], s[q + "o"] = (rg, d), (H * Dv, rg), (d, H * Dv)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {L['type']!r}")
        mlp = L.get("mlp")
        if mlp:
            s[p + "norm2"] = (d,)
            q = p + "mlp."
            kind = mlp.get("kind")
            if kind == "dense":
                s[q + "up"], s[q + "down"] = (int(mlp["ff"]), d), (d, int(mlp["ff"]))
            elif kind == "moe":
                z = _moe_sizes(mlp)
                for e in range(z["E"]):
                    s[f"{q}e{e}.gate"], s[f"{q}e{e}.up"], s[f"{q}e{e}.down"] = (z["ff"], d), (z["ff"], d), (d, z["ff"])
                s[q + "router"] = (z["E"], d)
                if z["shared_ff"]:
                    fs = z["shared_ff"]
                    s[q + "shared.gate"], s[q + "shared.up"], s[q + "shared.down"] = (fs, d), (fs, d), (d, fs)
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {kind!r}")
    s["final.norm"], s["head"] = (d,), (V, d)
    return s


def random_tensors(cfg: RogosunConfig, seed: int = 0, device="cpu", ranks: dict | None = None) -> dict[str, torch.Tensor]:
    """Seeded bf16 weights with the value ranges each kind of tensor needs (norm weights around one, decays that mostly
    keep), drawn on ``device``."""
    g = torch.Generator(device=device).manual_seed(seed)

    def rn(shape):
        return torch.randn(shape, generator=g, device=device)

    def ru(shape):
        return torch.rand(shape, generator=g, device=device)

    out = {}
    for name, shape in tensor_shapes(cfg, ranks=ranks or _RANKS).items():
        leaf = name.split(".")[-1]
        if leaf in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.1 * rn(shape)
        elif leaf == "b" and name.endswith("a2.b"):
            t = 1.0 + rn(shape)
        elif leaf == "A_log":
            t = torch.log(0.5 + 3.5 * ru(shape))
        elif leaf == "dt_bias":
            t = -4.0 + 4.0 * ru(shape)
        elif leaf == "embed":
            t = rn(shape)
        elif leaf == "router":
            t = rn(shape) * 2.0 / math.sqrt(shape[-1])
        else:
            t = rn(shape) / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out


class LayerState:
    """Per-layer dicts of state tensors, one row per state slot: ``S`` (matrix states, fp32) and, for parallel layers,
    ``conv`` (last conv inputs, model dtype)."""

    def __init__(self):
        self.layers: list[dict] = []

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for st in self.layers for t in st.values())


class _Layer:
    pass


def _sections(parts: list[tuple[str, torch.Tensor]], multiple: int = 32) -> tuple[torch.Tensor, dict[str, int]]:
    """Weights [rows_i, d] below one another, each starting at a multiple of 8 rows, the whole a multiple of
    ``multiple`` rows (zero rows between): (weight, first row of each part)."""
    off, rows, at = {}, [], 0
    d = parts[0][1].shape[1]

    def pad(n):
        nonlocal at
        if n:
            rows.append(torch.zeros(n, d, dtype=parts[0][1].dtype, device=parts[0][1].device))
            at += n

    for name, w in parts:
        pad(-at % 8)
        off[name] = at
        rows.append(w)
        at += w.shape[0]
    pad(-at % multiple)
    return torch.cat(rows, 0), off


class RogosunLM:
    plan = "segments"  # the model runner plans its steps as SegMeta runs (engine/model_runner.py)

    def __init__(self, cfg: RogosunConfig, device, dtype=torch.bfloat16, tp: int = 1, tp_rank: int = 0,
                 max_positions: int | None = None):
        if tp != 1:
            raise ValueError("Rogosun runs unsharded (tp = 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Rogosun runs in bfloat16 or float32")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp, self.tp_rank, self.ep, self.ep_rank = 1, 0, 1, 0
        self.dp_attention = False
        self.stream = self.tiled_only = False
        self.stream_max_m = 0
        self.max_positions = int(max_positions or 8192)
        self.layers: list[_Layer] = []
        self.attn_tile_tokens: list[int] = []
        self._rot: dict = {}

    # engine hooks shared with the other model classes ---------------------------------------------------------------
    STREAMED = ("w_in", "o", "up", "down", "sh_down")

    def _streamable(self, w) -> bool:
        return w is not None and w.dtype == torch.bfloat16 and w.is_cuda and \
            ops.stream_plan(1, w.shape[0], w.shape[1]) is not None

    def stream_weight_bytes(self) -> int:
        ws = [getattr(lw, n, None) for lw in self.layers for n in self.STREAMED + ("sh_gu",)] + [self.head]
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
            if lw.ff != "moe":
                continue
            if self._streamable(lw.sh_gu) and lw.sh_gu.shape[0] % 64 == 0:   # shared expert: silu * up in the epilogue
                lw.sh_gu_t = ops.tile_weight(lw.sh_gu, glu=True)
                added += lw.sh_gu.numel() * lw.sh_gu.element_size()
            if lw.w_gu.is_cuda and lw.w_gu.dtype == torch.bfloat16 and \
                    hops.moe_grouped_ok(torch.empty(1, lw.w_gu.shape[2], dtype=lw.w_gu.dtype, device=self.device),
                                        lw.w_gu, lw.w_down) and \
                    ops.stream_moe_supported(lw.w_gu.shape[1], lw.w_gu.shape[2]) and \
                    ops.stream_moe_supported(lw.w_down.shape[1], lw.w_down.shape[2]):
                lw.w_gu_t = ops.tile_experts(lw.w_gu, glu=True)   # routed experts: grouped streaming kernel
                lw.w_down_t = ops.tile_experts(lw.w_down)
                added += (lw.w_gu.numel() + lw.w_down.numel()) * lw.w_gu.element_size()
        if self._streamable(self.head):
            self.head_t = ops.tile_weight(self.head)
            added += self.head.numel() * self.head.element_size()
        self.stream = added > 0
        self.stream_max_m = ops.STREAM_MAX_M
        return added

    def _streams(self, M: int, w, wt) -> bool:
        return self.stream and wt is not None and 0 < M <= self.stream_max_m and \
            ops.stream_plan(M, w.shape[0], w.shape[1]) is not None

    def _lin(self, x, w, wt=None, slabs: bool = False):
        """x @ w^T: the weight-streaming kernel for decode-sized steps when the weight has a tiled copy, else
        hipBLASLt. ``slabs``: the caller takes the split-K slabs [S, T, N] as they are."""
        if self._streams(x.shape[0], w, wt):
            y = ops.linear_stream(x, wt)
            return ops.slab_reduce(y) if ops.is_slab(y) and not slabs else y
        return F.linear(x, w)

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self._tensors)

    # weights --------------------------------------------------------------------------------------------------
    def load_tensors(self, W: dict[str, torch.Tensor]) -> "RogosunLM":
        """Checkpoint tensors (any float dtype) -> device tensors: projections that read the same input fused into
        one GEMM weight in the model dtype, the low-rank second factors of a delta mixer on the diagonal of one weight,
        a parallel layer's output projections side by side, experts stacked; norm weights of the residual and of the
        query / key heads, decay biases and rates and the router fp32."""
        cfg, dev, dt = self.cfg, self.device, self.dtype
        for k, shp in tensor_shapes(cfg, W).items():
            if k not in W:
                raise KeyError(f"checkpoint lacks tensor {k!r}")
            if tuple(W[k].shape) != tuple(shp):
                raise ValueError(f"tensor {k!r}: shape {tuple(W[k].shape)}, config says {tuple(shp)}")
        self._tensors = []

        def keep(t):
            t = t.contiguous()
            self._tensors.append(t)
            return t

        def raw(name):
            return W[name].to(device=dev, dtype=dt)

        def act(name):  # model dtype
            return keep(raw(name))

        def f32(name):
            return keep(W[name].to(device=dev, dtype=torch.float32))

        d = cfg.hidden_size
        self.embed = f32("embed")  # the residual starts (and stays) fp32; bf16 table values are exact in it
        self.final_norm = act("final.norm")
        # the sampler reads logits rows in 8-element vectors: the head is padded with zero rows to a multiple of 8
        # and the extra columns are cut off as a view
        pad = -cfg.vocab_size % 8
        self.head = keep(torch.cat([raw("head"), torch.zeros(pad, d, dtype=dt, device=dev)], 0))
        self.layers = []
        tiles = set()
        for i, L in enumerate(cfg.layers):
            p, m = f"l{i}.", L["mixer"]
            lw = _Layer()
            lw.type, lw.m = L["type"], m
            lw.norm1 = f32(p + "norm1")
            if lw.type == "gla":
                H = int(m["heads"])
                q = p + "mix."
                lw.tau = float(m["tau"])
                if not lw.tau > 0:
                    raise ValueError(f"layer {i}: tau must be positive")
                w_in, lw.off = _sections([(n, raw(q + n)) for n in ("q", "k", "v", "g", "a1")])
                lw.w_in = keep(w_in)
                a2 = raw(q + "a2")                                    # zero columns up to a multiple of 8: the padding
                lw.low = keep(F.pad(a2, (0, -a2.shape[1] % 8)))       # columns behind a1 in the fused row are zero too
                lw.z_bias = f32(q + "a2.b")
                lw.hnorm = keep(raw(q + "norm").repeat(H))            # one weight vector for all heads
                lw.o = act(q + "o")
            else:
                a, b = m["left"], m["right"]
                H, G, D = (int(a[k]) for k in ("heads", "kv_heads", "dim"))
                if G < 1 or H % G:
                    raise ValueError(f"layer {i}: {H} query heads over {G} key heads")
                if int(a.get("vdim", D)) != D:
                    raise ValueError(f"layer {i}: keys double as values, so dim and vdim must agree")
                Hr, Gr, Dr, Dvr = (int(b[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
                if Gr < 1 or Hr % Gr:
                    raise ValueError(f"layer {i}: {Hr} delta-rule heads over {Gr} query/key heads")
                q, r = p + "mix.left.", p + "mix.right."
                qkv = torch.cat([raw(r + n) for n in ("q", "k", "v")], 0)
                a1, g1 = raw(r + "a1"), raw(r + "g1")
                w_in, lw.off = _sections([("qk", torch.cat([raw(q + "q"), raw(q + "k")], 0)), ("conv", qkv),
                                          ("low", torch.cat([a1, g1], 0)), ("b", raw(r + "b"))])
                lw.w_in = keep(w_in)
                lw.conv = keep(torch.cat([raw(r + n + ".conv") for n in ("q", "k", "v")], 0))
                low = torch.block_diag(raw(r + "a2").float(), raw(r + "g2").float()).to(dt)
                lw.low = keep(F.pad(low, (0, -low.shape[1] % 8)))
                lw.z_bias = f32(r + "dt_bias")
                lw.rate = keep(-torch.exp(W[r + "A_log"].to(device=dev, dtype=torch.float32)))
                lw.hnorm = keep(raw(r + "norm").repeat(Hr))
                lw.q_norm, lw.k_norm = f32(q + "q.norm"), f32(q + "k.norm")
                lw.sink = keep(torch.zeros(H, dtype=torch.float32, device=dev))   # the denominator's further score
                rot = a.get("rot") or None
                lw.rot_dims = int(rot["dims"]) if rot else 0
                if lw.rot_dims > D or lw.rot_dims % 2:
                    raise ValueError(f"layer {i}: rot.dims must be even and at most the head size")
                lw.cos_sin = self._rot_table(rot) if lw.rot_dims else None
                lw.scale = float(a["scale"])
                lw.left_scale, lw.right_scale = float(m["left_scale"]), float(m["right_scale"])
                lw.o = keep(torch.cat([raw(q + "o"), raw(r + "o")], 1))           # [left heads | right heads]
                tiles.add(hops.sig_tile_tokens(H, G))
            mlp = L.get("mlp")
            lw.ff = mlp["kind"] if mlp else None
            if lw.ff:
                lw.norm2 = f32(p + "norm2")
            if lw.ff == "dense":
                lw.up, lw.down = act(p + "mlp.up"), act(p + "mlp.down")
            elif lw.ff == "moe":
                z = _moe_sizes(mlp)
                E = z["E"]
                if not 1 <= z["top"] <= E or z["groups"] < 1 or E % z["groups"] or \
                        not 1 <= z["keep"] <= z["groups"] or z["keep"] * (E // z["groups"]) < z["top"]:
                    raise ValueError(f"layer {i}: {z['top']} of {E} experts in {z['keep']} of {z['groups']} groups")
                lw.z = z
                lw.router = f32(p + "mlp.router")
                lw.w_gu = keep(torch.stack([torch.cat([W[f"{p}mlp.e{e}.gate"], W[f"{p}mlp.e{e}.up"]], 0)
                                            for e in range(E)]).to(device=dev, dtype=dt))       # [E, 2 ff, d]
                lw.w_down = keep(torch.stack([W[f"{p}mlp.e{e}.down"] for e in range(E)]).to(device=dev, dtype=dt))
                lw.sh_gu = lw.sh_down = None
                if z["shared_ff"]:
                    lw.sh_gu = keep(torch.cat([raw(p + "mlp.shared.gate"), raw(p + "mlp.shared.up")], 0))
                    lw.sh_down = act(p + "mlp.shared.down")
            self.layers.append(lw)
        # tile sizes (tokens) the step plan must carry for the matrix-core attention kernel
        self.attn_tile_tokens = sorted(tiles)
        return self

    def _rot_table(self, rot: dict) -> torch.Tensor:
        """fp32 [positions, dims]: cos | sin of fp32 position x fp32 frequency, one table per rotation."""
        sc = rot.get("scaling") or None
        key = (int(rot["dims"]), float(rot["base"]), float(sc["factor"]) if sc else None)
        if key not in self._rot:
            spec = {"dims": key[0], "base": key[1]}
            if sc:
                spec["scaling"] = {"factor": key[2]}
            self._rot[key] = rotary_table(self.max_positions, spec, self.device)
        return self._rot[key]

    # caches ---------------------------------------------------------------------------------------------------
    def page_bytes(self) -> int:
        """Bytes of one 16-token page over every parallel layer."""
        es = torch.empty(0, dtype=self.dtype).element_size()
        return sum(PAGE * 2 * int(L["mixer"]["left"]["kv_heads"]) * int(L["mixer"]["left"]["dim"]) * es
                   for L in self.cfg.layers if L["type"] == "parallel") or 1

    def alloc_cache(self, num_blocks: int, num_slots: int):
        """(per layer (keys [blocks, 16, G dim], values [blocks, G dim, 16]) or None, per-layer slot state: matrix states
        [slots, heads, dim, vdim] fp32, conv inputs [slots, taps - 1, channels]). Zeroed once: a masked key's row is
        never used, but fresh memory must not hold NaN patterns for the debug checks."""
        dev, dt = self.device, self.dtype
        pages, state = [], LayerState()
        for lw in self.layers:
            m, st = lw.m, {}
            if lw.type == "parallel":
                C = int(m["left"]["kv_heads"]) * int(m["left"]["dim"])
                pages.append((torch.zeros(num_blocks, PAGE, C, dtype=dt, device=dev),
                              torch.zeros(num_blocks, C, PAGE, dtype=dt, device=dev)))
                st["conv"] = torch.zeros(num_slots, lw.conv.shape[1] - 1, lw.conv.shape[0], dtype=dt, device=dev)
                m = m["right"]
            else:
                pages.append(None)
            st["S"] = torch.zeros(num_slots, int(m["heads"]), int(m["dim"]), int(m["vdim"]), dtype=torch.float32,
                                  device=dev)
            state.layers.append(st)
        return pages, state

    # one step ---------------------------------------------------------------------------------------------------
    def forward(self, inp, pages: list, state: LayerState, gather: bool = True,
                layers_out: list | None = None) -> torch.Tensor:
        """Logits fp32 [n, V] for ``inp.logit_rows``. ``layers_out``: a list that receives the residual stream after
        every layer (fp32 [T, d] copies; debugging and the per-layer tests)."""
        cfg, dt, dev = self.cfg, self.dtype, self.device
        m: SegMeta = inp.attn
        d, eps = cfg.hidden_size, cfg.norm_eps
        x = F.embedding(inp.tokens, self.embed)       # fp32 [T, d] residual
        h = torch.empty(x.shape, dtype=dt, device=dev)
        h.copy_(x)                                    # what the sublayers read: x in the model dtype
        for i, lw in enumerate(self.layers):
            st = state.layers[i]
            last = i + 1 == len(self.layers)
            y = self._gla(lw, h, m, st) if lw.type == "gla" else self._parallel(i, lw, h, inp, m, pages, st)
            hops.norm_add(x, y, None, lw.norm1, eps, None if last and not lw.ff else h)
            if lw.ff == "dense":
                u = self._lin(h, lw.up, getattr(lw, "up_t", None))
                a = torch.empty_like(u)
                hops.relu2(u, a)
                hops.norm_add(x, self._lin(a, lw.down, getattr(lw, "down_t", None), slabs=True), None, lw.norm2, eps,
                              None if last else h)
            elif lw.ff == "moe":
                y1, y2 = self._experts(lw, h)
                hops.norm_add(x, y1, y2, lw.norm2, eps, None if last else h)
            if layers_out is not None:
                layers_out.append(x.clone())
        xs = x.index_select(0, inp.logit_rows)
        hf = torch.empty(xs.shape[0], d, dtype=dt, device=dev)
        hops.rms_norm(xs, self.final_norm, eps, hf)
        return self._lin(hf, self.head, getattr(self, "head_t", None)).float()[:, :cfg.vocab_size]

    def _gla(self, lw, h, m: SegMeta, st: dict) -> torch.Tensor:
        H, D, Dv = (int(lw.m[k]) for k in ("heads", "dim", "vdim"))
        T, dt, dev, off = h.shape[0], self.dtype, self.device, lw.off
        proj = self._lin(h, lw.w_in, getattr(lw, "w_in_t", None))                 # [q | k | v | g | a1]
        z = F.linear(proj[:, off["a1"]:off["a1"] + lw.low.shape[1]], lw.low)      # raw decays
        o = torch.empty(T, H * Dv, dtype=torch.float32, device=dev)
        chunks, short = m.chunks(hops.LIN_CHUNK, hops.LIN_CHUNK_MIN)
        hops.lin_scan(proj, off["q"], off["k"], proj[:, off["v"]:off["v"] + H * Dv], z, lw.z_bias, H, H, D, Dv,
                      m.tok_seg, m.seg, st["S"], o, tau=lw.tau, chunks=chunks, rows=short)
        on = torch.empty(T, H * Dv, dtype=dt, device=dev)
        hops.head_norm_gate(o, lw.hnorm, proj, off["g"], H, self.cfg.norm_eps, on, act="silu")
        return self._lin(on, lw.o, getattr(lw, "o_t", None), slabs=True)

    def _parallel(self, i: int, lw, h, inp, m: SegMeta, pages: list, st: dict) -> torch.Tensor:
        a, b = lw.m["left"], lw.m["right"]
        H, G, D = (int(a[k]) for k in ("heads", "kv_heads", "dim"))
        Hr, Gr, Dr, Dvr = (int(b[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        T, dt, dev, off, eps = h.shape[0], self.dtype, self.device, lw.off, self.cfg.norm_eps
        # [q | k || conv inputs q | k | v | low-rank decay | gate | beta]
        proj = self._lin(h, lw.w_in, getattr(lw, "w_in_t", None))
        both = torch.empty(T, H * D + Hr * Dvr, dtype=dt, device=dev)             # [left heads | right heads]
        k_cache, v_cache_t = pages[i]
        q = torch.empty(T, H * D, dtype=dt, device=dev)
        hops.rope_kv_store(proj, H, G, D, D, inp.positions, lw.cos_sin, lw.rot_dims, False, None, k_cache, v_cache_t,
                           inp.slot_mapping, q, lw.q_norm, lw.k_norm, eps, v_off=H * D)
        hops.window_attn(q, k_cache, v_cache_t, m.block_tables, m.tok_seg, inp.positions, H, G, lw.scale, 0, lw.sink,
                         both[:, :H * D], m.tiles.get(hops.sig_tile_tokens(H, G)), m.max_keys,
                         out_scale=lw.left_scale, kinds=m.tile_kinds(hops.sig_tile_tokens(H, G)))
        qkv = torch.empty(T, lw.conv.shape[0], dtype=dt, device=dev)
        hops.short_conv(proj, off["conv"], lw.conv, None, m.tok_seg, m.seg, st["conv"], qkv, act="silu")
        low = F.linear(proj[:, off["low"]:off["low"] + lw.low.shape[1]], lw.low)  # raw decays | output gate
        o = torch.empty(T, Hr * Dvr, dtype=torch.float32, device=dev)
        chunks, short = m.chunks(hops.LIN_CHUNK, hops.LIN_CHUNK_MIN)
        hops.lin_scan(qkv, 0, Gr * Dr, qkv[:, 2 * Gr * Dr:], low[:, :Hr * Dr], lw.z_bias, Hr, Gr, Dr, Dvr, m.tok_seg,
                      m.seg, st["S"], o, rate=lw.rate, beta=proj[:, off["b"]:off["b"] + Hr], chunks=chunks,
                      rows=short)
        hops.head_norm_gate(o, lw.hnorm, low, Hr * Dr, Hr, eps, both[:, H * D:], lw.right_scale)
        return self._lin(both, lw.o, getattr(lw, "o_t", None), slabs=True)

    def _experts(self, lw, h):
        """(routed experts' weighted sum fp32 [T, d], shared expert's output [T, d] or None)."""
        z = lw.z
        T, d, dt, dev = h.shape[0], self.cfg.hidden_size, self.dtype, self.device
        tw, te, _ = hops.moe_router_grouped(h, lw.router, None, z["top"], z["groups"], z["keep"], score="sigmoid",
                                            group_score="top2", norm=False, scale=z["scale"])
        out = torch.empty(T, d, dtype=torch.float32, device=dev)
        hops.moe_experts(h, lw.w_gu, lw.w_down, tw, te, out, getattr(lw, "w_gu_t", None), getattr(lw, "w_down_t", None))
        if lw.sh_gu is None:
            return out, None
        if self._streams(T, lw.sh_gu, getattr(lw, "sh_gu_t", None)):
            a = ops.linear_glu(h, lw.sh_gu_t)
        else:
            a = torch.empty(T, z["shared_ff"], dtype=dt, device=dev)
            hops.silu_mul(F.linear(h, lw.sh_gu), a)
        return out, self._lin(a, lw.sh_down, getattr(lw, "sh_down_t", None))


def load_checkpoint(model: RogosunLM, path: str | Path) -> RogosunLM:
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


def save_checkpoint(cfg: RogosunConfig, W: dict[str, torch.Tensor], folder: str | Path) -> None:
    from safetensors.torch import save_file

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    save_file({k: v.contiguous() for k, v in W.items()}, str(folder / "model.safetensors"))
    (folder / "config.json").write_text(json.dumps(cfg.to_dict(), indent=1))
