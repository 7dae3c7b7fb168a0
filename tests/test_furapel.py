"""Furapel in the serving engine against the plain whole-sequence implementation of tests/furapel_plain.py.

Small configurations of odd sizes (nothing a multiple of 64, head sizes that differ between keys and values and between
layers, a layer without feed-forward, loops at the start, in the middle and at the end) with random weights made here. Each
test runs on the CPU reference ops and, marked ``gpu``, on the HIP kernels.
"""
import copy

import numpy as np
import pytest
import torch

import furapel_plain as plain
from kafka_llm_service_amd.engine.engine import EngineConfig, LLMEngine
from kafka_llm_service_amd.engine.sequence import SamplingParams
from kafka_llm_service_amd.models import furapel as fp
from kafka_llm_service_amd.models.budurax import rotary_table
from kafka_llm_service_amd.ops import hybrid as hops

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
YARN = {"base": 900.0, "dims": 10, "scaling": {"factor": 3.0, "original": 96, "fast": 8.0, "slow": 0.7}}


def _attn(heads=6, kv_heads=2, dim=14, vdim=11, rot=YARN, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5}
    if rot:
        m["rot"] = rot
    return m


def _latent(heads=5, dim=9, vdim=13, rank=21, window=19, scale=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "scale": scale or dim ** -0.5}
    if window:
        m["mask"] = {"size": window}
    return m


def _mlstm(heads=3, dim=12, vdim=20, cap=7.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def _moe(experts=7, top=3, ff=18):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def cfg_a(scale=None, loop=(1, 4, 2)):
    layers = [{"type": "mlstm", "mixer": _mlstm(), "mlp": _moe()},
              {"type": "latent_attention", "mixer": _latent(scale=scale), "mlp": _moe(4, 1, 30)},
              {"type": "attention", "mixer": _attn(scale=scale), "mlp": _moe(9, 4, 11)},
              {"type": "mlstm", "mixer": _mlstm(2, 30, 7, 12.0), "mlp": None},
              {"type": "attention", "mixer": _attn(3, 1, 22, 30, dict(YARN, dims=22), scale), "mlp": _moe()},
              {"type": "latent_attention", "mixer": _latent(2, 20, 6, 34, 33, scale), "mlp": None}]
    c = {"architecture": "Furapel", "vocab": 211, "width": 88, "norm": {"eps": 2e-5}, "layers": layers,
         "embedding": {"scale": 2.5}, "logit_scale": 0.3}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def cfg_b():
    """Ones and equal values: one head, as many key heads as query heads, a window of one, every expert chosen, a full
    rotation of two dimensions without scaling, scales of one, a loop that runs once over everything."""
    layers = [{"type": "attention", "mixer": _attn(1, 1, 16, 16, {"base": 100.0, "dims": 16}), "mlp": _moe(4, 4, 16)},
              {"type": "latent_attention", "mixer": _latent(1, 16, 16, 16, 1), "mlp": _moe(1, 1, 8)},
              {"type": "mlstm", "mixer": _mlstm(1, 1, 1, 1.0), "mlp": _moe(4, 2, 8)},
              {"type": "attention", "mixer": _attn(2, 2, 8, 8, {"base": 50.0, "dims": 2}), "mlp": None},
              {"type": "latent_attention", "mixer": _latent(2, 1, 1, 8, 0), "mlp": _moe(3, 1, 1)}]
    return {"architecture": "Furapel", "vocab": 97, "width": 48, "norm": {"eps": 1e-6}, "layers": layers,
            "embedding": {"scale": 1.0}, "logit_scale": 1.0, "loop": {"start": 0, "stop": 5, "times": 1}}


class Bench:
    """A config, its random weights and engines over them."""

    def __init__(self, cfg: dict, seed=0, keep=0.0):
        self.cfg = cfg
        self.mc = fp.FurapelConfig.from_dict(cfg, name="test")
        self.W = fp.random_tensors(self.mc, seed)
        for k in self.W:
            if keep and k.endswith("mix.f.b"):   # forget gates near one: far tokens stay in the matrix memories
                self.W[k] = (self.W[k].float() + keep).to(torch.bfloat16)
        self._oracle = {}

    def engine(self, device, dtype="float32", blocks=64, seqs=4, **kw):
        model = fp.FurapelLM(self.mc, device, dtype=getattr(torch, dtype), max_positions=1024).load_tensors(self.W)
        return LLMEngine(EngineConfig(model="test", device=device, num_kv_blocks=blocks, max_num_seqs=seqs,
                                      max_model_len=1024, dtype=dtype, **kw), model_cfg=self.mc, model=model)

    def oracle(self, tokens):
        key = tuple(tokens)
        if key not in self._oracle:
            self._oracle[key] = plain.forward(self.cfg, self.W, list(tokens)).float()
        return self._oracle[key]


def toks(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def row_errs(got, want):
    """Per row: rms of the mean-free difference over the rms of the mean-free expectation."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt()


def rel_err(got, want):
    return row_errs(got, want).max().item()


def mean_err(got, want):
    return row_errs(got, want).mean().item()


TOL = {"float32": 2e-4, "bfloat16": 0.08}


def feed_all(eng, rid, tokens, cuts):
    """Feed ``tokens`` in portions of the given sizes (the last size repeats), all positions wanted."""
    rows, at, i = [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - at)
        last = at + n == len(tokens)
        rows.append(eng.feed([(rid, tokens[at:at + n], list(range(n)))], [rid] if last else []))
        at += n
        i += 1
    return torch.cat(rows)


def poison_state(eng):
    """NaN in every state slot: a sequence's first portion must not read its slot."""
    for st in eng.runner.v_caches.layers:
        for t in st.values():
            t.fill_(float("nan"))


@pytest.fixture(scope="module")
def bench_a():
    return Bench(cfg_a())


@pytest.fixture(scope="module")
def bench_sharp():
    return Bench(cfg_a(scale=0.9), seed=3, keep=3.0)


def close(got, want, tol):
    return (got.double().cpu() - want.double()).abs().max().item() < tol * want.abs().max().item()


def seg_tensors(device, runs):
    """runs: (first row, rows, first position, slot) -> (tok_seg, seg)"""
    ts = [j for j, r in enumerate(runs) for _ in range(r[1])]
    return (torch.tensor(ts, dtype=torch.int32, device=device), torch.tensor(runs, dtype=torch.int32, device=device))


# ---- mechanisms alone ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d,T", [(1, 3), (70, 5), (88, 1), (1030, 3), (2048, 40), (4500, 2)])
def test_add_tanh_norm(device, d, T):
    """The residual's sum and what is read from it: y1 plain, in bf16, as split-K slabs, with and without y2, assigned
    instead of added, one and two norms, a copy into a column slice; arguments of the tanh from 1e-6 to far beyond
    saturation."""
    g = torch.Generator().manual_seed(d)
    x0, y1, y2 = (torch.randn(T, d, generator=g) for _ in range(3))
    x0 *= 10.0 ** torch.empty(T, d).uniform_(-6.0, 1.7, generator=g)
    slabs = torch.randn(5, T, d, generator=g)
    W = {f"n{k}{s}": t for k in (0, 1) for s, t in (("", 1.0 + 0.3 * torch.randn(d, generator=g)),
                                                    (".b", torch.randn(d, generator=g)),
                                                    (".alpha", torch.tensor([0.63, 1.9][k])))}
    W64 = {k: v.double() for k, v in W.items()}
    dv = lambda t: t.to(device)  # noqa: E731
    norms = [hops.TanhNorm(float(W[f"n{k}.alpha"]), dv(W[f"n{k}"]), dv(W[f"n{k}.b"])) for k in (0, 1)]
    for a, b, assign, n in ((None, None, False, 1), (y1, None, False, 2), (y1, y2, False, 2), (slabs, None, True, 2),
                            (slabs, y2, False, 0), (y1, None, True, 1)):
        y = 0.0 if a is None else a.double().sum(0) if a.dim() == 3 else a.double()
        y = y + (b.double() if b is not None else 0.0)
        want = y if assign else x0.double() + y
        for dt in (torch.float32, torch.bfloat16):
            for low in (False, True):
                if low and (a is None or a.dim() == 3 or dt == torch.float32):
                    continue
                ya = a.to(dt) if low else a
                wx = want if not low else want - y + a.to(dt).double() + (b.double() if b is not None else 0.0)
                x = dv(x0.clone())
                wide = torch.zeros(T, 2 * d + 3, dtype=dt, device=device)
                outs = [torch.empty(T, d, dtype=dt, device=device) for _ in range(n)]
                hops.add_tanh_norm(x, None if ya is None else dv(ya), None if b is None else dv(b), norms[:n], outs,
                                   wide[:, 2:2 + d], assign)
                assert (x.cpu().double() - wx).abs().max() < 1e-5 * max(1.0, float(wx.abs().max()))
                assert torch.equal(wide[:, 2:2 + d], x.to(dt)) and float(wide[:, 2 + d:].float().abs().sum()) == 0.0
                for k in range(n):
                    e = (outs[k].cpu().double() - plain.tanh_norm(x.cpu().double(), W64, f"n{k}")).abs().max()
                    assert e < (1e-6 if dt == torch.float32 else 2e-2), (k, dt)
    # small arguments keep their relative accuracy
    x = dv(x0.clone() * 1e-3)
    out = torch.empty(T, d, device=device)
    zero = hops.TanhNorm(0.63, dv(torch.ones(d)), dv(torch.zeros(d)))
    hops.add_tanh_norm(x, norms=[zero], outs=[out])
    want = torch.tanh(0.63 * x.cpu().double())
    assert ((out.cpu().double() - want).abs() <= 1e-6 * want.abs() + 1e-12).all()
    with pytest.raises((ValueError, RuntimeError)):
        hops.add_tanh_norm(x, assign=True)
    # a token's expert rows, gathered
    for dt, k in ((torch.float32, 3), (torch.bfloat16, 6)):
        inv = torch.randperm(T * k, generator=g).int().view(T, k)
        rows = torch.randn(T * k, d, generator=g).to(dt)
        x, out = dv(x0.clone()), torch.empty(T, d, dtype=dt, device=device)
        hops.add_tanh_norm(x, dv(y1.to(dt)), hops.ExpertRows(dv(rows), dv(inv)), norms[:1], [out])
        want = x0.double() + y1.to(dt).double() + rows.double()[inv.long()].sum(1)
        assert (x.cpu().double() - want).abs().max() < 1e-5 * max(1.0, float(want.abs().max()))
        e = (out.cpu().double() - plain.tanh_norm(x.cpu().double(), W64, "n0")).abs().max()
        assert e < (1e-6 if dt == torch.float32 else 2e-2)


@pytest.mark.parametrize("rot", [YARN, {"base": 10000.0, "dims": 24}, dict(YARN, dims=24),
                                 {"base": 500.0, "dims": 16, "scaling": {"factor": 8.0, "original": 40, "fast": 32.0,
                                                                         "slow": 1.0}},
                                 {"base": 1e6, "dims": 24, "scaling": {"factor": 1.5, "original": 1e6, "fast": 2.0,
                                                                       "slow": 1.9}},
                                 {"base": 20.0, "dims": 2, "scaling": {"factor": 4.0, "original": 7, "fast": 3.0,
                                                                       "slow": 0.01}}])
def test_rotation_table(rot):
    """The engine's table against the plain rotation: blended frequencies with ramps that start below the first pair, end
    behind the last, or have no width; the factor on cos and sin."""
    tab = rotary_table(300, rot, "cpu").double()
    half = rot["dims"] // 2
    x = torch.zeros(300, 1, rot["dims"], dtype=torch.float64)
    x[..., :half] = 1.0
    y = plain.rotate_halves(x, rot)[:, 0]
    assert (torch.cat([y[:, :half], y[:, half:]], 1) - tab).abs().max() < 5e-5
    assert torch.equal(plain.rotate_halves(x[:5], rot, 7), plain.rotate_halves(x, rot)[7:12])


class Paged:
    """Scattered pages for sequences of given lengths, fed in given portions: the step tensors the kernels take."""

    def __init__(self, device, lengths, seed=0):
        self.device = device
        self.n_pages = sum(-(-n // 16) for n in lengths) + 3
        perm = torch.randperm(self.n_pages, generator=torch.Generator().manual_seed(seed)).tolist()
        self.tables, at = [], 0
        for n in lengths:
            k = -(-n // 16)
            self.tables.append(perm[at:at + k])
            at += k

    def step(self, runs):
        """runs: (sequence, first position, rows) -> block tables, tok_seg, positions, slot mapping"""
        W = max(len(t) for t in self.tables)
        bt = torch.zeros(len(runs), W, dtype=torch.int32)
        ts, pos, sl = [], [], []
        for j, (s, p0, n) in enumerate(runs):
            bt[j, :len(self.tables[s])] = torch.tensor(self.tables[s], dtype=torch.int32)
            for p in range(p0, p0 + n):
                ts.append(j)
                pos.append(p)
                sl.append(self.tables[s][p // 16] * 16 + p % 16)
        d = self.device
        return (bt.to(d), torch.tensor(ts, dtype=torch.int32, device=d), torch.tensor(pos, dtype=torch.long, device=d),
                torch.tensor(sl, dtype=torch.long, device=d))


def _attn_case(g, n, H, G, D, Dv, rot, spots, gain=2.0):
    """Rows [q | k | v | gates] of a sequence with (row, key) pairs whose score stands out in the dimensions that do not
    turn (a full rotation: in all of them), and the plain result (the projections are selections of the row's columns)."""
    C = H * D + G * D + G * Dv + H
    h = torch.randn(n, C, generator=g)
    for i, (at, key) in enumerate(spots):
        hd = i % H
        c = H * D + (hd // (H // G)) * D
        lo = rot["dims"] if rot and rot["dims"] < D else 0
        h[at, hd * D + lo:(hd + 1) * D] = gain * h[key, c + lo:c + D]
    eye = torch.eye(C, dtype=torch.float64)
    o = (0, H * D, H * D + G * D, H * D + G * D + G * Dv, C)
    W = {k: eye[o[i]:o[i + 1]] for i, k in enumerate(("q", "k", "v", "g"))}
    return h, W


SPOTS = [(329, 0), (329, 329), (140, 127), (140, 128), (100, 15), (100, 16), (297, 1), (297, 2), (298, 40), (5, 0),
         (1, 1), (328, 31)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,rot", [(6, 2, 24, 20, YARN), (4, 4, 8, 70, None), (3, 1, 100, 9, dict(YARN, dims=100)),
                                          (1, 1, 8, 8, dict(YARN, dims=8)), (8, 2, 16, 130, dict(YARN, dims=6))])
def test_head_gated_attention_single_keys(device, H, G, D, Dv, rot):
    """Blended rotation (part of a head), softmax over every earlier key, a gate per head, through scattered pages, in
    portions, two sequences side by side. Loud keys sit at the first positions, on both sides of page borders, at the
    row's own position and hundreds of tokens back, for rows of a portion and for rows fed alone."""
    g = torch.Generator().manual_seed(H * 100 + D)
    n0, n1 = 330, 23
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": 4.0 * D ** -0.5}
    if rot:
        m["rot"] = rot
    cases = [_attn_case(g, n0, H, G, D, Dv, rot, SPOTS), _attn_case(g, n1, H, G, D, Dv, rot, [(22, 0), (20, 16)])]
    W = cases[0][1]
    want = [plain.attention_heads(h.double(), W, "", m).reshape(h.shape[0], -1) for h, _ in cases]
    pg = Paged(device, [n0, n1], seed=H)
    kc = torch.zeros(pg.n_pages, 16, G * D, device=device)
    vt = torch.zeros(pg.n_pages, G * Dv, 16, device=device)
    cs = rotary_table(512, rot, device) if rot else None
    dims = rot["dims"] if rot else 0
    got, at = [torch.empty(n0, H * Dv), torch.empty(n1, H * Dv)], [0, 0]
    for portions in ([(0, 97), (1, 2)], [(1, 20), (0, 1)], [(0, 2)], [(0, 197), (1, 1)], [(0, 1)], [(0, 1)], [(0, 31)]):
        runs = [(s, at[s], n) for s, n in portions]
        bt, ts, pos, sl = pg.step(runs)
        rows = torch.cat([cases[s][0][a:a + n] for s, a, n in runs]).to(device)
        q = torch.empty(rows.shape[0], H * D, device=device)
        hops.rope_kv_store(rows, H, G, D, Dv, pos, cs, dims, False, None, kc, vt, sl, q)
        out = torch.empty(rows.shape[0], H * Dv, device=device)
        hops.window_attn(q, kc, vt, bt, ts, pos, H, G, m["scale"], 0, None, out, gate=rows,
                         gate_off=H * D + G * D + G * Dv)
        r = 0
        for s, a, n in runs:
            got[s][a:a + n] = out[r:r + n].cpu()
            r += n
            at[s] += n
    assert at == [n0, n1]
    for s in (0, 1):
        assert close(got[s], want[s], 2e-4), s


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,Dv,rot,n", [(8, 2, 32, 48, 16, 300), (4, 4, 64, 20, 0, 700), (32, 1, 48, 96, 24, 200),
                                            (16, 2, 128, 128, 64, 1500), (2, 1, 256, 256, 128, 520)])
def test_head_gated_attention_matrix_cores(H, G, D, Dv, rot, n):
    """The bf16 attention inputs and the matrix-core attention with head gates against the plain function: prompt
    portions and decode rows, whole key ranges and split ones (the merge pass applies the gates there)."""
    dev = "cuda:0"
    g = torch.Generator().manual_seed(H * D + n)
    rot = {"base": 3000.0, "dims": rot, "scaling": {"factor": 4.0, "original": 128, "fast": 16.0, "slow": 1.0}} \
        if rot else None
    spots = [(n - 1, 0), (n - 1, n - 1), (140, 127), (140, 128), (100, 15), (n - 2, 1), (n - 1, n - 41), (n - 40, 3)]
    h, W = _attn_case(g, n, H, G, D, Dv, rot, spots, 1.0)
    hb = h.to(torch.bfloat16)
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": Dv, "scale": 2.0 * D ** -0.5, "rot": rot}
    want = plain.attention_heads(hb.double(), W, "", m).reshape(n, -1)
    pg = Paged(dev, [n], seed=5)
    kc = torch.zeros(pg.n_pages, 16, G * D, dtype=torch.bfloat16, device=dev)
    vt = torch.zeros(pg.n_pages, G * Dv, 16, dtype=torch.bfloat16, device=dev)
    cs = rotary_table(2048, rot, dev) if rot else None
    tt = hops.sig_tile_tokens(H, G)
    got, at = torch.empty(n, H * Dv), 0
    for rows in (n - 40, 1, 38, 1):
        bt, ts, pos, sl = pg.step([(0, at, rows)])
        src = hb[at:at + rows].to(dev)
        q = torch.empty(rows, H * D, dtype=torch.bfloat16, device=dev)
        hops.rope_kv_store(src, H, G, D, Dv, pos, cs, rot["dims"] if rot else 0, False, None, kc, vt, sl, q)
        tiles = torch.tensor([(a, min(tt, rows - a), 0, 0) for a in range(0, rows, tt)], dtype=torch.int32, device=dev)
        assert hops.window_attn_mfma_ok(q, kc, vt, H, G)
        outs = []
        # vector kernel; unsplit; split key ranges; a wave per tile
        for t, max_keys, kinds in ((None, 0, (True, False)), (tiles, 0, (True, False)), (tiles, at + rows, (True, False)),
                                   (tiles, at + rows, (rows % tt == 1, True))):
            out = torch.zeros(rows, H * Dv, dtype=torch.bfloat16, device=dev)
            hops.window_attn(q, kc, vt, bt, ts, pos, H, G, m["scale"], 0, None, out, t, max_keys, gate=src,
                             gate_off=H * D + G * D + G * Dv, kinds=kinds)
            outs.append(out.float().cpu())
        for o in outs[1:]:
            assert (o - outs[0]).abs().max() < 0.03 * want.abs().max()
        got[at:at + rows] = outs[2]
        at += rows
    assert at == n
    assert (got.double() - want).abs().max() < 0.05 * want.abs().max()


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,Dv,window,shared,lengths", [
    (8, 2, 32, 48, 0, False, (300, 70)), (4, 4, 64, 20, 129, False, (700, 5)), (32, 1, 48, 96, 0, False, (90, 33)),
    (16, 2, 128, 128, 0, False, (900, 41)), (6, 3, 96, 96, 1, False, (150, 150)), (8, 2, 128, 256, 200, False, (500, 65)),
    (2, 1, 256, 256, 0, False, (300, 1)), (12, 4, 80, 130, 33, False, (260, 97)), (6, 3, 48, 40, 0, True, (200, 47)),
    (20, 1, 64, 64, 50, False, (120, 1))])
def test_attention_of_prompt_portions(H, G, D, Dv, window, shared, lengths):
    """The wave-per-item attention (bf16) against the vector kernel and a direct softmax: two sequences side by side in
    unequal portions and single tokens, whole tiles and ends of tiles, windows whose edges fall inside blocks, a sink,
    head gates, an output scale, whole key rows, loud keys on the windows' edges and one outside."""
    from kafka_llm_service_amd.models.budurax import SegMeta

    dev = "cuda:0"
    g = torch.Generator().manual_seed(H * D + Dv)
    Dq = G * D if shared else D
    tt, w = hops.sig_tile_tokens(H, G), window or 10 ** 6
    data = []
    for n in lengths:
        q, k = 0.5 * torch.randn(n, H, Dq, generator=g), torch.randn(n, G, D, generator=g)
        v, gate = torch.randn(n, G, Dv, generator=g), torch.randn(n, H + 3, generator=g)
        for i, (at, key) in enumerate([(n - 1, 0), (n - 1, n - 1), (n - 1, max(0, n - w)), (n - 1, max(0, n - 1 - w)),
                                       (n // 2, max(0, n // 2 - w + 1)), (n // 2 + 1, max(0, n // 2 + 1 - w)),
                                       (n // 2, n // 3), (min(33, n - 1), min(32, n - 1))]):
            h, at = i % H, min(at, n - 1)
            if shared:
                q[at, h] = 1.5 * k[min(key, at)].reshape(-1) / G ** 0.5
            else:
                q[at, h] = 1.5 * k[min(key, at), h // (H // G)]
        data.append([x.to(torch.bfloat16) for x in (q, k, v, gate)])
    sink, scale = torch.randn(H, generator=g), 1.5 * Dq ** -0.5
    want = []
    for q, k, v, gate in data:
        n = q.shape[0]
        kk = k.double().reshape(n, 1, -1).expand(n, H, -1) if shared else k.double().repeat_interleave(H // G, 1)
        s = torch.einsum("ihd,jhd->hij", q.double(), kk) * scale
        ok = plain.visible(n, window or None)
        s = torch.cat([s.masked_fill(~ok, float("-inf")), sink.double().view(H, 1, 1).expand(H, n, 1)], 2)
        o = torch.einsum("hij,jhv->ihv", torch.softmax(s, -1)[:, :, :n], v.double().repeat_interleave(H // G, 1))
        want.append((0.6 * o * torch.sigmoid(gate[:, 2:2 + H].double())[:, :, None]).reshape(n, -1))
    pg = Paged(dev, lengths, seed=3)
    kc = torch.zeros(pg.n_pages, 16, G * D, dtype=torch.bfloat16, device=dev)
    vt = torch.zeros(pg.n_pages, G * Dv, 16, dtype=torch.bfloat16, device=dev)
    at, got, seen = [0, 0], [[], []], set()
    cuts = ((1, 2), (tt + 1, 3), (10 ** 6, 1), (0, 10 ** 6))
    for step, (a, b) in enumerate(cuts):
        left = [lengths[0] - at[0], lengths[1] - at[1]]
        take = [min(a, max(0, left[0] - (0 if step >= 2 else 2))), min(b, left[1])]
        runs = [(s, at[s], take[s]) for s in (0, 1) if take[s]]
        if not runs:
            continue
        bt, ts, pos, sl = pg.step(runs)
        rows = [torch.cat([data[s][x][p:p + m] for s, p, m in runs]).to(dev) for x in range(4)]
        T = rows[0].shape[0]
        hops.kv_store(torch.cat([rows[1].reshape(T, -1), rows[2].reshape(T, -1)], 1), 0, G * D, kc, vt, sl)
        q0, segs, tiles = 0, [], []
        for j, (s, p, m) in enumerate(runs):
            segs.append((q0, m, p, 0))
            tiles += [(q0 + x, min(tt, m - x), j, 0) for x in range(0, m, tt)]
            q0 += m
        seg = torch.tensor(segs, dtype=torch.int32, device=dev)
        kinds = SegMeta(T, len(runs), seg, ts, bt, seg_host=np.asarray(segs)).tile_kinds(tt)
        seen.add(kinds)
        qq = rows[0].reshape(T, -1).contiguous()
        assert hops.window_attn_mfma_ok(qq, kc, vt, H, G, shared)
        tl, outs = torch.tensor(tiles, dtype=torch.int32, device=dev), []
        for t, kd in ((None, (True, False)), (tl, kinds)):
            wide = torch.zeros(T, H * Dv + 6, dtype=torch.bfloat16, device=dev)
            hops.window_attn(qq, kc, vt, bt, ts, pos, H, G, scale, window, sink.to(dev), wide[:, :H * Dv], t,
                             max(p + m for _, p, m in runs), shared, 0.6, rows[3], 2, kd)
            assert float(wide[:, H * Dv:].abs().max()) == 0.0
            outs.append(wide[:, :H * Dv].float().cpu())
        assert (outs[0] - outs[1]).abs().max() < 0.02 * max(x.abs().max() for x in want), kinds
        q0 = 0
        for s, p, m in runs:
            got[s].append(outs[1][q0:q0 + m])
            at[s] += m
            q0 += m
    assert tuple(at) == tuple(lengths) and any(k[1] for k in seen)
    for s in (0, 1):
        assert (torch.cat(got[s]).double() - want[s]).abs().max() < 0.03 * want[s].abs().max(), s


def _latent_case(g, n, H, D, Dv, R, spots):
    """Rows [q | latent] with loud (row, key) pairs, random up-projections; the engine's result is W_uv of its latent
    output, compared before the output projection."""
    W = {"uk": torch.randn(H * D, R, generator=g).double() / R ** 0.5, "uv": torch.randn(H * Dv, R, generator=g).double(),
         "dkv.norm": 1.0 + 0.2 * torch.randn(R, generator=g).double(), "o": torch.eye(H * Dv).double()}
    h = torch.randn(n, H * D + R, generator=g)
    c = plain.rms_unit(h[:, H * D:].double(), 1e-3) * W["dkv.norm"]
    k = (c @ W["uk"].T).view(n, H, D)
    for i, (at, key) in enumerate(spots):
        hd = i % H
        kv = k[key, hd]
        h[at, hd * D:(hd + 1) * D] = (9.0 * kv / (kv * kv).sum()).float() * D ** 0.5
    eye = torch.eye(H * D + R).double()
    W["q"], W["dkv"] = eye[:H * D], eye[H * D:]
    return h, W


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dv,R,window", [(5, 12, 10, 40, 10), (3, 8, 9, 33, 37), (1, 4, 6, 16, 1),
                                             (9, 20, 4, 200, 0), (2, 6, 8, 600, 129)])
def test_latent_attention_single_keys(device, H, D, Dv, R, window):
    """The latent row's norm and store, the windowed softmax in the latent space and both up-projections through
    scattered pages in portions. Loud keys: the first position, both sides of page borders, the row's own position, the
    window's last visible position and the one before it (for rows of a portion and for a row fed alone), far behind
    the window."""
    g = torch.Generator().manual_seed(H + R)
    n, eps = 150, 1e-3
    w = window or 10 ** 6
    spots = [(149, 0), (149, 149), (140, 127), (140, 128), (100, 15), (100, 16), (120, max(0, 120 - w + 1)),
             (121, max(0, 121 - w)), (149, 3), (97, max(0, 97 - w + 1)), (98, max(0, 98 - w)), (1, 0), (2, 0)]
    h, W = _latent_case(g, n, H, D, Dv, R, spots)
    m = {"heads": H, "dim": D, "vdim": Dv, "kv_rank": R, "scale": D ** -0.5}
    if window:
        m["mask"] = {"size": window}
    want = plain.latent_attention(h.double(), W, "", m, eps)
    pg = Paged(device, [n], seed=H)
    cache = torch.zeros(pg.n_pages, 16, R, device=device)
    uk = W["uk"].float().view(H, D, R).to(device)
    uv = W["uv"].float().view(H, Dv, R).transpose(1, 2).contiguous().to(device)
    got, at = [], 0
    for rows in (97, 1, 1, 2, 31, 18):
        bt, ts, pos, sl = pg.step([(0, at, rows)])
        src = h[at:at + rows].to(device)
        seg = torch.tensor([(0, rows, at, 0)], dtype=torch.int32, device=device)
        q_rot = torch.empty(rows, H, 0, device=device)
        hops.latent_prep(src, H, D, 0, R, H * D, W["dkv.norm"].float().to(device), eps, pos, None, 0, cache, sl, q_rot)
        ql = torch.bmm(src[:, :H * D].reshape(rows, H, D).transpose(0, 1), uk)
        ol = torch.empty(H, rows, R, device=device)
        hops.latent_attn(ql, q_rot, cache, bt, ts, seg, pos, m["scale"], ol, window=window)
        got.append(torch.bmm(ol, uv).transpose(0, 1).reshape(rows, -1).cpu())
        at += rows
    assert at == n
    assert close(torch.cat(got), want, 2e-4)


MLSTM_SIZES = [(3, 10, 14), (1, 1, 1), (2, 48, 65), (4, 64, 64), (2, 128, 130), (1, 256, 24), (2, 16, 256), (3, 112, 40)]
MLSTM_PORTIONS = [[(0, 9), (1, 2)], [(1, 1), (0, 1)], [(0, 2), (1, 3)], [(1, 7)], [(0, 130), (1, 65)], [(0, 1)],
                  [(1, 201), (0, 3)], [(0, 129), (1, 128)]]


def _mlstm_case(g, n, H, D, Dv, cap, slow):
    """Raw rows q | k | v and raw gates of a sequence. ``slow``: forget gates near one and a loud early token that late
    queries ask for; else forget gates around a half with a run that forgets nearly everything, input gates over the
    whole capped range."""
    qkv = torch.randn(n, H * (2 * D + Dv), generator=g)
    gates = torch.randn(n, 2 * H, generator=g)
    if slow:
        gates[:, H:] += 8.0
        qkv[3, 2 * H * D:] *= 30.0
        qkv[n - 12:, :H * D] = 3.0 * qkv[3, H * D:2 * H * D]
        gates[3, :H] = cap
    else:
        gates[:, :H] *= 3.0 * cap / 2.0
        gates[50:60, H:] = -3.0 * cap
        gates[100:140, :H] -= 2.0 * cap
    return qkv, gates


def _mlstm_want(qkv, gates, H, D, Dv, cap):
    n = qkv.shape[0]
    q, k, v = qkv.double().split([H * D, H * D, H * Dv], 1)
    ig, fg = plain.log_gates(gates[:, :H].double(), gates[:, H:].double(), cap)
    return plain.mlstm_scan(q.reshape(n, H, D) * D ** -0.5, k.reshape(n, H, D), v.reshape(n, H, Dv), ig, fg).reshape(n, -1)


def _chunks(device, segs):
    tabs = hops.chunk_tables(np.asarray(segs, dtype=np.int32), hops.MLSTM_CHUNK, hops.MLSTM_CHUNK_MIN)
    return None if tabs is None or device == "cpu" else tuple(torch.from_numpy(x).to(device) for x in tabs)


def _head_errs(o, want, H, Dv):
    """Per (row, head) against its own size (a read-out is divided by |n . q|, which may be small)."""
    return (o - want).view(-1, H, Dv).abs().amax(-1) / (want.view(-1, H, Dv).abs().amax(-1) + 1e-3)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,Dv", MLSTM_SIZES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_mlstm_scan(device, H, D, Dv, dtype):
    """The matrix memory through portions of 1, 2, 3, 7, 9 rows and long ones (in chunks on the GPU where the sizes
    allow) of two sequences from NaN slots: far tokens that stay, tokens that are forgotten at once, gates at their
    caps."""
    g = torch.Generator().manual_seed(H * 100 + D)
    cap, lengths = 6.0, [275, 407]
    cases = [_mlstm_case(g, n, H, D, Dv, cap, s == 0) for s, n in enumerate(lengths)]
    cases = [(q.to(dtype), z) for q, z in cases]
    want = [_mlstm_want(q, z, H, D, Dv, cap) for q, z in cases]
    S = torch.full((3, H, D, Dv), float("nan"), device=device)
    nrm, mx = torch.full((3, H, D), float("nan"), device=device), torch.full((3, H), float("nan"), device=device)
    at, got = [0, 0], [[], []]
    for portions in MLSTM_PORTIONS:
        runs, r0 = [], 0
        for s, n in portions:
            n = min(n, lengths[s] - at[s])
            runs.append((s, at[s], n, r0))
            r0 += n
        segs = [(q0, n, p0, 2 - s) for s, p0, n, q0 in runs]              # slots 2 and 1 of 3
        ts, seg = seg_tensors(device, segs)
        rows = torch.cat([cases[s][0][p0:p0 + n] for s, p0, n, _ in runs]).to(device)
        gates = torch.cat([cases[s][1][p0:p0 + n] for s, p0, n, _ in runs]).to(device)
        out = torch.full((r0, H * Dv), float("nan"), device=device)
        hops.mlstm_scan(rows, gates, H, D, Dv, cap, ts, seg, S, nrm, mx, out, _chunks(device, segs))
        for s, p0, n, q0 in runs:
            got[s].append(out[q0:q0 + n].cpu())
            at[s] += n
    assert at == lengths
    for s in (0, 1):
        e = _head_errs(torch.cat(got[s]).double(), want[s], H, Dv)
        assert e.median() < 1e-5 and (e < 5e-3).all() and (e < 2e-4).double().mean() > 0.99, s
    assert not torch.isnan(S[1:]).any() and torch.isnan(S[0]).all()


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,Dv", [(3, 48, 72), (2, 16, 8), (2, 128, 256), (1, 256, 64), (4, 144, 40), (9, 64, 128)])
def test_mlstm_in_chunks(H, D, Dv):
    """The chunked form against the token-by-token kernel and the plain function: every kind of last chunk, segments that
    continue from a state beside fresh ones, heads inside wider rows, the state it leaves and what single tokens make of
    it."""
    dev = "cuda:0"
    assert hops.ext().hy_mlstm_chunk() == hops.MLSTM_CHUNK
    g = torch.Generator().manual_seed(D)
    cap, lengths = 9.0, [21 + 48 + 2, 150 + 257 + 3, 128 + 129 + 1]
    cases = []
    for s, n in enumerate(lengths):
        qkv, gates = _mlstm_case(g, n, H, D, Dv, cap, s == 1)
        cases.append((torch.cat([qkv, torch.randn(n, 8, generator=g)], 1).to(torch.bfloat16), gates))
    want = [_mlstm_want(q[:, :-8], z, H, D, Dv, cap) for q, z in cases]
    steps = [[(0, 21), (1, 150)], [(2, 128), (1, 257), (0, 48)], [(0, 1), (2, 129)], [(1, 1), (0, 1), (2, 1)],
             [(1, 2)]]
    res = []
    for chunked in (False, True):
        S = torch.full((4, H, D, Dv), float("nan"), device=dev)
        nrm, mx = torch.full((4, H, D), float("nan"), device=dev), torch.full((4, H), float("nan"), device=dev)
        at, got = [0, 0, 0], [[], [], []]
        for st in steps:
            segs, r0 = [], 0
            for s, n in st:
                segs.append((r0, n, at[s], 3 - s))
                r0 += n
            rows = torch.cat([cases[s][0][at[s]:at[s] + n] for s, n in st]).to(dev)
            gates = torch.cat([cases[s][1][at[s]:at[s] + n] for s, n in st]).to(dev)
            ts, seg = seg_tensors(dev, segs)
            out = torch.full((r0, H * Dv), float("nan"), device=dev)
            assert hops.mlstm_chunk_ok(H, D, Dv, rows)
            hops.mlstm_scan(rows, gates, H, D, Dv, cap, ts, seg, S, nrm, mx, out, _chunks(dev, segs) if chunked else None)
            r0 = 0
            for s, n in st:
                got[s].append(out[r0:r0 + n].cpu())
                at[s] += n
                r0 += n
        assert at == lengths
        res.append([torch.cat(x).double() for x in got] + [S[1:].cpu(), nrm[1:].cpu(), mx[1:].cpu()])
        for s in range(3):
            e = _head_errs(res[-1][s], want[s], H, Dv)
            assert e.median() < 1e-5 and (e < 5e-3).all() and (e < 2e-4).double().mean() > 0.99, (chunked, s)
        assert torch.isnan(S[0]).all()
    for a, b in zip(res[0][3:], res[1][3:]):
        assert close(b, a, 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,k,d,ff", [(7, 3, 40, 24), (1, 1, 16, 8), (70, 8, 33, 10), (6, 6, 64, 130)])
def test_router_and_experts(device, E, k, d, ff):
    """Softmax over all experts, the largest chosen, weights as they are (they do not sum to one); squared-relu experts
    without a gate."""
    g = torch.Generator().manual_seed(E)
    T = 37
    h, w = torch.randn(T, d, generator=g), torch.randn(E, d, generator=g) / 4
    up, down = torch.randn(E, ff, d, generator=g) / d ** 0.5, torch.randn(E, d, ff, generator=g) / ff ** 0.5
    W = {"router": w.double()}
    for e in range(E):
        W[f"e{e}.up"], W[f"e{e}.down"] = up[e].double(), down[e].double()
    want = plain.experts(h.double(), W, "", {"router": {"top": k}})
    tw, te, _ = hops.moe_router_grouped(h.to(device), w.to(device), None, k, 1, 1, norm=False)
    dense = torch.zeros(T, E, dtype=torch.float64).scatter_(1, te.long().cpu(), tw.double().cpu())
    assert close(dense, plain.route(h.double() @ w.double().T, k), 1e-5)
    out = torch.empty(T, d, device=device)
    hops.moe_experts(h.to(device), up.to(device), down.to(device), tw, te, out, act="relu2")
    assert close(out, want, 1e-4)


@pytest.mark.gpu
@pytest.mark.parametrize("E,k,T", [(6, 3, 1), (6, 3, 5), (16, 4, 64), (40, 8, 130), (16, 4, 300), (5, 2, 700), (3, 1, 2000)])
def test_experts_on_the_matrix_cores(E, k, T):
    """The squared-relu experts in bf16: expert-sorted GEMMs and, on tiled weights, the grouped streaming kernel (both
    epilogues) against the per-pair kernels and the plain function; experts without a row, experts with most rows."""
    dev = "cuda:0"
    g = torch.Generator().manual_seed(T)
    d, ff = 256, 256
    from kafka_llm_service_amd import ops

    h = torch.randn(T, d, generator=g).to(torch.bfloat16)
    w = torch.randn(E, d, generator=g) / 8
    w[1] = -1.0 + 0.01 * w[1]
    h[:, :8] = h[:, :8].abs()
    up = (torch.randn(E, ff, d, generator=g) / d ** 0.5).to(torch.bfloat16)
    down = (torch.randn(E, d, ff, generator=g) / ff ** 0.5).to(torch.bfloat16)
    W = {"router": w.double()}
    for e in range(E):
        W[f"e{e}.up"], W[f"e{e}.down"] = up[e].double(), down[e].double()
    want = plain.experts(h.double(), W, "", {"router": {"top": k}})
    tw, te, _ = hops.moe_router_grouped(h.to(dev), w.to(dev), None, k, 1, 1, norm=False)
    hd, ud, dd = h.to(dev), up.to(dev), down.to(dev)
    assert hops.moe_grouped_ok(hd, ud, dd, glu=False) and ops.stream_moe_supported(ff, d)
    res = []
    for tiled in (False, True):
        out = torch.empty(T, d, device=dev)
        hops.moe_experts(hd, ud, dd, tw, te, out, ops.tile_experts(ud) if tiled else None,
                         ops.tile_experts(dd) if tiled else None, act="relu2")
        res.append(out)
    out = torch.empty(T, d, device=dev)
    hops.moe_rows(hd, ud, dd, tw, te, out, act="relu2")
    for r in res + [out]:
        assert close(r, want, 0.02)


@pytest.mark.gpu
@pytest.mark.parametrize("n_exp,k,T", [(1, 1, 3), (3, 2, 5), (16, 4, 64), (16, 4, 2048), (70, 8, 333), (512, 16, 700),
                                       (8, 2, 8192)])
def test_sort_by_expert(n_exp, k, T):
    """Entries by expert, in token order inside an expert; experts without entries, stretches that end inside a wave."""
    from kafka_llm_service_amd import ops

    g = torch.Generator().manual_seed(T)
    te = torch.stack([torch.randperm(n_exp, generator=g)[:k] for _ in range(T)]).int()
    if n_exp > 8:
        te[:, 0] = torch.where(te[:, 0] == 5, (te[:, 1] + 1) % n_exp, te[:, 0])
        te[T // 2:, 1] = 7
    tw = torch.rand(T, k, generator=g)
    a, b = ops.moe_sort(tw.cuda(), te.cuda(), n_exp, inverse=True), ops.moe_sort(tw, te, n_exp, inverse=True)
    for n in ("perm_tok", "perm_w", "expert_off", "tile_off", "inv"):
        assert torch.equal(getattr(a, n).cpu(), getattr(b, n)), n


@pytest.mark.gpu
@pytest.mark.parametrize("E,k,T,d,ff", [(6, 3, 700, 256, 256), (3, 1, 130, 512, 320), (70, 8, 900, 128, 64),
                                        (2, 2, 1000, 384, 576)])
def test_wide_expert_products(E, k, T, d, ff):
    """The kernels for long steps on tiled weights, every epilogue against the CPU functions: row tiles that end inside an
    expert, experts without rows, column tiles that end inside a workgroup."""
    from kafka_llm_service_amd import ops

    g = torch.Generator().manual_seed(E)
    te = torch.stack([torch.randperm(E, generator=g)[:k] for _ in range(T)]).int()
    if E > 4:
        te[te == 2] = 3
    tw = torch.rand(T, k, generator=g)
    h = torch.randn(T, d, generator=g).to(torch.bfloat16)
    gu = (torch.randn(E, 2 * ff, d, generator=g) / d ** 0.5).to(torch.bfloat16)
    down = (torch.randn(E, 128, 2 * ff, generator=g) / ff ** 0.5).to(torch.bfloat16)
    r, rc = ops.moe_sort(tw.cuda(), te.cuda(), E), ops.moe_sort(tw, te, E)
    gd, dd = gu.cuda(), down.cuda()
    for kw in ({}, {"limit": 1.5, "alpha": 1.7}):
        a = ops.grouped_wide(h.cuda(), ops.tile_experts(gd, glu=True), r, "glu", True, **kw)
        assert close(a.float(), ops.grouped_wide(h, ops.tile_experts(gu, glu=True), rc, "glu", True, **kw).float(), 1e-2)
    a = ops.grouped_wide(h.cuda(), ops.tile_experts(gd), r, "relu2", True)
    ac = ops.grouped_wide(h, ops.tile_experts(gu), rc, "relu2", True)
    assert close(a.float(), ac.float(), 1e-2)
    if 2 * ff % 128 == 0:
        out, oc = torch.zeros(T, 128, device="cuda"), torch.zeros(T, 128)
        ops.grouped_wide(a, ops.tile_experts(dd), r, "combine", False, out)
        ops.grouped_wide(a.cpu(), ops.tile_experts(down), rc, "combine", False, oc)
        assert close(out, oc, 1e-2)
        rows = ops.grouped_wide(a, ops.tile_experts(dd), r, "rows", False)
        r2 = ops.moe_sort(tw.cuda(), te.cuda(), E, inverse=True)
        assert close(hops.ExpertRows(rows, r2.inv).sum(), oc, 1e-2)


@pytest.mark.parametrize("device", DEVICES)
def test_products_with_fp32_results(device):
    """Few weight rows (their own kernel in bf16) and many, with and without a bias."""
    g = torch.Generator().manual_seed(1)
    for M, N, K in ((1, 8, 16), (5, 256, 64), (300, 40, 96), (16, 64, 1024), (17, 3, 32), (33, 17, 4096), (2, 1, 64)):
        x, w, b = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g), torch.randn(N, generator=g)
        for dt in (torch.float32, torch.bfloat16):
            a, c = x.to(dt), w.to(dt)
            for bias in (None, b):
                y = hops.linear_f32(a.to(device), c.to(device), None if bias is None else bias.to(device))
                want = a.double() @ c.double().T + (0.0 if bias is None else b.double())
                assert y.dtype == torch.float32 and close(y, want, 2e-6)


@pytest.mark.gpu
@pytest.mark.parametrize("E,k,d,T", [(16, 4, 256, 70), (1, 1, 32, 3), (64, 16, 96, 33), (37, 5, 512, 1), (16, 16, 64, 16),
                                     (48, 8, 4096, 40)])
def test_router_with_its_product(E, k, d, T):
    """The router in one kernel against the two-step form and the plain function: ties take the lower index, weights as they
    are, normalised and scaled."""
    g = torch.Generator().manual_seed(E)
    h = torch.randn(T, d, generator=g).to(torch.bfloat16)
    w = (2.0 * torch.randn(E, d, generator=g) / d ** 0.5).to(torch.bfloat16)
    if E > 8:
        w[7] = w[3]
    hd, wd = h.cuda(), w.cuda()
    assert hops.narrow_ok(hd, wd)
    want = plain.route(h.double() @ w.double().T, k)
    for norm, scale in ((False, 1.0), (True, 2.5)):
        tw, te, _ = hops.moe_router_grouped(hd, wd.float(), None, k, 1, 1, norm=norm, scale=scale, w_act=wd)
        t2, e2, _ = hops.moe_router_grouped(hd, wd.float(), None, k, 1, 1, norm=norm, scale=scale)
        got = torch.zeros(T, E, dtype=torch.float64).scatter_(1, te.long().cpu(), tw.double().cpu())
        ref = want * scale / (want.sum(-1, keepdim=True) if norm else 1.0)
        assert close(got, ref, 1e-5) and close(tw, t2.cpu(), 1e-5) and (te == e2).float().mean() > 0.99


# ---- the model in the engine ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_and_layers(bench_a, device, dtype):
    t = toks(75, 211, 1)
    eng = bench_a.engine(device, dtype)
    lo = []
    got = eng.feed([("a", t, list(range(75)))], ["a"], layers_out=lo)
    if dtype == "float32":
        want_l = []
        plain.forward(bench_a.cfg, bench_a.W, t, layers_out=want_l)
        assert len(lo) == len(want_l) == 9
        for i, (a, b) in enumerate(zip(lo, want_l)):
            assert (a.cpu().double() - b).abs().max() < 1e-4 * b.abs().max(), i
        assert rel_err(got, bench_a.oracle(t)) < TOL[dtype]
    else:
        assert mean_err(got, bench_a.oracle(t)) < TOL[dtype]


@pytest.mark.parametrize("device", DEVICES)
def test_other_sizes_and_ones(device):
    b = Bench(cfg_b(), seed=5)
    t = toks(41, 97, 2)
    eng = b.engine(device)
    assert rel_err(feed_all(eng, "a", t, [41]), b.oracle(t)) < TOL["float32"]
    assert rel_err(feed_all(eng, "b", t, [7, 1, 2]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("loop", [None, (0, 1, 1), (0, 3, 3), (5, 6, 4), (2, 6, 2), (0, 6, 2)])
def test_loops(device, loop):
    """No loop, loops at the start, the end and over everything, one and several passes: every pass reads the embedding
    rows again and its own cache and state."""
    b = Bench(cfg_a(scale=0.9, loop=loop), seed=11, keep=3.0)
    t = toks(50, 211, 4)
    eng = b.engine(device)
    assert len(eng.k_cache) == len(plain.layer_runs(b.cfg))
    assert rel_err(feed_all(eng, "a", t, [30, 1, 2, 17]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("k", range(6))
def test_models_of_one_layer_kind(device, k):
    c = cfg_a(scale=0.9, loop=(1, 2, 2))
    c["layers"] = [copy.deepcopy(c["layers"][k]) for _ in range(2)]
    b = Bench(c, seed=6, keep=3.0)
    t = toks(50, 211, 3)
    assert rel_err(feed_all(b.engine(device), "a", t, [30, 1, 19]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [16], [17, 15, 1, 2], [31, 1, 1, 1, 33], [64, 2]])
def test_portions_and_decoding(bench_sharp, device, cuts):
    """Prompts cut into portions of every size down to two tokens and single decoded tokens, with a peaky softmax and
    memories that keep far tokens, from NaN state slots: every cut lands inside pages and windows somewhere along 90
    tokens."""
    t = toks(90, 211, 7)
    eng = bench_sharp.engine(device)
    poison_state(eng)
    assert rel_err(feed_all(eng, "a", t, cuts), bench_sharp.oracle(t)) < TOL["float32"]
    assert eng.kvm.num_free() == eng.num_blocks


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_and_reuse(bench_a, bench_sharp, device, dtype):
    """Four unequal requests through two slots and ten pages: portions beside single tokens, a request left out of a
    step, pages and slots freed and used again by later requests; every request against itself alone."""
    b = bench_sharp if dtype == "float32" else bench_a
    eng = b.engine(device, dtype, blocks=10, seqs=2)
    poison_state(eng)
    A, B, C, D = toks(100, 211, 11), toks(33, 211, 12), toks(50, 211, 13), toks(17, 211, 14)
    got = {k: [] for k in "ABCD"}

    def step(entries, end=()):
        out = eng.feed([(k, tk, list(range(len(tk)))) for k, tk in entries], list(end))
        r = 0
        for k, tk in entries:
            got[k].append(out[r:r + len(tk)])
            r += len(tk)

    step([("A", A[:30]), ("B", B[:2])])
    step([("B", B[2:3]), ("A", A[30:97])])
    step([("A", A[97:98])])
    step([("A", A[98:99]), ("B", B[3:33])], end=["B"])
    step([("C", C[:40]), ("A", A[99:100])], end=["A"])          # C takes B's slot and pages
    step([("C", C[40:41]), ("D", D[:5])])
    step([("D", D[5:16]), ("C", C[41:50])], end=["C"])
    step([("D", D[16:])], end=["D"])
    assert eng.kvm.num_free() == 10 and eng.slots.num_free() == 2
    for k, tk in (("A", A), ("B", B), ("C", C), ("D", D)):
        g = torch.cat(got[k])
        if dtype == "float32":
            assert rel_err(g, b.oracle(tk)) < TOL["float32"], k
        else:
            assert mean_err(g, b.oracle(tk)) < TOL["bfloat16"], k
            # (per-row rounding can flip a close router call: all rows but a few agree with the request alone)
            alone = row_errs(g, feed_all(b.engine(device, dtype), "x", tk, [len(tk)]).cpu())
            assert alone.median() < 0.03 and (alone > 0.1).float().mean() < 0.1, k


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(bench_sharp, device):
    """A 40-token prompt and 150 single tokens from NaN state, past the rotation's original context: memories are carried
    token by token, every window passes over decoded tokens, the prompt's keys stay visible."""
    t = toks(190, 211, 21)
    eng = bench_sharp.engine(device)
    poison_state(eng)
    assert rel_err(feed_all(eng, "a", t, [40, 1]), bench_sharp.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
def test_long_prompt(bench_sharp, device):
    """300 tokens: keys 18 pages back; whole and in portions."""
    t = toks(300, 211, 22)
    eng = bench_sharp.engine(device)
    assert rel_err(feed_all(eng, "a", t, [300]), bench_sharp.oracle(t)) < TOL["float32"]
    assert rel_err(feed_all(eng, "b", t, [129, 2, 100, 1]), bench_sharp.oracle(t)) < TOL["float32"]


@pytest.mark.gpu
def test_preset_sizes_matrix_cores_and_streamed_projections():
    """The smallest preset in bf16 (attention on the matrix-core kernels, the matrix memory in chunks, tiled projections
    and experts on the weight-streaming kernels for steps of few rows): single tokens and short portions against the
    whole prompt, the whole prompt against the oracle."""
    from kafka_llm_service_amd.models.config import FURAPEL_PRESETS

    cfg = copy.deepcopy(FURAPEL_PRESETS["furapel-tiny"])
    cfg["vocab"] = 1000
    b = Bench(cfg, seed=2)
    t = toks(200, 1000, 4)
    eng = b.engine("cuda:0", "bfloat16")
    eng.model.enable_stream_weights()
    assert eng.model.stream and eng.model.attn_tile_tokens
    assert hasattr(eng.model.layers[0], "w_up_t") and hasattr(eng.model, "loop_in_t")
    whole = feed_all(eng, "w", t, [200])
    assert row_errs(whole, b.oracle(t)).median() < 0.05
    for cuts in ([150, 1], [3, 64, 5]):
        e = row_errs(feed_all(eng, "c", t, cuts), whole.cpu())
        assert e.median() < 0.03 and (e > 0.1).float().mean() < 0.1, cuts
    f32 = b.engine("cuda:0", "float32")
    assert rel_err(feed_all(f32, "f", t, [150, 1]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(bench_a, device):
    """engine.generate: the engine's scheduler, chunked prefill (8-token chunks), slot-limited admission (3 prompts,
    2 slots), sampling kernel; every generated token is the plain model's argmax up to a rounding-sized gap."""
    eng = bench_a.engine(device, seqs=2, max_prefill_chunk=8, max_num_batched_tokens=24)
    prompts = [toks(n, 211, 30 + n) for n in (21, 9, 34)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=7, ignore_eos=True))
    assert all(len(o) == 7 for o in outs)
    for p, o in zip(prompts, outs):
        lg = bench_a.oracle(p + o)
        for i, tok in enumerate(o):
            row = lg[len(p) - 1 + i]
            assert (row.max() - row[tok]).item() < 1e-3 * row.abs().max().item(), i
    assert eng.slots.num_free() == 2 and eng.kvm.num_free() == eng.num_blocks


def test_config_registry_and_checkpoint(tmp_path):
    from kafka_llm_service_amd.models.config import get_config

    b = Bench(cfg_a(), seed=8)
    fp.save_checkpoint(b.mc, b.W, tmp_path / "m")
    mc = get_config(str(tmp_path / "m"))
    assert mc.arch == "furapel" and mc.num_layers == 6 and mc.vocab_size == 211 and mc.hidden_size == 88
    assert mc.runs() == plain.layer_runs(b.cfg) and mc.logit_scale == 0.3 and mc.embed_scale == 2.5
    eng = LLMEngine(EngineConfig(model=str(tmp_path / "m"), weights=str(tmp_path / "m"), device="cpu",
                                 num_kv_blocks=8, max_num_seqs=2, max_model_len=128, dtype="float32"))
    t = toks(20, 211, 9)
    assert rel_err(feed_all(eng, "x", t, [20]), b.oracle(t)) < TOL["float32"]
    bad = copy.deepcopy(b.W)
    bad["loop.in"] = bad["loop.in"][:, :-1]
    with pytest.raises(ValueError):
        fp.FurapelLM(b.mc, "cpu").load_tensors(bad)
    for gone in ("loop.in", "l0.norm1.alpha", "l2.mix.g", "l0.mlp.e3.up"):
        bad = copy.deepcopy(b.W)
        del bad[gone]
        with pytest.raises(KeyError):
            fp.FurapelLM(b.mc, "cpu").load_tensors(bad)
    for spoil in (lambda c: c["layers"][2]["mixer"].update(kv_heads=4),            # 6 heads over 4
                  lambda c: c["layers"][2]["mixer"].update(rot=dict(YARN, dims=16)),   # beyond the head
                  lambda c: c["layers"][1]["mixer"].update(mask={"size": 0}),
                  lambda c: c["layers"][0]["mixer"].update(gate_cap=0.0),
                  lambda c: c["layers"][0]["mlp"]["router"].update(top=8),             # more than there are
                  lambda c: c["layers"][0]["mlp"].update(kind="dense"),
                  lambda c: c["loop"].update(stop=7), lambda c: c["loop"].update(times=0),
                  lambda c: c["layers"][1].update(type="mamba2")):
        c = cfg_a()
        spoil(c)
        with pytest.raises((ValueError, KeyError)):
            mc2 = fp.FurapelConfig.from_dict(c)
            fp.FurapelLM(mc2, "cpu").load_tensors(fp.random_tensors(mc2))
    tiny = get_config("furapel-tiny")
    assert tiny.arch == "furapel" and tiny.num_params() > 0 and len(tiny.runs()) == 6


def test_trace_runner_command_line(tmp_path):
    """bin/trace_run as a program (reference ops on the CPU): a checkpoint folder, three steps on standard input - a
    new request, two requests in one step, a step in which nothing is wanted - then the logits files, the "done"
    lines and the exit code."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    root = Path(__file__).resolve().parents[1]
    b = Bench(cfg_b(), seed=14)
    fp.save_checkpoint(b.mc, b.W, tmp_path / "m")
    t, u = toks(21, 97, 1), toks(6, 97, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:9], "want": [0, 8]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": u, "want": [5]}, {"id": "a", "tokens": t[9:20], "want": []}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": t[20:], "want": [0]}], "end": ["a"]}]
    out = subprocess.run([sys.executable, str(root / "bin/trace_run"), "--model", str(tmp_path / "m"), "--dtype",
                          "float32", "--out", str(tmp_path / "o"), "--max-tokens", "64", "--device", "cpu"],
                         input="".join(json.dumps(x) + "\n" for x in steps), capture_output=True, text=True,
                         timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert [ln for ln in out.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    got = {n: torch.from_numpy(np.fromfile(tmp_path / "o" / f"{n}.f32", dtype="<f4").reshape(-1, 97)) for n in range(3)}
    assert rel_err(got[0], b.oracle(t)[[0, 8]]) < TOL["float32"]
    assert rel_err(got[1], b.oracle(u)[[5]]) < TOL["float32"]
    assert rel_err(got[2], b.oracle(t)[[20]]) < TOL["float32"]
