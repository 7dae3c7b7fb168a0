"""Rogosun in the serving engine against the plain whole-sequence implementation of tests/rogosun_plain.py.

Small configurations of odd sizes (nothing a multiple of 64, head sizes that differ between keys and values and between
layers, a layer without feed-forward, dense and routed feed-forwards with and without groups and a shared expert) with
random weights made here. Each test runs on the CPU reference ops and, marked ``gpu``, on the HIP kernels.
"""
import copy

import numpy as np
import pytest
import torch

import rogosun_plain as plain
from kafka_llm_service_amd.engine.engine import EngineConfig, LLMEngine
from kafka_llm_service_amd.engine.sequence import SamplingParams
from kafka_llm_service_amd.models import rogosun as rg
from kafka_llm_service_amd.models.budurax import rotary_table
from kafka_llm_service_amd.ops import hybrid as hops

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
RANKS = {"gla.a": 5, "right.a": 7, "right.g": 12}


def _gla(heads=3, dim=20, vdim=28, tau=8.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def _par(heads=6, kv_heads=2, dim=14, rot=8, base=5000.0, factor=4.0, rh=4, rg_=2, rd=18, rv=11, conv=3, ls=0.7, rs=1.1,
         scale=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale or dim ** -0.5}
    if rot:
        left["rot"] = {"base": base, "dims": rot}
        if factor:
            left["rot"]["scaling"] = {"factor": factor}
    right = {"heads": rh, "kv_heads": rg_, "dim": rd, "vdim": rv, "conv": conv}
    return {"left": left, "right": right, "left_scale": ls, "right_scale": rs}


def _dense(ff=52):
    return {"kind": "dense", "ff": ff}


def _moe(experts=12, top=3, ff=20, count=4, keep=2, scale=1.7, shared=28):
    r = {"experts": experts, "top": top, "scale": scale}
    if count:
        r["groups"] = {"count": count, "keep": keep}
    m = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def cfg_a(scale=None):
    layers = [{"type": "parallel", "mixer": _par(scale=scale), "mlp": _moe()},
              {"type": "gla", "mixer": _gla(), "mlp": _dense()},
              {"type": "gla", "mixer": _gla(1, 70, 9, tau=1.0), "mlp": None},
              {"type": "parallel", "mixer": _par(4, 4, 10, rot=0, rh=3, rg_=3, rd=33, rv=70, conv=5, ls=1.2, rs=0.4,
                                                 scale=scale), "mlp": _dense(30)},
              {"type": "gla", "mixer": _gla(2, 17, 40, tau=16.0), "mlp": _moe(6, 2, 33, 0, 0, 0.8, 0)},
              {"type": "parallel", "mixer": _par(3, 1, 22, rot=22, factor=None, rh=1, rg_=1, rd=9, rv=16, conv=2,
                                                 scale=scale), "mlp": None}]
    return {"architecture": "Rogosun", "vocab": 211, "width": 88, "norm": {"eps": 2e-5}, "layers": layers}


def cfg_b():
    """Ones and equal values: one head, as many key heads as query heads, one conv tap, a full rotation of two
    dimensions, groups of one expert, all groups kept, scales of one."""
    layers = [{"type": "parallel", "mixer": _par(1, 1, 16, rot=16, factor=1.0, rh=1, rg_=1, rd=16, rv=16, conv=1, ls=1.0,
                                                 rs=1.0), "mlp": _moe(4, 4, 16, 2, 2, 1.0, 16)},
              {"type": "gla", "mixer": _gla(1, 16, 16, tau=1.0), "mlp": _moe(4, 2, 8, 4, 2, 1.0, 0)},
              {"type": "parallel", "mixer": _par(2, 1, 8, rot=2, rh=2, rg_=1, rd=1, rv=1), "mlp": _moe(3, 1, 8, 1, 1)},
              {"type": "gla", "mixer": _gla(2, 1, 1), "mlp": _dense(8)}]
    return {"architecture": "Rogosun", "vocab": 97, "width": 48, "norm": {"eps": 1e-6}, "layers": layers}


class Bench:
    """A config, its random weights and engines over them."""

    def __init__(self, cfg: dict, seed=0, sharpen=1.0, keep=0.0, ranks=RANKS):
        self.cfg = cfg
        self.mc = rg.RogosunConfig.from_dict(cfg, name="test")
        self.W = rg.random_tensors(self.mc, seed, ranks=ranks)
        for k in self.W:
            # scores far from zero: single keys carry the result; decays near one: far tokens stay in the states
            if sharpen != 1.0 and k.endswith("left.q.norm"):
                self.W[k] = (self.W[k].float() * sharpen).to(torch.bfloat16)
            if keep and k.endswith("a2.b"):
                self.W[k] = (self.W[k].float() + keep).to(torch.bfloat16)
            if keep and k.endswith("dt_bias"):
                self.W[k] = (self.W[k].float() - keep).to(torch.bfloat16)
        self._oracle = {}

    def engine(self, device, dtype="float32", blocks=64, seqs=4, **kw):
        model = rg.RogosunLM(self.mc, device, dtype=getattr(torch, dtype), max_positions=1024).load_tensors(self.W)
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
    return Bench(cfg_a(scale=0.9), seed=3, sharpen=3.0, keep=3.0)


def close(got, want, tol):
    return (got.double().cpu() - want.double()).abs().max().item() < tol * want.abs().max().item()


def seg_tensors(device, runs):
    """runs: (first row, rows, first position, slot) -> (tok_seg, seg)"""
    ts = [j for j, r in enumerate(runs) for _ in range(r[1])]
    return (torch.tensor(ts, dtype=torch.int32, device=device), torch.tensor(runs, dtype=torch.int32, device=device))


# ---- mechanisms alone ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d", [1, 70, 88, 1030, 2048, 4500, 9000])
def test_norm_add(device, d):
    """x += norm(y1 + y2) w: rows that stay in registers and wider ones, vector and scalar sizes, y1 plain, as split-K
    slabs, y1 fp32 beside a bf16 y2 and output; an eps that matters."""
    g = torch.Generator().manual_seed(d)
    T, eps = 5, 0.3
    x0, y1, y2 = (torch.randn(T, d, generator=g) for _ in range(3))
    slabs = torch.randn(4, T, d, generator=g)
    w = 1.0 + 0.3 * torch.randn(d, generator=g)
    dv = lambda t: t.to(device)  # noqa: E731
    for a, b in ((y1, None), (y1, y2), (slabs, None), (slabs, y2)):
        y = (a.double().sum(0) if a.dim() == 3 else a.double()) + (b.double() if b is not None else 0.0)
        want = x0.double() + plain.rms_norm(y, w.double(), eps)
        x, h = dv(x0.clone()), torch.empty(T, d, device=device)
        hops.norm_add(x, dv(a), dv(b) if b is not None else None, dv(w), eps, h)
        assert close(x, want, 1e-5) and torch.equal(h, x)
        x = dv(x0.clone())
        hops.norm_add(x, dv(a), dv(b) if b is not None else None, dv(w), eps)
        assert close(x, want, 1e-5)
        bb = b.to(torch.bfloat16) if b is not None else None
        y = (a.double().sum(0) if a.dim() == 3 else a.double()) + (bb.double() if b is not None else 0.0)
        x, h = dv(x0.clone()), torch.empty(T, d, dtype=torch.bfloat16, device=device)
        hops.norm_add(x, dv(a), dv(bb) if b is not None else None, dv(w), eps, h)
        assert close(x, x0.double() + plain.rms_norm(y, w.double(), eps), 1e-5) and torch.equal(h, x.to(torch.bfloat16))
    yb = y1.to(torch.bfloat16)
    x, h = dv(x0.clone()), torch.empty(T, d, dtype=torch.bfloat16, device=device)
    hops.norm_add(x, dv(yb), None, dv(w), eps, h)
    assert close(x, x0.double() + plain.rms_norm(yb.double(), w.double(), eps), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("F", [1, 20, 64, 1000])
def test_feed_forward_activations_and_head_gate(device, F):
    g = torch.Generator().manual_seed(F)
    T = 7
    for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        u = torch.randn(T, 2 * F, generator=g).to(dt)
        out = torch.empty(T, F, dtype=dt, device=device)
        hops.silu_mul(u.to(device), out)
        assert close(out, plain.silu(u[:, :F].double()) * u[:, F:].double(), tol)
        hops.relu2(u[:, :F].contiguous().to(device), out)
        assert close(out, torch.relu(u[:, :F].double()) ** 2 + 1e-30, tol)
        o, w = torch.randn(T, 3 * F, generator=g), (1.0 + 0.2 * torch.randn(F, generator=g)).to(dt)
        gate = torch.randn(T, 3 * F + 5, generator=g).to(dt)
        both = torch.zeros(T, 3 * F + 9, dtype=dt, device=device)
        for act, fn in (("silu", plain.silu), ("sigmoid", torch.sigmoid)):
            hops.head_norm_gate(o.to(device), w.repeat(3).to(device), gate.to(device), 5, 3, 1e-4, both[:, 9:], 0.6, act)
            want = plain.rms_norm(o.double().view(T, 3, F), w.double(), 1e-4).reshape(T, -1) * fn(gate[:, 5:].double()) * 0.6
            assert close(both[:, 9:], want, tol) and float(both[:, :9].abs().max()) == 0.0


@pytest.mark.gpu
@pytest.mark.parametrize("C,taps,lengths", [(64, 4, [2100, 30]), (40, 2, [7, 19]), (128, 3, [2050, 1]), (24, 4, [1, 3])])
def test_short_conv_vectors(C, taps, lengths):
    """The bf16 vector form of the convolution (a thread per row, or per eight rows in long steps): two sequences from
    NaN slots, then more of both: windows that reach into the slots' tails, over segment borders inside a thread's rows,
    and not into the neighbouring sequence."""
    dev = "cuda:0"
    g = torch.Generator().manual_seed(C)
    w = torch.randn(C, taps, generator=g).to(torch.bfloat16)
    xs = [torch.randn(n + 2100, C + 16, generator=g).to(torch.bfloat16) for n in lengths]
    want = [plain.silu(plain.short_conv(x[:, 8:8 + C].float(), w.float())) for x in xs]
    state = torch.full((3, taps - 1, C), float("nan"), dtype=torch.bfloat16, device=dev)
    at, got = [0, 0], [[], []]
    for sizes in (lengths, [1, 1], [2, 5], [1, 1], [2090, 3]):
        segs = [(0, sizes[0], at[0], 2), (sizes[0], sizes[1], at[1], 0)]
        ts, seg = seg_tensors(dev, segs)
        x = torch.cat([xs[s][at[s]:at[s] + sizes[s]] for s in (0, 1)]).to(dev)
        out = torch.empty(x.shape[0], C, dtype=torch.bfloat16, device=dev)
        hops.short_conv(x, 8, w.to(dev), None, ts, seg, state, out, act="silu")
        got[0].append(out[:sizes[0]].cpu())
        got[1].append(out[sizes[0]:].cpu())
        at = [at[0] + sizes[0], at[1] + sizes[1]]
    for s in (0, 1):
        assert close(torch.cat(got[s]).float(), want[s][:at[s]], 1e-2), s


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,k,count,keep", [(12, 3, 4, 2), (16, 3, 2, 1), (6, 2, 1, 1), (8, 4, 8, 4), (130, 6, 10, 3),
                                            (4, 4, 2, 2), (3, 1, 3, 1)])
def test_router(device, E, k, count, keep):
    """Sigmoid scores, groups by the sum of their two largest (a group with the single best expert loses to one with
    two good ones), weights not normalised but scaled; groups of one expert; everything kept."""
    g = torch.Generator().manual_seed(E)
    T, d = 60, 24
    h, w = torch.randn(T, d, generator=g), torch.randn(E, d, generator=g) / 3
    want = plain.route(h.double() @ w.double().T, {"experts": E, "top": k, "groups": {"count": count, "keep": keep},
                                                   "scale": 1.9})
    tw, te, gate = hops.moe_router_grouped(h.to(device), w.to(device), None, k, count, keep, score="sigmoid",
                                           group_score="top2", norm=False, scale=1.9)
    assert gate is None
    got = torch.zeros(T, E, dtype=torch.float64)
    got.scatter_(1, te.long().cpu(), tw.double().cpu())
    assert close(got, want, 1e-5)
    if (E, count) == (12, 4):   # constructed scores: expert 0 is the best of all, but its group's second is poor
        z = torch.full((1, 12), -4.0)
        z[0, 0], z[0, 3], z[0, 4], z[0, 9], z[0, 10] = 3.0, 1.5, 1.4, 1.3, 1.2
        eye = torch.eye(12)
        tw, te, _ = hops.moe_router_grouped(z.to(device), eye.to(device), None, 3, 4, 2, score="sigmoid",
                                            group_score="top2", norm=False)
        assert sorted(te[0].tolist()) == [3, 4, 9]


def _lin_case(g, n, H, G, D, Dv):
    """Raw inputs of a sequence: rows q | k | v, raw decays, raw beta."""
    return {"qkv": torch.randn(n, 2 * G * D + H * Dv, generator=g), "z": torch.randn(n, H * D, generator=g),
            "beta": torch.randn(n, H, generator=g)}


def _lin_want(c, H, G, D, Dv, zb, rate, tau):
    """The plain result for the raw inputs of ``_lin_case``."""
    n = c["qkv"].shape[0]
    q = c["qkv"][:, :G * D].double().view(n, G, D)
    k = c["qkv"][:, G * D:2 * G * D].double().view(n, G, D)
    v = c["qkv"][:, 2 * G * D:].double().view(n, H, Dv)
    z = (c["z"].double() + zb.double()).view(n, H, D)
    rep = H // G
    if rate is None:
        return plain.gla_scan((q * D ** -0.5).repeat_interleave(rep, 1), k.repeat_interleave(rep, 1), v,
                              torch.sigmoid(z) ** (1.0 / tau)).reshape(n, -1)
    return plain.delta_scan((plain.unit(q) * D ** -0.5).repeat_interleave(rep, 1),
                            plain.unit(k).repeat_interleave(rep, 1), v,
                            torch.exp(rate.double()[None, :, None] * plain.softplus(z)),
                            torch.sigmoid(c["beta"].double())).reshape(n, -1)


LIN_SIZES = [(3, 3, 10, 14), (4, 2, 64, 64), (2, 1, 100, 130), (4, 4, 48, 65), (1, 1, 1, 1), (2, 2, 200, 8),
             (3, 1, 128, 33), (1, 1, 256, 20)]
LIN_PORTIONS = [[(0, 9), (1, 2)], [(1, 1), (0, 1)], [(0, 2), (1, 3)], [(1, 7)], [(0, 130), (1, 65)], [(0, 1)],
                [(1, 201), (0, 3)]]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv", LIN_SIZES)
@pytest.mark.parametrize("delta", [False, True])
def test_lin_scan(device, H, G, D, Dv, delta):
    """Both recurrences through portions of 1, 2, 3, 7, 9 rows and long ones (in chunks on the GPU) from NaN slots, two
    sequences side by side, fp32 and bf16 inputs. One sequence's decays are close to one - what its loud early token
    wrote stays readable hundreds of tokens later -, the other's fast, some channels vanishing within one token (the
    chunked form's pair-by-pair products)."""
    g = torch.Generator().manual_seed(H * 100 + D + delta)
    lengths = [146, 279]
    zb = 0.3 * torch.randn(H * D, generator=g)
    rate = -(0.2 + 3.0 * torch.rand(H, generator=g)) if delta else None
    tau = 1.0 if D % 2 else 12.0
    cases = [_lin_case(g, n, H, G, D, Dv) for n in lengths]
    cases[0]["z"] += -9.0 if delta else 9.0
    cases[0]["qkv"][3, 2 * G * D:] *= 30.0
    cases[0]["qkv"][140:, :G * D] = cases[0]["qkv"][3, G * D:2 * G * D]      # late queries ask for the early key
    cases[1]["z"][:, ::3] += (40.0 if delta else -60.0)
    cases[1]["z"][50:60] += (4.0 if delta else -8.0)
    for dt in (torch.float32, torch.bfloat16):
        if dt == torch.bfloat16:
            for c in cases:
                for n in c:
                    c[n] = c[n].to(dt)
        want = [_lin_want(c, H, G, D, Dv, zb, rate, tau) for c in cases]
        S = torch.full((3, H, D, Dv), float("nan"), device=device)
        at, got = [0, 0], [[], []]
        for portions in LIN_PORTIONS:
            runs, r0 = [], 0
            for s, n in portions:
                n = min(n, lengths[s] - at[s])
                runs.append((s, at[s], n, r0))
                r0 += n
            segs = [(q0, n, p0, 2 - s) for s, p0, n, q0 in runs]              # slots 2 and 1 of 3
            ts, seg = seg_tensors(device, segs)
            cat = {k: torch.cat([cases[s][k][p0:p0 + n] for s, p0, n, _ in runs]).to(device) for k in cases[0]}
            tabs = hops.lin_chunk_tables(np.asarray(segs, dtype=np.int32)) if device != "cpu" else None
            if tabs is not None:
                tabs = tuple(torch.from_numpy(x).to(device) for x in tabs)
            out = torch.full((r0, H * Dv), float("nan"), device=device)
            hops.lin_scan(cat["qkv"], 0, G * D, cat["qkv"][:, 2 * G * D:], cat["z"], zb.to(device), H, G, D, Dv, ts,
                          seg, S, out, tau, rate.to(device) if delta else None, cat["beta"] if delta else None, tabs)
            for s, p0, n, q0 in runs:
                got[s].append(out[q0:q0 + n].cpu())
                at[s] += n
        assert at == lengths
        for s in (0, 1):
            assert close(torch.cat(got[s]), want[s], 5e-5), (s, dt)
        # (row by row: small rows beside loud ones)
        e = (torch.cat(got[1]).double() - want[1]).abs().max(-1).values
        assert (e < 2e-4 * want[1].abs().max(-1).values + 1e-6).all(), dt
        assert not torch.isnan(S[1:]).any() and torch.isnan(S[0]).all()


@pytest.mark.gpu
@pytest.mark.parametrize("delta", [False, True])
@pytest.mark.parametrize("n", [64, 65, 79, 95, 96, 97, 128, 161, 700])
def test_lin_scan_in_chunks(delta, n):
    """The chunked form against the token-by-token kernel and the plain function: every kind of last chunk, a segment
    that continues from a state, the state it leaves."""
    dev = "cuda:0"
    assert hops.ext().hy_lin_chunk() == hops.LIN_CHUNK
    H, G, D, Dv, tau = 3, 3, 40, 50, 4.0
    g = torch.Generator().manual_seed(n)
    zb = torch.randn(H * D, generator=g)
    rate = -(0.1 + torch.rand(H, generator=g)) if delta else None
    c = _lin_case(g, n + 21, H, G, D, Dv)
    want = _lin_want(c, H, G, D, Dv, zb, rate, tau)
    outs = []
    for chunked in (False, True):
        S = torch.full((2, H, D, Dv), float("nan"), device=dev)
        got = []
        for p0, m in ((0, 21), (21, n)):
            segs = [(0, m, p0, 1)]
            ts, seg = seg_tensors(dev, segs)
            tabs = hops.lin_chunk_tables(np.asarray(segs, dtype=np.int32)) if chunked else None
            assert (tabs is not None) == (chunked and m >= 64)
            if tabs is not None:
                tabs = tuple(torch.from_numpy(x).to(dev) for x in tabs)
            x = {k: v[p0:p0 + m].to(dev) for k, v in c.items()}
            out = torch.empty(m, H * Dv, device=dev)
            hops.lin_scan(x["qkv"], 0, G * D, x["qkv"][:, 2 * G * D:], x["z"], zb.to(dev), H, G, D, Dv, ts, seg, S, out,
                          tau, rate.to(dev) if delta else None, x["beta"] if delta else None, tabs,
                          (m, m) if tabs is None else None)
            got.append(out.cpu())
        outs.append((torch.cat(got), S[1].cpu()))
        assert close(outs[-1][0], want, 3e-5), chunked
    assert close(outs[1][1], outs[0][1], 3e-5)


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


def _attn_case(g, n, H, G, D, rot, factor, spots):
    """Rows [q | k] of a sequence with (row, key) pairs whose score stands out, and the plain result (the projections are
    selections of the row's columns, the output projection is the identity). Where the first rows' scores are all far
    below zero the added one carries the denominator."""
    C = H * D + G * D
    h = torch.randn(n, C, generator=g)
    for i, (at, key) in enumerate(spots):
        hd = i % H
        c = H * D + (hd // (H // G)) * D
        if rot:   # the pair's rotations differ: align only the dimensions that pass (a full rotation: all of them)
            lo = rot if rot < D else 0
        else:
            lo = 0
        h[at, hd * D + lo:(hd + 1) * D] = 2.0 * h[key, c + lo:c + D]
    h[0, :H * D] = -2.0 * h[0, H * D:].view(G, D).repeat_interleave(H // G, 0).reshape(-1)
    eye = torch.eye(C, dtype=torch.float64)
    W = {"q": eye[:H * D], "k": eye[H * D:], "q.norm": 1.0 + 0.2 * torch.randn(D, generator=g).double(),
         "k.norm": 1.0 + 0.2 * torch.randn(D, generator=g).double(), "o": torch.eye(H * D).double()}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": 4.0 * D ** -0.5}
    if rot:
        m["rot"] = {"dims": rot, "base": 777.0, "scaling": {"factor": factor}}
    return h, m, W


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,rot,factor", [(6, 2, 24, 10, 3.0), (4, 4, 8, 0, 1.0), (3, 1, 100, 100, 8.0),
                                              (1, 1, 8, 8, 1.0), (8, 2, 16, 6, 2.5)])
def test_attention_on_raw_keys_single_keys(device, H, G, D, rot, factor):
    """Per-head norms, linearly scaled rotation (part of a head), keys as projected as values, the softmax with one
    added to its denominator, the scaled result in a column slice, through scattered pages, in portions, two sequences
    side by side. Loud keys sit at the first positions, on both sides of page borders, at the row's own position and
    hundreds of tokens back, for rows of a portion and for rows fed alone."""
    g = torch.Generator().manual_seed(H * 100 + D)
    n0, n1, eps = 330, 23, 1e-4
    spots = [(329, 0), (329, 329), (140, 127), (140, 128), (100, 15), (100, 16), (297, 1), (297, 2), (298, 40), (5, 0),
             (1, 1), (328, 31)]
    cases = [_attn_case(g, n0, H, G, D, rot, factor, spots), _attn_case(g, n1, H, G, D, rot, factor, [(22, 0), (20, 16)])]
    W, m = cases[0][2], cases[0][1]
    want = [plain.shared_kv_attention(h.double(), W, "", m, eps) * 0.6 for h, _, _ in cases]
    pg = Paged(device, [n0, n1], seed=H)
    kc = torch.zeros(pg.n_pages, 16, G * D, device=device)
    vt = torch.zeros(pg.n_pages, G * D, 16, device=device)
    cs = rotary_table(512, m["rot"], device) if rot else None
    qn, kn = W["q.norm"].float().to(device), W["k.norm"].float().to(device)
    sink = torch.zeros(H, device=device)
    got = [torch.empty(n0, H * D), torch.empty(n1, H * D)]
    at = [0, 0]
    for portions in ([(0, 97), (1, 2)], [(1, 20), (0, 1)], [(0, 2)], [(0, 197), (1, 1)], [(0, 1)], [(0, 1)], [(0, 31)]):
        runs = [(s, at[s], n) for s, n in portions]
        bt, ts, pos, sl = pg.step(runs)
        rows = torch.cat([cases[s][0][a:a + n] for s, a, n in runs]).to(device)
        q = torch.empty(rows.shape[0], H * D, device=device)
        hops.rope_kv_store(rows, H, G, D, D, pos, cs, rot, False, None, kc, vt, sl, q, qn, kn, eps, v_off=H * D)
        both = torch.zeros(rows.shape[0], H * D + 7, device=device)
        hops.window_attn(q, kc, vt, bt, ts, pos, H, G, m["scale"], 0, sink, both[:, :H * D], out_scale=0.6)
        assert float(both[:, H * D:].abs().max()) == 0.0
        r = 0
        for s, a, n in runs:
            got[s][a:a + n] = both[r:r + n, :H * D].cpu()
            r += n
            at[s] += n
    assert at == [n0, n1]
    for s in (0, 1):
        assert close(got[s], want[s], 2e-4), s


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,rot", [(4, 2, 128, 128), (3, 1, 64, 32), (5, 5, 16, 16), (2, 1, 8, 0), (6, 3, 256, 96),
                                       (2, 2, 48, 48)])
def test_attention_inputs_bf16(H, G, D, rot):
    """Norm, rotation and paged store of bf16 rows (registers where the head size is a power of two, LDS otherwise)
    against the plain functions, inside wider rows, at positions far from zero."""
    dev = "cuda:0"
    g = torch.Generator().manual_seed(D + rot)
    n, eps = 37, 1e-3
    rows = torch.randn(n, (H + G) * D + 24, generator=g).to(torch.bfloat16)
    qn, kn = 1.0 + 0.2 * torch.randn(D, generator=g), 1.0 + 0.2 * torch.randn(D, generator=g)
    pg = Paged(dev, [500])
    _, _, pos, sl = pg.step([(0, 401, n)])
    kc = torch.zeros(pg.n_pages, 16, G * D, dtype=torch.bfloat16, device=dev)
    vt = torch.zeros(pg.n_pages, G * D, 16, dtype=torch.bfloat16, device=dev)
    cs = rotary_table(512, {"dims": rot, "base": 33.0, "scaling": {"factor": 2.0}}, dev) if rot else None
    q = torch.empty(n, H * D, dtype=torch.bfloat16, device=dev)
    hops.rope_kv_store(rows.to(dev), H, G, D, D, pos, cs, rot, False, None, kc, vt, sl, q, qn.to(dev), kn.to(dev), eps,
                       v_off=H * D)
    r = rows.double()
    wq = plain.rms_norm(r[:, :H * D].view(n, H, D), qn.double(), eps)
    wk = plain.rms_norm(r[:, H * D:(H + G) * D].view(n, G, D), kn.double(), eps)
    if rot:
        pad = torch.zeros(401, 1, 1, dtype=torch.float64)
        wq = plain.rotate_halves(torch.cat([pad.expand(401, H, D), wq]), rot, 33.0, 2.0)[401:]
        wk = plain.rotate_halves(torch.cat([pad.expand(401, G, D), wk]), rot, 33.0, 2.0)[401:]
    assert close(q.float(), wq.reshape(n, -1), 1e-2)
    assert close(kc.view(-1, G * D)[sl].float(), wk.reshape(n, -1), 1e-2)
    v = vt.permute(0, 2, 1).reshape(-1, G * D)[sl].cpu()
    assert torch.equal(v, rows[:, H * D:(H + G) * D])
    assert kc.count_nonzero() == kc.view(-1, G * D)[sl].count_nonzero()      # nothing outside the rows' slots


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,n", [(8, 2, 32, 300), (4, 4, 64, 700), (32, 1, 48, 200), (16, 2, 128, 1500),
                                     (2, 1, 256, 520)])
def test_attention_on_raw_keys_matrix_cores(H, G, D, n):
    """The matrix-core attention (bf16) against the plain function: prompt portions and decode rows, whole key ranges and
    split ones, the denominator's one, the scale, a column slice as the output."""
    dev = "cuda:0"
    g = torch.Generator().manual_seed(H * D + n)
    spots = [(n - 1, 0), (n - 1, n - 1), (140, 127), (140, 128), (100, 15), (n - 2, 1), (n - 1, n - 41), (n - 40, 3)]
    h, m, W = _attn_case(g, n, H, G, D, 0, 1.0, spots)
    hb = h.to(torch.bfloat16)
    want = plain.shared_kv_attention(hb.double(), W, "", m, 1e-5) * 0.7
    pg = Paged(dev, [n], seed=5)
    kc = torch.zeros(pg.n_pages, 16, G * D, dtype=torch.bfloat16, device=dev)
    vt = torch.zeros(pg.n_pages, G * D, 16, dtype=torch.bfloat16, device=dev)
    tt = hops.sig_tile_tokens(H, G)
    got = torch.empty(n, H * D)
    at = 0
    for rows in (n - 40, 1, 38, 1):
        bt, ts, pos, sl = pg.step([(0, at, rows)])
        q = torch.empty(rows, H * D, dtype=torch.bfloat16, device=dev)
        hops.rope_kv_store(hb[at:at + rows].to(dev), H, G, D, D, pos, None, 0, False, None, kc, vt, sl, q,
                           W["q.norm"].float().to(dev), W["k.norm"].float().to(dev), 1e-5, v_off=H * D)
        tiles = torch.tensor([(a, min(tt, rows - a), 0, 0) for a in range(0, rows, tt)], dtype=torch.int32, device=dev)
        assert hops.window_attn_mfma_ok(q, kc, vt, H, G)
        outs = []
        for max_keys in (0, at + rows):   # unsplit; split key ranges where the launch has few tiles
            both = torch.zeros(rows, H * D + 8, dtype=torch.bfloat16, device=dev)
            hops.window_attn(q, kc, vt, bt, ts, pos, H, G, m["scale"], 0, torch.zeros(H, device=dev), both[:, :H * D],
                             tiles, max_keys, out_scale=0.7)
            outs.append(both[:, :H * D].float().cpu())
        assert (outs[0] - outs[1]).abs().max() < 0.02 * want.abs().max()
        got[at:at + rows] = outs[1]
        at += rows
    assert at == n
    assert (got.double() - want).abs().max() < 0.04 * want.abs().max()


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
        assert len(lo) == len(want_l) == 6
        for i, (a, b) in enumerate(zip(lo, want_l)):
            assert (a.cpu().double() - b).abs().max() < 1e-4 * b.abs().max(), i
        assert rel_err(got, bench_a.oracle(t)) < TOL[dtype]
    else:
        assert mean_err(got, bench_a.oracle(t)) < TOL[dtype]


@pytest.mark.parametrize("device", DEVICES)
def test_other_sizes_and_ones(device):
    b = Bench(cfg_b(), seed=5, ranks={"gla.a": 1, "right.a": 1, "right.g": 8})
    t = toks(41, 97, 2)
    eng = b.engine(device)
    assert rel_err(feed_all(eng, "a", t, [41]), b.oracle(t)) < TOL["float32"]
    assert rel_err(feed_all(eng, "b", t, [7, 1, 2]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("k", range(6))
def test_models_of_one_layer_kind(device, k):
    c = cfg_a(scale=0.9)
    c["layers"] = [copy.deepcopy(c["layers"][k]) for _ in range(2)]
    b = Bench(c, seed=6, sharpen=2.0, keep=3.0)
    t = toks(50, 211, 3)
    assert rel_err(feed_all(b.engine(device), "a", t, [30, 1, 19]), b.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2], [16], [17, 15, 1, 2], [31, 1, 1, 1, 33], [64, 2]])
def test_portions_and_decoding(bench_sharp, device, cuts):
    """Prompts cut into portions of every size down to two tokens and single decoded tokens, with a peaky softmax and
    states that keep far tokens, from NaN state slots: every cut lands inside pages somewhere along 90 tokens."""
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
    """A 40-token prompt and 150 single tokens from NaN state: the recurrent states and the convolutions' tails are
    carried token by token and the prompt's keys stay visible."""
    t = toks(190, 211, 21)
    eng = bench_sharp.engine(device)
    poison_state(eng)
    assert rel_err(feed_all(eng, "a", t, [40, 1]), bench_sharp.oracle(t)) < TOL["float32"]


@pytest.mark.parametrize("device", DEVICES)
def test_long_prompt(bench_sharp, device):
    """300 tokens: keys 18 pages back, recurrences in chunks on the GPU; whole and in portions."""
    t = toks(300, 211, 22)
    eng = bench_sharp.engine(device)
    assert rel_err(feed_all(eng, "a", t, [300]), bench_sharp.oracle(t)) < TOL["float32"]
    assert rel_err(feed_all(eng, "b", t, [129, 2, 100, 1]), bench_sharp.oracle(t)) < TOL["float32"]


@pytest.mark.gpu
def test_chunks_beside_short_segments_in_the_engine(bench_sharp):
    """A 500-token portion beside a short one in the same step (chunked and token-by-token launches of one scan), then
    more of both."""
    t, u = toks(560, 211, 23), toks(30, 211, 24)
    eng = bench_sharp.engine("cuda:0")
    poison_state(eng)
    a = eng.feed([("a", t[:20], list(range(20)))], [])
    b = eng.feed([("u", u[:9], list(range(9))), ("a", t[20:520], list(range(500)))], [])
    c = eng.feed([("u", u[9:], list(range(21))), ("a", t[520:], list(range(40)))], ["a", "u"])
    assert rel_err(torch.cat([a, b[9:], c[21:]]), bench_sharp.oracle(t)) < TOL["float32"]
    assert rel_err(torch.cat([b[:9], c[:21]]), bench_sharp.oracle(u)) < TOL["float32"]


@pytest.mark.gpu
def test_preset_sizes_matrix_cores_and_streamed_projections():
    """The smallest preset in bf16 (attention on the matrix-core kernel, tiled projections and experts on the
    weight-streaming kernels for steps of few rows): single tokens and short portions against the whole prompt, the
    whole prompt against the oracle."""
    from kafka_llm_service_amd.models.config import ROGOSUN_PRESETS

    cfg = copy.deepcopy(ROGOSUN_PRESETS["rogosun-tiny"])
    cfg["vocab"] = 1000
    b = Bench(cfg, seed=2, ranks={"gla.a": 16, "right.a": 24, "right.g": 40})
    t = toks(200, 1000, 4)
    eng = b.engine("cuda:0", "bfloat16")
    eng.model.enable_stream_weights()
    assert eng.model.stream and eng.model.attn_tile_tokens
    moe = [lw for lw in eng.model.layers if lw.ff == "moe"][0]
    assert hasattr(moe, "w_gu_t") and hasattr(moe, "sh_gu_t")
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
    rg.save_checkpoint(b.mc, b.W, tmp_path / "m")
    mc = get_config(str(tmp_path / "m"))
    assert mc.arch == "rogosun" and mc.num_layers == 6 and mc.vocab_size == 211 and mc.hidden_size == 88
    eng = LLMEngine(EngineConfig(model=str(tmp_path / "m"), weights=str(tmp_path / "m"), device="cpu",
                                 num_kv_blocks=8, max_num_seqs=2, max_model_len=128, dtype="float32"))
    t = toks(20, 211, 9)
    assert rel_err(feed_all(eng, "x", t, [20]), b.oracle(t)) < TOL["float32"]
    bad = copy.deepcopy(b.W)
    bad["l0.mix.right.q.conv"] = bad["l0.mix.right.q.conv"][:-1]
    with pytest.raises(ValueError):
        rg.RogosunLM(b.mc, "cpu").load_tensors(bad)
    for gone in ("l0.mix.right.q.conv", "l1.mix.a1", "l0.mlp.e3.up"):
        bad = copy.deepcopy(b.W)
        del bad[gone]
        with pytest.raises(KeyError):
            rg.RogosunLM(b.mc, "cpu").load_tensors(bad)
    for spoil in (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4),          # 6 heads over 4
                  lambda c: c["layers"][0]["mixer"]["right"].update(kv_heads=3),         # 4 heads over 3
                  lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=16),      # beyond the head
                  lambda c: c["layers"][0]["mixer"]["left"].update(vdim=13),             # values are the keys
                  lambda c: c["layers"][0]["mlp"]["router"].update(top=7),               # more than the kept groups hold
                  lambda c: c["layers"][1]["mixer"].update(tau=0.0),
                  lambda c: c["layers"][1]["mlp"].update(kind="glu"),
                  lambda c: c["layers"][1].update(type="mamba2")):
        c = cfg_a()
        spoil(c)
        with pytest.raises((ValueError, KeyError)):
            mc2 = rg.RogosunConfig.from_dict(c)
            rg.RogosunLM(mc2, "cpu").load_tensors(rg.random_tensors(mc2, ranks=RANKS))
    tiny = get_config("rogosun-tiny")
    assert tiny.arch == "rogosun" and tiny.num_params() > 0


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
    rg.save_checkpoint(b.mc, b.W, tmp_path / "m")
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
