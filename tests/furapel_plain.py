"""Plain, slow Furapel forward for the tests: one function per mechanism, whole sequences only, no cache, nothing
carried between calls, float64 by default. It shares nothing with the package: the engine's chunked, paged and batched
results are compared with what these functions give for the whole token list at once.

``cfg`` is the model's config.json as a dict, ``W`` maps tensor names to torch tensors.
"""
from __future__ import annotations

import math

import torch


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def tanh_norm(x, W, name):
    """Element-wise: tanh of the scaled value, times a weight, plus an offset; no statistic of the row."""
    return torch.tanh(W[name + ".alpha"] * x) * W[name] + W[name + ".b"]


def visible(T, window):
    """[T, T] bool: row i sees column j when 0 <= i - j < window (window None: every earlier position)."""
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    ok = dist >= 0
    if window is not None:
        ok = ok & (dist < int(window))
    return ok


def masked_softmax(scores, ok):
    return torch.softmax(scores.masked_fill(~ok, float("-inf")), -1)


def rotation(rot):
    """(angle per position of every pair, factor on cos and sin). With ``scaling`` slow pairs turn ``factor`` times
    slower, fast ones as without it, a linear ramp between the pair numbers that make ``fast`` and ``slow`` turns over
    ``original`` positions."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=torch.float64), 1.0

    def pair_of(turns):
        return dims * math.log(float(sc["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(pair_of(float(sc["slow"]))), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / float(sc["factor"]) * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=torch.float64), 0.1 * math.log(float(sc["factor"])) + 1.0


def rotate_halves(x, rot, first=0):
    """x [T, heads, D] at positions first ..: dimension i turns with dimension i + dims / 2; the rest pass."""
    f, mag = rotation(rot)
    dims = int(rot["dims"])
    half = dims // 2
    ang = torch.arange(first, first + x.shape[0], dtype=torch.float64)[:, None] * f[None]
    c, s = (mag * torch.cos(ang)).to(x.dtype)[:, None], (mag * torch.sin(ang)).to(x.dtype)[:, None]
    a, b = x[..., :half], x[..., half:dims]
    out = x.clone()
    out[..., :half] = a * c - b * s
    out[..., half:dims] = b * c + a * s
    return out


def attention_heads(h, W, p, m):
    """Grouped-query softmax attention before the output projection, every head times one gate: [T, H, Dv]."""
    T = h.shape[0]
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q = (h @ W[p + "q"].T).view(T, H, D)
    k = (h @ W[p + "k"].T).view(T, G, D)
    v = (h @ W[p + "v"].T).view(T, G, Dv)
    if m.get("rot"):
        q, k = rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"])
    gate = torch.sigmoid(h @ W[p + "g"].T)
    ok = visible(T, (m.get("mask") or {}).get("size"))
    rows = []
    for hd in range(H):
        g = hd // (H // G)
        pw = masked_softmax(q[:, hd] @ k[:, g].T * float(m["scale"]), ok)
        rows.append(gate[:, hd:hd + 1] * (pw @ v[:, g]))
    return torch.stack(rows, 1)


def attention(h, W, p, m, eps):
    return attention_heads(h, W, p, m).reshape(h.shape[0], -1) @ W[p + "o"].T


def latent_attention(h, W, p, m, eps):
    """Keys and values of every head from one normed latent row per token; no positions; a sliding window."""
    T = h.shape[0]
    H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
    q = (h @ W[p + "q"].T).view(T, H, D)
    c = rms_unit(h @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    k = (c @ W[p + "uk"].T).view(T, H, D)
    v = (c @ W[p + "uv"].T).view(T, H, Dv)
    ok = visible(T, (m.get("mask") or {}).get("size"))
    rows = [masked_softmax(q[:, hd] @ k[:, hd].T * float(m["scale"]), ok) @ v[:, hd] for hd in range(H)]
    return torch.stack(rows, 1).reshape(T, H * Dv) @ W[p + "o"].T


def mlstm_scan(q, k, v, ig, fg):
    """q (scaled), k [T, H, D], v [T, H, Dv], log gates [T, H] -> read-outs [T, H, Dv]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    n = torch.zeros(H, D, dtype=q.dtype)
    mx = torch.zeros(H, dtype=q.dtype)
    rows = []
    for t in range(T):
        new = torch.maximum(fg[t] + mx, ig[t])
        keep, gain = torch.exp(fg[t] + mx - new), torch.exp(ig[t] - new)
        S = keep[:, None, None] * S + gain[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + gain[:, None] * k[t]
        mx = new
        num = (S * q[t][:, :, None]).sum(1)
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-mx)) + 1e-6
        rows.append(num / den[:, None])
    return torch.stack(rows)


def log_gates(zi, zf, cap):
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm(h, W, p, m, eps):
    T = h.shape[0]
    H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    ig, fg = log_gates(h @ W[p + "i"].T + W[p + "i.b"], h @ W[p + "f"].T + W[p + "f.b"], float(m["gate_cap"]))
    o = rms_unit(mlstm_scan(q, k, v, ig, fg), eps).reshape(T, H * Dv)
    return (o * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def route(z, top):
    """Router logits [T, E] -> weights [T, E]: a softmax over all experts, zero for those not among the ``top``."""
    s = torch.softmax(z, -1)
    out = torch.zeros_like(s)
    for t in range(z.shape[0]):
        for _, e in sorted((-s[t, e].item(), e) for e in range(z.shape[1]))[:top]:
            out[t, e] = s[t, e]
    return out


def experts(h, W, p, mlp):
    w = route(h @ W[p + "router"].T, int(mlp["router"]["top"]))
    y = torch.zeros_like(h)
    for e in range(w.shape[1]):
        rows = (w[:, e] != 0).nonzero()[:, 0]
        if len(rows):
            a = torch.relu(h[rows] @ W[f"{p}e{e}.up"].T) ** 2
            y[rows] += w[rows, e:e + 1] * (a @ W[f"{p}e{e}.down"].T)
    return y


def layer_runs(cfg):
    """(layer, whether a pass of the loop starts before it) in the order of execution."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = int(lp["start"]), int(lp["stop"])
    runs = [(i, False) for i in range(a)]
    for _ in range(int(lp["times"])):
        runs += [(i, i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


MIXERS = {"attention": attention, "latent_attention": latent_attention, "mlstm": mlstm}


def forward(cfg: dict, W: dict, tokens, dtype=torch.float64, layers_out: list | None = None):
    """Logits [T, vocab] of one whole sequence. ``layers_out`` receives the residual after every layer run."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    x = x0
    for i, enters in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if enters:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T
        y = MIXERS[L["type"]](tanh_norm(x, W, p + "norm1"), W, p + "mix.", L["mixer"], eps)
        if L.get("mlp"):
            y = y + experts(tanh_norm(x, W, p + "norm2"), W, p + "mlp.", L["mlp"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x)
    return tanh_norm(x, W, "final.norm") @ W["head"].T * float(cfg.get("logit_scale", 1.0))
