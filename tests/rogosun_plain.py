"""Plain, slow Rogosun forward for the tests: one function per mechanism, whole sequences only, no cache, nothing
carried between calls, float64 by default. It shares nothing with the package: the engine's chunked, paged and batched
results are compared with what these functions give for the whole token list at once.

``cfg`` is the model's config.json as a dict, ``W`` maps tensor names to torch tensors.
"""
from __future__ import annotations

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate_halves(x, dims, base, factor=1.0):
    """x [T, heads, D]: dimension i turns with dimension i + dims / 2 (i < dims / 2) by position * base^(-2i/dims) /
    factor; the other dimensions pass."""
    half = dims // 2
    f = torch.tensor([float(base) ** (-2.0 * i / dims) / factor for i in range(half)], dtype=torch.float64)
    ang = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * f[None]
    c, s = torch.cos(ang).to(x.dtype)[:, None], torch.sin(ang).to(x.dtype)[:, None]
    a, b = x[..., :half], x[..., half:dims]
    out = x.clone()
    out[..., :half] = a * c - b * s
    out[..., half:dims] = b * c + a * s
    return out


def softmax_one_more(s):
    """s [H, T, T] -> e^s_ij / (1 + sum_{j <= i} e^s_ij): a softmax with a further score of 0 in its denominator."""
    T = s.shape[-1]
    ok = torch.ones(T, T, dtype=torch.bool).tril()
    s = s.masked_fill(~ok, float("-inf"))
    m = s.max(-1, keepdim=True).values.clamp(min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def shared_kv_attention(h, W, p, m, eps):
    """Grouped-query attention whose values are the raw key projection; per-head RMS norm on q and k, then rotation."""
    T = h.shape[0]
    H, G, D = (int(m[k]) for k in ("heads", "kv_heads", "dim"))
    q = (h @ W[p + "q"].T).view(T, H, D)
    k = (h @ W[p + "k"].T).view(T, G, D)
    v = k
    q = rms_norm(q, W[p + "q.norm"], eps)
    k = rms_norm(k, W[p + "k.norm"], eps)
    rot = m.get("rot")
    if rot:
        f = float((rot.get("scaling") or {}).get("factor", 1.0))
        q = rotate_halves(q, int(rot["dims"]), rot["base"], f)
        k = rotate_halves(k, int(rot["dims"]), rot["base"], f)
    rows = []
    for hd in range(H):
        g = hd // (H // G)
        pw = softmax_one_more((q[:, hd] @ k[:, g].T * float(m["scale"]))[None])[0]
        rows.append(pw @ v[:, g])
    return torch.stack(rows, 1).reshape(T, H * D) @ W[p + "o"].T


def short_conv(x, w):
    """x [T, C], w [C, taps], the last column belongs to the current row; zeros before the start."""
    out = torch.zeros_like(x)
    taps = w.shape[1]
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] = out[t] + x[s] * w[:, j]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta):
    """Per head (q, k, g [T, H, D], v [T, H, Dv], beta [T, H]): S <- g S; u = beta (v - S^T k); S <- S + k u^T;
    out S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    rows = []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        rows.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(rows)


def delta_inputs(h, W, p, m):
    T = h.shape[0]
    H, G, D, Dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q, k, v = (silu(short_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = (unit(q.view(T, G, D)) * D ** -0.5).repeat_interleave(H // G, 1)
    k = unit(k.view(T, G, D)).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    dt = softplus((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]).view(T, H, D)
    g = torch.exp(-torch.exp(W[p + "A_log"])[None, :, None] * dt)
    return q, k, v.view(T, H, Dv), g, beta


def gated_delta(h, W, p, m, eps):
    T = h.shape[0]
    H, Dv = int(m["heads"]), int(m["vdim"])
    o = rms_norm(delta_scan(*delta_inputs(h, W, p, m)), W[p + "norm"], eps).reshape(T, H * Dv)
    return (o * torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)) @ W[p + "o"].T


def gla_scan(q, k, v, a):
    """Per head: S <- diag(a) S + k v^T, out S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    rows = []
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        rows.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(rows)


def gla(h, W, p, m, eps):
    T = h.shape[0]
    H, D, Dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    a = (torch.sigmoid(z) ** (1.0 / float(m["tau"]))).view(T, H, D)
    o = rms_norm(gla_scan(q, k, v, a), W[p + "norm"], eps).reshape(T, H * Dv)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    return float(m["left_scale"]) * shared_kv_attention(h, W, p + "left.", m["left"], eps) + \
        float(m["right_scale"]) * gated_delta(h, W, p + "right.", m["right"], eps)


def glu(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z, r):
    """Router logits z [T, E] -> weights [T, E] (zero for experts not chosen)."""
    E, top = int(r["experts"]), int(r["top"])
    gr = r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(gr["count"]), int(gr["keep"])
    s = torch.sigmoid(z)
    out = torch.zeros_like(s)
    n = E // count
    for t in range(z.shape[0]):
        score = []
        for g in range(count):
            best = sorted(s[t, g * n:(g + 1) * n].tolist(), reverse=True)[:2]
            score.append((-sum(best), g))
        kept = [g for _, g in sorted(score)[:keep]]
        cand = sorted((-s[t, e].item(), e) for g in kept for e in range(g * n, (g + 1) * n))[:top]
        for _, e in cand:
            out[t, e] = s[t, e] * float(r.get("scale", 1.0))
    return out


def feed_forward(h, W, p, mlp):
    if mlp["kind"] == "dense":
        return torch.relu(h @ W[p + "up"].T) ** 2 @ W[p + "down"].T
    w = route(h @ W[p + "router"].T, mlp["router"])
    y = torch.zeros_like(h)
    for e in range(w.shape[1]):
        rows = (w[:, e] != 0).nonzero()[:, 0]
        if len(rows):
            y[rows] += w[rows, e:e + 1] * glu(h[rows], W, f"{p}e{e}.")
    if mlp.get("shared"):
        y = y + glu(h, W, p + "shared.")
    return y


def forward(cfg: dict, W: dict, tokens, dtype=torch.float64, layers_out: list | None = None):
    """Logits [T, vocab] of one whole sequence. ``layers_out`` receives the residual after every layer."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        mix = {"gla": gla, "parallel": parallel}[L["type"]]
        x = x + rms_norm(mix(x, W, p + "mix.", L["mixer"], eps), W[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + rms_norm(feed_forward(x, W, p + "mlp.", L["mlp"]), W[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T
