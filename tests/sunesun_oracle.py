"""Sunesun, slowly: every mechanism of the design as one plain function over a whole sequence, in
float64, with no cache and no batching.  Tests compare the engine with it; it shares no code with
the package.

``t`` maps tensor names of the safetensors file to tensors, ``cfg`` is config.json as a dict.
"""
import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def yarn(dims, base, scaling):
    """(frequency of every pair, factor of cos and sin)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(f, dtype=F64), 1.0

    def dim(turns):
        """The dimension whose pair makes ``turns`` turns within the original length."""
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(dim(scaling["fast"])), 0)
    hi = min(math.ceil(dim(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(scaling["factor"]) + 1.0


def rotate(x, pos, rot):
    """x [T, heads, D]: entries 2i and 2i + 1 are a pair, on the first ``dims`` entries of every head."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    f, amp = yarn(dims, rot["base"], rot.get("scaling"))
    out = x.clone()
    for i in range(dims // 2):
        a = pos.to(F64) * f[i]
        co, si = (a.cos() * amp)[:, None], (a.sin() * amp)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * co - v * si
        out[..., 2 * i + 1] = v * co + u * si
    return out


def visible(T, window):
    """[T, T] bool: row i sees j with 0 <= i - j (< window)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    return (d >= 0) & (d < window) if window else d >= 0


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def attend(q, k, v, scale, cap, window):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]."""
    T, H, _ = q.shape
    G = k.shape[1]
    vis = visible(T, window)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = capped(q[:, h] @ k[:, g].T * scale, cap).masked_fill(~vis, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def attention(t, p, m, h):
    """The values are the keys as projected, in front of their rotation."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(T)
    q = rotate((h @ t[p + "q"].to(F64).T).view(T, H, D), pos, m.get("rot"))
    v = (h @ t[p + "k"].to(F64).T).view(T, G, D)
    k = rotate(v, pos, m.get("rot"))
    o = attend(q, k, v, m["scale"], m.get("softcap"), (m.get("mask") or {}).get("size"))
    return o.reshape(T, -1) @ t[p + "o"].to(F64).T


def expert(t, p, h):
    return torch.relu(h @ t[p + "up"].to(F64).T).pow(2) @ t[p + "down"].to(F64).T


def choose(s, top, groups):
    """One token's scores [E] -> the chosen experts' indices, best first."""
    E = s.shape[0]
    ok = list(range(E))
    if groups:
        n = E // groups["count"]
        best = [sum(sorted((float(v) for v in s[g * n:(g + 1) * n]), reverse=True)[:2]) for g in range(groups["count"])]
        kept = sorted(range(groups["count"]), key=lambda g: (-best[g], g))[:groups["keep"]]
        ok = [e for e in ok if e // n in kept]
    return sorted(ok, key=lambda e: (-float(s[e]), e))[:top]


def feed_forward(t, p, f, h):
    r = f["router"]
    s = torch.sigmoid(h @ t[p + "router"].to(F64).T)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e in choose(s[i], r["top"], r.get("groups")):
            out[i] += s[i, e] * expert(t, f"{p}e{e}.", h[i:i + 1])[0]
    return out


def sublayer(t, cfg, p, q, xs, norm, fn):
    """One sublayer around the streams xs [S, T, W] (``fn`` maps the normed input to the sublayer's output)."""
    inn, out, mix = (t[f"{p}hc{q}.{n}"].to(F64) for n in ("in", "out", "mix"))
    S = xs.shape[0]
    u = sum(inn[s] * xs[s] for s in range(S))
    y = fn(unit_rms(u, cfg["norm"]["eps"]) * t[norm].to(F64))
    m = cfg.get("residual_mult", 1.0)
    return torch.stack([sum(mix[s, r] * xs[s] for s in range(S)) + m * out[r] * y for r in range(S)])


def forward(t, cfg, ids, layers_out=None):
    """Logits [T, vocab] of one whole sequence ``ids`` (a list of ints)."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    x = t["embed"].to(F64)[ids] * cfg["embedding"]["scale"]
    S = cfg.get("streams")
    xs = x[None].repeat(S or 1, 1, 1)
    for i, L in enumerate(cfg["layers"]):
        j = i
        while "weights_of" in cfg["layers"][j]:
            j = cfg["layers"][j]["weights_of"]
        p = f"l{j}."
        steps = [(1, lambda h: attention(t, p + "mix.", L["mixer"], h))]
        if L.get("mlp") is not None:
            steps.append((2, lambda h: feed_forward(t, p + "mlp.", L["mlp"], h)))
        for q, fn in steps:
            if S:
                xs = sublayer(t, cfg, p, q, xs, f"{p}norm{q}", fn)
            else:
                h = unit_rms(xs[0], cfg["norm"]["eps"]) * t[f"{p}norm{q}"].to(F64)
                xs = xs + cfg.get("residual_mult", 1.0) * fn(h)[None]
        if layers_out is not None:
            layers_out.append(xs.sum(0))
    return (unit_rms(xs.sum(0), cfg["norm"]["eps"]) * t["final.norm"].to(F64)) @ t["head"].to(F64).T
