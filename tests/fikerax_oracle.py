"""Fikerax, slowly: every mechanism of the design as one plain function over a whole sequence, in
float64, with no cache and no batching.  Tests compare the engine with it; it shares no code with
the package.

``t`` maps tensor names of the safetensors file to tensors, ``cfg`` is config.json as a dict.
"""
import math

import torch

F64 = torch.float64


def w64(t, name):
    return t[name].to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def stretched(dims, base, sc):
    """Frequencies of the pairs where long wavelengths are stretched and short ones kept."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def yarn(dims, base, sc):
    """(frequency of every pair, factor of cos and sin)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def dim(turns):
        """The pair that makes ``turns`` turns within the original length."""
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(dim(sc["fast"])), 0), min(math.ceil(dim(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, pos, first, second, freqs, amp=1.0):
    """x [T, heads, D]; entry first[i] is paired with entry second[i] and turned by pos * freqs[i]."""
    out = x.clone()
    for i, f in enumerate(freqs):
        a = pos.to(F64) * f
        co, si = (a.cos() * amp)[:, None], (a.sin() * amp)[:, None]
        u, v = x[..., first[i]], x[..., second[i]]
        out[..., first[i]] = u * co - v * si
        out[..., second[i]] = v * co + u * si
    return out


def rotate_half(x, pos, rot):
    n = rot["dims"] // 2
    return rotate(x, pos, list(range(n)), list(range(n, 2 * n)), stretched(rot["dims"], rot["base"], rot.get("scaling")))


def rotate_pairs(x, pos, rot):
    n = rot["dims"] // 2
    f, amp = yarn(rot["dims"], rot["base"], rot.get("scaling"))
    return rotate(x, pos, list(range(0, 2 * n, 2)), list(range(1, 2 * n, 2)), f, amp)


def visible(T, window):
    """[T, T] bool: row i sees j with 0 <= i - j (< window)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    return (d >= 0) & (d < window) if window else d >= 0


def weights_over_keys(s, vis, sink=None):
    """Softmax of the scores s [T, T] over the visible keys; a sink is one more score without a key."""
    s = s.masked_fill(~vis, -math.inf)
    if sink is None:
        return torch.softmax(s, -1)
    return torch.softmax(torch.cat([s, torch.full((s.shape[0], 1), float(sink), dtype=F64)], 1), -1)[:, :-1]


def decayed_memory(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V] -> [T, H, V]: S <- decay_h S + k v^T, read with q."""
    T, H, D = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        S = torch.zeros(D, v.shape[-1], dtype=F64)
        for i in range(T):
            S = decay[h] * S + torch.outer(k[i, h], v[i, h])
            out[i, h] = S.T @ q[i, h]
    return out


def lightning(t, p, m, h, eps):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w64(t, p + "q").T).view(T, H, D)
    k = silu(h @ w64(t, p + "k").T).view(T, H, D)
    v = silu(h @ w64(t, p + "v").T).view(T, H, V)
    o = decayed_memory(q, k, v, m["decay"]).reshape(T, H * V)
    o = unit_rms(o, eps) * w64(t, p + "norm")
    return (o * torch.sigmoid(h @ w64(t, p + "g").T)) @ w64(t, p + "o").T


def attention(t, p, m, h, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = (h @ w64(t, p + "q").T + w64(t, p + "q.b")).view(T, H, D)
    k = (h @ w64(t, p + "k").T + w64(t, p + "k.b")).view(T, G, D)
    v = (h @ w64(t, p + "v").T + w64(t, p + "v.b")).view(T, G, V)
    if m.get("rot"):
        q, k = rotate_half(q, pos, m["rot"]), rotate_half(k, pos, m["rot"])
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    vis = visible(T, (m.get("mask") or {}).get("size"))
    o = torch.zeros(T, H, V, dtype=F64)
    for i in range(H):
        g = i // (H // G)
        o[:, i] = weights_over_keys(q[:, i] @ k[:, g].T * m["scale"], vis) @ v[:, g]
    return o.reshape(T, H * V) @ w64(t, p + "o").T


def latent_attention(t, p, m, h, eps):
    """Keys and values formed per head from the latents, as the equations have them."""
    T, H, D, R, V, K = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    cq = unit_rms(h @ w64(t, p + "dq").T, eps) * w64(t, p + "dq.norm")
    q = (cq @ w64(t, p + "uq").T).view(T, H, D + R)
    kv = h @ w64(t, p + "dkv").T
    c = unit_rms(kv[:, :K], eps) * w64(t, p + "dkv.norm")
    kr = rotate_pairs(kv[:, None, K:], pos, m["rot"])[:, 0]
    qr = rotate_pairs(q[..., D:], pos, m["rot"])
    k = (c @ w64(t, p + "uk").T).view(T, H, D)
    v = (c @ w64(t, p + "uv").T).view(T, H, V)
    vis = visible(T, (m.get("mask") or {}).get("size"))
    o = torch.zeros(T, H, V, dtype=F64)
    for i in range(H):
        s = (q[:, i, :D] @ k[:, i].T + qr[:, i] @ kr.T) * m["scale"]
        o[:, i] = weights_over_keys(s, vis, w64(t, p + "sink")[i]) @ v[:, i]
    return o.reshape(T, H * V) @ w64(t, p + "o").T


MIXERS = {"lightning": lightning, "attention": attention, "latent_attention": latent_attention}


def feed_forward(t, p, h):
    return (silu(h @ w64(t, p + "gate").T) * (h @ w64(t, p + "up").T)) @ w64(t, p + "down").T


def order_of_runs(cfg):
    """[(layer, the embedding output is added first)] in the order the layers run."""
    lp, n = cfg.get("loop"), len(cfg["layers"])
    if not lp:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(lp["start"])]
    for turn in range(lp["times"]):
        runs += [(i, turn > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(t, cfg, ids, layers_out=None):
    """Logits [T, vocab] of one whole sequence ``ids`` (a list of ints)."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    start = w64(t, "embed")[ids] * cfg["embedding"]["scale"]
    x = start
    for i, again in order_of_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + start
        x = x + MIXERS[L["type"]](t, p + "mix.", L["mixer"], zero_centred_norm(x, w64(t, p + "norm1"), eps), eps)
        if L.get("mlp") is not None:
            x = x + feed_forward(t, p + "mlp.", zero_centred_norm(x, w64(t, p + "norm2"), eps))
        if layers_out is not None:
            layers_out.append(x)
    return zero_centred_norm(x, w64(t, "final.norm"), eps) @ w64(t, "head").T
