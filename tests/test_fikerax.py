"""Fikerax through the engine against the plain implementation in ``fikerax_oracle.py``:
each mechanism alone, prefill against token-by-token decoding, portions, mixed batches,
reuse of pages and state slots, keys at window and page borders, the first tokens of a
sequence, long decoding, repeated layers, other sizes, and greedy generation through
``submit`` / ``step``.

Every case runs on the CPU (the ops' fp32 forms, the same engine, cache manager and
scheduler) and, marked ``gpu``, on the HIP kernels in fp32 and bf16.
"""
import io
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import fikerax_oracle as O
from k8s_llm_rca_amd.engine.engine import EngineConfig, LLMEngine
from k8s_llm_rca_amd.models.fikerax import FikeraxConfig, FikeraxModel
from k8s_llm_rca_amd.ops import norm as N
from k8s_llm_rca_amd.ops import seq_ops as S

GPU = pytest.mark.gpu
BACKENDS = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
            pytest.param(("cuda", torch.float32), id="gpu-f32", marks=GPU),
            pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=GPU)]
MFMA_BACKEND = [pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=GPU)]
DT = torch.float64
STALE = 2.0 ** 15     # what unwritten page entries hold in these tests (exact in bfloat16)


def row_errs(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-30)


def agrees(got, want, dtype, mult=1.0):
    """Logits rows against the oracle's: every row in fp32; in bf16 (rounding of a dozen sublayers) most rows close and
    none far (a wrong key or a lost state moves a row by tens of percent here, an unrelated row differs by 1.4)."""
    e = row_errs(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 3e-5 * mult
    return float(e.median()) < 0.02 * mult and float(e.max()) < 0.08 * mult


def close(got, want, dtype, scale=1.0):
    """Element-wise check of an op's output against fp64."""
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape
    t = (2e-5 if dtype == torch.float32 else 2e-2) * scale
    err = float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))
    assert err < t, err


# ------------------------------------------------------------------ configurations and weights
STRETCH = {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 40}
YARN = {"factor": 3.0, "original": 60, "fast": 6.0, "slow": 1.0}


def lig(heads=3, dim=8, vdim=12, decay=None, **_):
    decay = decay or [0.5 + 0.49 * (h + 1) / heads for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def att(heads=6, kv_heads=3, dim=8, vdim=10, scale=1.3, window=21, rot=6, base=300.0, scaling=STRETCH):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if scaling:
            m["rot"]["scaling"] = scaling
    return {"type": "attention", "mixer": m}


def lat(heads=5, dim=8, rot=6, vdim=7, q_rank=20, kv_rank=12, scale=0.4, window=17, base=200.0, scaling=YARN):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"dims": rot, "base": base}}
    if scaling:
        m["rot"]["scaling"] = scaling
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def config(layers, width=48, vocab=512, eps=1e-5, scale=7.0, loop=None):
    d = {"architecture": "Fikerax", "vocab": vocab, "width": width, "embedding": {"scale": scale},
         "layers": [dict(mix, mlp={"kind": "dense", "ff": ff} if ff else None) for mix, ff in layers], "norm": {"eps": eps}}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def default_config(**kw):
    kw.setdefault("loop", (1, 4, 2))
    return config([(lat(), 40), (lig(), 0), (att(), 36), (lat(heads=3, window=30, rot=8), 0), (lig(heads=2, vdim=8), 28),
                   (att(heads=2, kv_heads=2, dim=6, vdim=6, rot=4, window=9), 0)], **kw)


def weights(d, seed=0):
    """Random weights under the checkpoint's names, rounded to bfloat16."""
    g = torch.Generator().manual_seed(seed)
    W = d["width"]

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    def lin(o, i, mul=1.0):
        return r(o, i, std=mul * i ** -0.5)

    t = {"embed": r(d["vocab"], W, std=1.0 / d["embedding"]["scale"]), "head": lin(d["vocab"], W), "final.norm": r(W, std=0.2)}
    for i, L in enumerate(d["layers"]):
        p, m = f"l{i}.mix.", L["mixer"]
        t[f"l{i}.norm1"] = r(W, std=0.2)
        H = m["heads"]
        if L["type"] == "lightning":
            for n, rows in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * m["vdim"]), ("g", H * m["vdim"])):
                t[p + n] = lin(rows, W, 1.5)
            t[p + "norm"], t[p + "o"] = r(H * m["vdim"], std=0.2, mean=1.0), lin(W, H * m["vdim"])
        elif L["type"] == "attention":
            for n, rows in (("q", H * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                t[p + n], t[p + n + ".b"] = lin(rows, W), r(rows, std=0.4)
            t[p + "o"] = lin(W, H * m["vdim"])
        else:
            K = m["kv_rank"]
            t[p + "dq"], t[p + "dq.norm"] = lin(m["q_rank"], W), r(m["q_rank"], std=0.2, mean=1.0)
            t[p + "uq"] = lin(H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            t[p + "dkv"], t[p + "dkv.norm"] = lin(K + m["rot_dim"], W), r(K, std=0.2, mean=1.0)
            t[p + "uk"], t[p + "uv"] = lin(H * m["dim"], K), lin(H * m["vdim"], K)
            t[p + "sink"], t[p + "o"] = r(H, std=1.0), lin(W, H * m["vdim"])
        if L["mlp"]:
            t[f"l{i}.norm2"] = r(W, std=0.2)
            f, q = L["mlp"]["ff"], f"l{i}.mlp."
            t[q + "gate"], t[q + "up"], t[q + "down"] = lin(f, W, 2.0), lin(f, W, 2.0), lin(W, f)
    return t


def engine(d, W, backend, num_blocks=24, block_size=32, slots=4, **kw):
    dev, dt = backend
    model = FikeraxModel(FikeraxConfig.from_json(d, "test"), dev, dt, init=False)
    model.load_tensors(W.__getitem__)
    cfg = dict(model="test", device=dev, dtype=dt, num_blocks=num_blocks, block_size=block_size, state_slots=slots,
               max_batch_tokens=1024, use_graphs=False, temperature=0.0)
    cfg.update(kw)
    eng = LLMEngine(EngineConfig(**cfg), model=model)
    if eng.states is not None:
        for t in eng.states.t.values():       # a fresh slot must not be read: make a read loud
            t.fill_(float("nan"))
    for c in eng.kv.kc + [t for t in eng.kv.vc + eng.kv.vt if t is not None]:
        c.fill_(STALE)                        # stale pages hold finite garbage (a masked key's weight is 0)
    return eng


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def feed_all(eng, sid, tokens, cuts):
    """Feed ``tokens`` in portions ``cuts`` (the rest one by one); logits of every position."""
    out, at = [], 0
    for n in list(cuts) + [1] * len(tokens):
        if at >= len(tokens):
            break
        n = min(n, len(tokens) - at)
        out.append(eng.feed([(sid, tokens[at:at + n], list(range(n)))]))
        at += n
    return torch.cat(out)


def seg_meta(lens, pos0, slots, dev, block_tables=None, n_single=0):
    row0 = [0]
    for n in lens:
        row0.append(row0[-1] + n)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    row_seg = [s for s, n in enumerate(lens) for _ in range(n)]
    bt = i32(block_tables if block_tables is not None else [[0]] * len(lens))
    return S.SegMeta(len(lens), i32(row_seg), i32(row0), i32(pos0), i32(slots), bt, row0, list(pos0), list(slots),
                     n_single=n_single)


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=DT) * std


def b16(z):
    return z.to(torch.bfloat16).double()


def f32(z, dev):
    return None if z is None else z.float().to(dev)


def in_portions(fn, total, cuts):
    out, at = [], 0
    for n in list(cuts) + [total]:
        if at >= total:
            break
        e = min(total, at + n)
        out.append(fn(at, e))
        at = e
    return torch.cat(out)


def shuffled_pages(n, BS, seed):
    n_pages = -(-n // BS)
    return n_pages + 2, torch.randperm(n_pages + 2, generator=torch.Generator().manual_seed(seed)).tolist()[:n_pages]


def slots_of(order, BS, a, e, dev):
    p = torch.arange(a, e)
    return (torch.tensor(order)[p // BS] * BS + p % BS).to(torch.int32).to(dev)


# ------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("W", [6, 48, 300, 1024])
@pytest.mark.parametrize("streams", [1, 3, 5])
def test_residual_reads_the_embedding_output_again(backend, W, streams):
    """x + y (+ the embedding output), and the next sublayer's norm of it in the same pass; with one stream (the plain
    residual), with several."""
    dev, dt = backend
    T, eps, sc = 9, 1e-3, 3.5
    x, y = rnd(T, streams, W, seed=1, std=2.0), rnd(T, W, seed=2)
    emb = b16(rnd(20, W, seed=3))
    ids = torch.tensor([3, 19, 0, 3, 7, 7, 1, 2, 18], dtype=torch.int32, device=dev)
    nw, out, inn, mix = rnd(W, seed=4) + 1.0, rnd(streams, seed=5), rnd(streams, seed=6), rnd(streams, streams, seed=7)
    if streams == 1:
        out, inn, mix = torch.ones(1, dtype=DT), torch.ones(1, dtype=DT), torch.ones(1, 1, dtype=DT)
    for again in (True, False):
        X = f32(x, dev)
        h = N.hyper_step(X, f32(y, dev), f32(out, dev), f32(mix, dev), inn=f32(inn, dev), nw=f32(nw, dev), eps=eps,
                         out_dtype=dt, again=(ids, emb.to(dev).to(dt), sc) if again else None)
        want = torch.einsum("sr,tsw->trw", mix, x) + out[None, :, None] * y[:, None]
        if again:
            want = want + (emb[ids.cpu().long()] * sc)[:, None]
        close(X, want, torch.float32)
        close(h, O.unit_rms(torch.einsum("s,tsw->tw", inn, want), eps) * nw, dt)


@pytest.mark.parametrize("dims,base,sc", [
    (64, 20000.0, {"factor": 6.0, "low": 1.5, "high": 5.0, "original": 300}), (6, 300.0, STRETCH), (2, 10.0, STRETCH),
    (32, 5000.0, {"factor": 2.5, "low": 0.5, "high": 20.0, "original": 1000}),
    (16, 1e6, {"factor": 1.0, "low": 1.0, "high": 2.0, "original": 64}), (8, 77.0, None)])
def test_stretched_frequencies(dims, base, sc):
    """Short wavelengths kept, long ones divided, a mix between: all three kinds, and none at all."""
    rope = S.make_rope(dims, base, "cpu", stretch=tuple(sc[k] for k in ("factor", "low", "high", "original")) if sc else None)
    assert torch.allclose(rope.freq, torch.tensor(O.stretched(dims, base, sc), dtype=DT), rtol=1e-12) and rope.amp == 1.0
    if sc and dims == 32:
        plain = torch.tensor([base ** (-2.0 * i / dims) for i in range(16)], dtype=DT)
        ratio = rope.freq / plain
        assert float(ratio.max()) == 1.0 and abs(float(ratio.min()) - 1 / sc["factor"]) < 1e-9
        assert int(((ratio < 0.999) & (ratio > 1 / sc["factor"] + 1e-3)).sum()) > 2


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,G,D,V,rot", [(6, 3, 8, 10, 6), (3, 1, 6, 5, 6), (2, 2, 16, 16, 0), (5, 1, 70, 3, 32),
                                         (16, 2, 128, 128, 128), (4, 2, 64, 64, 32), (8, 1, 32, 64, 32), (4, 4, 256, 64, 64),
                                         (6, 3, 96, 96, 64), (2, 1, 64, 128, 4)])
@pytest.mark.parametrize("T", [9, 1100])
def test_preparation_with_biases_and_a_norm_behind_the_rotation(backend, H, G, D, V, rot, T):
    """Biases added, q and k rotated (entry i with i + rot / 2, stretched) and then divided by their root mean square;
    keys, values and the values' transposed twin in their pages, rows without a slot skipped."""
    dev, dt = backend
    if T > 100 and (H, G, D) not in ((16, 2, 128), (6, 3, 8)):
        pytest.skip("the long form at two sizes")
    BS, eps, base = 8, 1e-3, 777.0
    nq, nk, nv = H * D, G * D, G * V
    pos = torch.arange(T) + 70000 - 4
    pos[:3] = torch.arange(3)
    x, b = rnd(T, nq + nk + nv, seed=H + D, std=2.0), rnd(nq + nk + nv, seed=3)
    rd = {"dims": rot, "base": base, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 500}} if rot else None
    rope = S.make_rope(rot, base, dev, stretch=(4.0, 1.0, 3.0, 500.0)) if rot else None
    y = x + b

    def heads(z, n):
        z = z.reshape(T, n, D)
        return O.unit_rms(O.rotate_half(z, pos, rd) if rot else z, eps)

    n_pages, order = shuffled_pages(T, BS, 5)
    sl = slots_of(order, BS, 0, T, dev)
    sl[T - 2] = -1                                                       # a row without a slot
    kc = torch.full((n_pages, BS, nk), STALE, device=dev, dtype=dt)
    vc = torch.full((n_pages, BS, nv), STALE, device=dev, dtype=dt)
    vt = torch.full((n_pages, nv, BS), STALE, device=dev, dtype=dt)
    pd = pos.to(torch.int32).to(dev)
    got = S.attn_prep(f32(x, dev), f32(b, dev), H, G, D, V, pd, sl, kc, vc, dt, norm="head", eps=eps, rope=rope,
                      rope_cs=S.rope_table(pd, rope) if rot else None, vt=vt)
    close(got, heads(y[:, :nq], H).reshape(T, -1), dt)
    ok = (sl >= 0).cpu()
    so = sl.cpu().long()[ok]
    k, v = heads(y[:, nq:nq + nk], G).reshape(T, -1), y[:, nq + nk:]
    close(kc.view(-1, nk).cpu()[so], k[ok], dt)
    close(vc.view(-1, nv).cpu()[so], v[ok], dt)
    close(vt.cpu()[so // BS, :, so % BS], v[ok], dt)
    assert int((kc.view(-1, nk)[:, 0] == STALE).sum()) == n_pages * BS - T + 1     # nothing else written
    assert int((vt[:, 0] == STALE).sum()) == n_pages * BS - T + 1


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("QR,KR,R,pad,H,D", [(20, 12, 6, 32, 5, 8), (7, 3, 2, 2, 1, 1), (96, 64, 64, 64, 16, 128),
                                             (300, 520, 20, 32, 3, 5), (8, 16, 0, 0, 2, 4)])
def test_latent_rows_and_rotated_query_parts(backend, QR, KR, R, pad, H, D):
    dev, dt = backend
    T, BS, eps = 11, 8, 1e-3
    pos = torch.tensor([0, 1, 2, 3, 4, 5, 6, 7, 8, 90001, 90002])
    rd = {"dims": R, "base": 555.0, "scaling": YARN}
    dn, wq, wk = rnd(T, QR + KR + R + 3, seed=QR, std=3.0), b16(rnd(QR, seed=2) + 1.0), b16(rnd(KR, seed=3) + 1.0)
    pd = pos.to(torch.int32).to(dev)
    rope = S.make_rope(R, 555.0, dev, pairs=True, yarn=(3.0, 60, 6.0, 1.0)) if R else None
    cs = S.rope_table(pd, rope) if R else None
    n_pages, order = shuffled_pages(T, BS, 6)
    sl = slots_of(order, BS, 0, T, dev)
    cache = torch.full((n_pages, BS, KR + pad), STALE, device=dev, dtype=dt)
    ct = torch.full((n_pages, KR, BS), STALE, device=dev, dtype=dt)
    got = S.latent_norm(f32(dn, dev)[:, :QR + KR + R], wq.to(dev).to(dt), wk.to(dev).to(dt), sl, cache, QR, KR, eps, dt,
                        cache_t=ct, tail=R, tail_cs=cs)
    close(got, O.unit_rms(dn[:, :QR], eps) * wq, dt)
    c = O.unit_rms(dn[:, QR:QR + KR], eps) * wk
    rows = cache.view(-1, KR + pad).cpu()[sl.cpu().long()]
    close(rows[:, :KR], c, dt)
    close(ct.cpu()[sl.cpu().long() // BS, :, sl.cpu().long() % BS], c, dt)
    assert int((cache.view(-1, KR + pad)[:, 0] == STALE).sum()) == n_pages * BS - T
    if R:
        close(rows[:, KR:KR + R], O.rotate_pairs(dn[:, None, QR + KR:QR + KR + R], pos, rd)[:, 0], dt)
        assert float(rows[:, KR + R:].abs().sum()) == 0.0
        q = b16(rnd(T, H * (D + R), seed=9))
        qr = S.rotated_tail(q.to(dev).to(dt), cs, H, D, pad)
        close(qr[:, :, :R], O.rotate_pairs(q.view(T, H, D + R)[:, :, D:], pos, rd), dt)
        assert float(qr[:, :, R:].abs().sum()) == 0.0


def latent_case(dev, dt, H, R, P, n, BS, seed, sharp=None):
    """Random absorbed queries [n, H, R], rotated parts [n, H, P] and cache rows [R + P] of one sequence in shuffled
    pages.  ``sharp`` = (i, j): key j stands out for query i."""
    q, qr, c, kr = (b16(rnd(*s, seed=seed + k)) for k, s in enumerate(((n, H, R), (n, H, P), (n, R), (n, P))))
    if sharp is not None:
        i, j = sharp
        q[i], qr[i] = q[i, 0], qr[i, 0]                       # every head asks the same
        both = torch.cat([q[i, 0], qr[i, 0]])
        both = b16(40.0 * both / both.norm())
        c[j], kr[j] = both[:R], both[R:]
    n_pages, order = shuffled_pages(n, BS, seed)
    cache = torch.full((n_pages, BS, R + P), STALE, device=dev, dtype=dt)
    ct = torch.full((n_pages, R, BS), STALE, device=dev, dtype=dt)
    sl = slots_of(order, BS, 0, n, dev).long()
    cache.view(-1, R + P)[sl] = torch.cat([c, kr], 1).to(dev).to(dt)
    ct[sl // BS, :, sl % BS] = c.to(dev).to(dt)
    return q, qr, c, kr, cache, ct, [list(order)]


def latent_reference(q, qr, c, kr, scale, window, sink):
    n, H, R = q.shape
    out = torch.zeros(n, H, R, dtype=DT)
    for h in range(H):
        s = (q[:, h] @ c.T + qr[:, h] @ kr.T) * scale
        out[:, h] = O.weights_over_keys(s, O.visible(n, window), None if sink is None else sink[h]) @ c
    return out


def run_latent(dev, dt, q, qr, cache, ct, bt, a, e, scale, window, sink, n_single=0, mfma=False, head_major=True):
    sg = seg_meta([e - a], [a], [0], dev, bt, n_single=n_single)
    P = qr.shape[-1]
    kw = dict(window=window, sink=f32(sink, dev), head_major=head_major)
    if mfma:
        qd = q[a:e].to(dev).to(dt).transpose(0, 1).contiguous().transpose(0, 1) if head_major else q[a:e].to(dev).to(dt)
        pos = torch.arange(a, e, dtype=torch.int32, device=dev)
        return S.latent_attention_mfma(qd, cache, ct, None, sg, pos, scale,
                                       qr=qr[a:e].to(dev).to(dt).contiguous() if P else None, **kw)
    return S.latent_attention(f32(q[a:e], dev), cache, None, sg, scale, dt, qr=f32(qr[a:e], dev).contiguous() if P else None,
                              **kw)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,R,P,window,sink", [(5, 12, 32, 17, True), (1, 3, 2, 1, True), (6, 40, 0, 0, True),
                                               (3, 64, 32, 33, False), (20, 128, 32, 64, True), (2, 12, 6, 70, False)])
def test_latent_attention_with_a_shared_key_part(backend, H, R, P, window, sink):
    """Over shuffled pages, whole, in portions and token by token; windows of 1 to more than the sequence."""
    dev, dt = backend
    n, BS, scale = 75, 16, 0.2
    q, qr, c, kr, cache, ct, bt = latent_case(dev, dt, H, R, P, n, BS, seed=R + H)
    sk = rnd(H, seed=4) * 2.0 if sink else None
    want = latent_reference(q, qr, c, kr, scale, window, sk)
    for cuts in [(n,), (40, 1, 1, 2, 30), (3, 70)]:
        got = in_portions(lambda a, e: run_latent(dev, dt, q, qr, cache, ct, bt, a, e, scale, window, sk), n, cuts)
        close(got, want, dt)
    close(run_latent(dev, dt, q, qr, cache, ct, bt, 0, n, scale, window, sk, head_major=False), want, dt)


@pytest.mark.parametrize("backend", MFMA_BACKEND)
@pytest.mark.parametrize("H,R,P,window", [(6, 64, 32, 75), (16, 256, 64, 200), (3, 32, 32, 1), (1, 128, 0, 33), (24, 96, 32, 64),
                                          (5, 192, 64, 0), (40, 64, 64, 130), (7, 512, 32, 300), (2, 384, 64, 96)])
def test_latent_attention_on_the_matrix_cores(backend, H, R, P, window):
    """Prompt portions and decoding rows (their keys split over partitions) against the plain softmax; two sequences of
    unequal length in one step."""
    dev, dt = backend
    n, BS, scale = 330, 32, 2.0 * R ** -0.5
    assert S.mfma_tiles(R, dt, dev, P)
    q, qr, c, kr, cache, ct, bt = latent_case(dev, dt, H, R, P, n, BS, seed=R + H)
    sk = rnd(H, seed=4) * 2.0
    for sink in (sk, None):
        want = latent_reference(q, qr, c, kr, scale, window, sink)
        for cuts, single in [((n,), False), ((40, 1, 1, 2, 30, 17), False), ((300, 3, 9, 1), True), ((1, 64, 130), False)]:
            got = in_portions(lambda a, e: run_latent(dev, dt, q, qr, cache, ct, bt, a, e, scale, window, sink,
                                                      n_single=e - a if single and e - a < 20 else 0, mfma=True), n, cuts)
            close(got, want, dt)
    # a decoding row of one sequence (and a short portion as decoding rows) beside a portion of another
    sg = seg_meta([1, 3, 70], [n - 1, 200, 101], [0, 1, 2], dev, bt * 3, n_single=4)
    rows = torch.cat([torch.arange(n - 1, n), torch.arange(200, 203), torch.arange(101, 171)])
    got = S.latent_attention_mfma(q[rows].to(dev).to(dt), cache, ct, None, sg, rows.to(torch.int32).to(dev), scale,
                                  qr=qr[rows].to(dev).to(dt) if P else None, window=window, sink=f32(sk, dev))
    close(got, latent_reference(q, qr, c, kr, scale, window, sk)[rows], dt)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("aim", ["edge_in", "edge_out", "page_last", "page_first", "self", "future"])
@pytest.mark.parametrize("R,P,window", [(12, 32, 70), (64, 32, 64), (64, 32, 33), (256, 64, 150), (64, 32, 1)])
def test_one_latent_stands_out(backend, aim, R, P, window):
    """One key draws nearly all of query i's weight: just inside and just outside the window, at both sides of a page
    border, the query's own, the one behind it -- as part of a prompt, of a portion, decoded alone."""
    dev, dt = backend
    H, n, BS, i = 4, 302, 32, 300
    j = {"edge_in": i - window + 1, "edge_out": i - window, "page_last": 287, "page_first": 288, "self": i, "future": i + 1}[aim]
    seen = 0 <= i - j < window
    q, qr, c, kr, cache, ct, bt = latent_case(dev, dt, H, R, P, n, BS, seed=3, sharp=(i, j))
    sk = torch.zeros(H, dtype=DT)
    want = latent_reference(q, qr, c, kr, 0.5, window, sk)
    assert (float((want[i] - c[j]).abs().max()) < 0.2) == seen                   # the case is what its name says
    forms = [False] + ([True] if dev == "cuda" and dt == torch.bfloat16 and S.mfma_tiles(R, dt, dev, P) else [])
    for mfma in forms:
        for a, e, single in ((0, n, 0), (290, n, 0), (i, i + 1, 1), (i, i + 1, 0)):
            got = run_latent(dev, dt, q, qr, cache, ct, bt, a, e, 0.5, window, sk, n_single=single, mfma=mfma)
            close(got[i - a], want[i], dt)


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_sink_takes_its_share_once(backend):
    """Equal scores: n visible keys and a sink of the same score share the weight n : 1; a large sink takes all."""
    dev, dt = backend
    H, R, P, n = 3, 64, 32, 40
    q, qr, c, kr, cache, ct, bt = latent_case(dev, dt, H, R, P, n, 32, seed=8)
    q, qr = torch.zeros_like(q), torch.zeros_like(qr)
    for mfma in [False] + ([True] if dev == "cuda" and dt == torch.bfloat16 else []):
        for sink, share in ((0.0, 1.0), (math.log(5.0), 5.0), (40.0, None)):
            sk = torch.full((H,), sink, dtype=DT)
            for a, e, single in ((0, n, 0), (n - 1, n, 1)):
                got = run_latent(dev, dt, q, qr, cache, ct, bt, a, e, 1.0, 8, sk, n_single=single, mfma=mfma)
                want = c[n - 8:n].sum(0) / (8 + share) if share else torch.zeros(R, dtype=DT)
                assert float((got[-1].double().cpu() - want).abs().max()) < (1e-5 if dt == torch.float32 else 1e-2)


def masked_case(dev, dt, H, G, D, V, n, BS, seed, sharp=None):
    q, k, v = (b16(rnd(*s, seed=seed + i)) for i, s in enumerate(((n, H, D), (n, G, D), (n, G, V))))
    if sharp is not None:
        i, j = sharp
        q[i] = q[i, 0]
        k[j] = b16(8.0 * q[i, 0] / q[i, 0].norm())
    n_pages, order = shuffled_pages(n, BS, seed)
    kc = torch.full((n_pages, BS, G * D), STALE, device=dev, dtype=dt)
    vc = torch.full((n_pages, BS, G * V), STALE, device=dev, dtype=dt)
    vt = torch.full((n_pages, G * V, BS), STALE, device=dev, dtype=dt)
    sl = slots_of(order, BS, 0, n, dev).long()
    kc.view(-1, G * D)[sl] = k.reshape(n, -1).to(dev).to(dt)
    vc.view(-1, G * V)[sl] = v.reshape(n, -1).to(dev).to(dt)
    vt[sl // BS, :, sl % BS] = v.reshape(n, -1).to(dev).to(dt)
    return q, k, v, kc, vc, vt, [list(order)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("aim", ["edge_in", "edge_out", "page_first", "future"])
@pytest.mark.parametrize("H,G,D,V,window", [(6, 3, 8, 10, 70), (6, 2, 64, 64, 90), (4, 2, 128, 64, 33), (2, 1, 64, 64, 1)])
def test_one_key_stands_out_in_the_windowed_attention(backend, aim, H, G, D, V, window):
    dev, dt = backend
    n, BS, i = 302, 32, 300
    j = {"edge_in": i - window + 1, "edge_out": i - window, "page_first": 288, "future": i + 1}[aim]
    q, k, v, kc, vc, vt, bt = masked_case(dev, dt, H, G, D, V, n, BS, seed=5, sharp=(i, j))
    vis = O.visible(n, window)
    want = torch.stack([O.weights_over_keys(q[:, h] @ k[:, h // (H // G)].T, vis) @ v[:, h // (H // G)] for h in range(H)], 1)
    seen = 0 <= i - j < window
    assert (float((want[i] - v[j].repeat_interleave(H // G, 0)).abs().max()) < 0.2) == seen
    twin = vt if dev == "cuda" and dt == torch.bfloat16 and S.masked_mfma_ok(H, G, D, V, dt, dev) else None
    for a, e in ((0, n), (290, n), (i, i + 1)):
        got = S.masked_attention(q[a:e].reshape(e - a, -1).to(dev).to(dt).contiguous(), H, G, D, V, kc, vc,
                                 seg_meta([e - a], [a], [0], dev, bt), 1.0, window=window, vt=twin)
        close(got[i - a], want[i].reshape(-1), dt)


def decay_reference(x, H, D, V, decay, S0, silu, dt):
    T = x.shape[0]
    z = O.silu(x) if silu else x
    if silu and dt == torch.bfloat16:
        z = b16(z)                                                # the activations behind the projection are bfloat16
    q, k, v = z[:, :H * D].view(T, H, D), z[:, H * D:2 * H * D].view(T, H, D), z[:, 2 * H * D:].view(T, H, V)
    St, out = S0.clone(), torch.zeros(T, H, V, dtype=DT)
    for i in range(T):
        St = decay[:, None, None] * St + k[i][:, :, None] * v[i][:, None, :]
        out[i] = torch.einsum("hdv,hd->hv", St, q[i])
    return out.reshape(T, -1), St


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,D,V", [(3, 8, 12), (1, 1, 1), (4, 64, 64), (3, 128, 128), (2, 32, 48), (2, 96, 160), (5, 70, 33),
                                   (4, 128, 16), (2, 200, 40)])
@pytest.mark.parametrize("silu", [True, False])
def test_decaying_memory_across_portions_and_slots(backend, H, D, V, silu, monkeypatch):
    """Decays of 0 and 1 among them; the state in front of position 0 must not be read.  Portions on, before and behind
    the borders of the 64-token blocks; ranges of a portion in parallel and one after the other."""
    dev, dt = backend
    T = 330
    x = b16(rnd(T, H * (2 * D + V) + 4, seed=D))
    decay = torch.linspace(0.6, 0.999, H, dtype=DT).float().double()
    if H > 2:
        decay[0], decay[1] = 0.0, 1.0
    want, Sw = decay_reference(x[:, :-4], H, D, V, decay, torch.zeros(H, D, V, dtype=DT), silu, dt)
    xd = x.to(dev).to(dt)
    tol = torch.float32 if dt == torch.float32 else torch.bfloat16
    for fill, cuts in [(1 << 20, (T,)), (0, (T,)), (256, (64, 1, 1, 63, 200, 1)), (0, (130, 2, 17, 100)), (1 << 20, (2, 3, 1, 20, 304))]:
        monkeypatch.setattr(S, "LIN_GROUPS", fill)
        state = torch.full((3, H, D, V), float("nan"), device=dev)
        got = in_portions(lambda a, e: S.decay_attention(xd[a:e, :-4], H, D, V, f32(decay, dev), state,
                                                         seg_meta([e - a], [a], [1], dev), silu=silu), T, cuts)
        assert got.dtype == torch.float32
        close(got, want, tol, scale=3.0 if dt == torch.float32 else 0.15)
        close(state[1], Sw, tol, scale=3.0 if dt == torch.float32 else 0.15)
        assert bool(torch.isnan(state[0]).all()) and bool(torch.isnan(state[2]).all())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("D,V,fill", [(16, 24, 256), (64, 64, 1 << 20), (64, 64, 0), (128, 32, 1 << 20)])
def test_sequences_in_one_step_keep_their_own_memory(backend, D, V, fill, monkeypatch):
    """A long portion beside a short one and a single token, slots not in segment order: each gets what it gets alone."""
    dev, dt = backend
    monkeypatch.setattr(S, "LIN_GROUPS", fill)
    H, lens, pos0, slots = 3, [200, 3, 1, 65], [0, 5, 9, 64], [2, 0, 3, 1]
    T = sum(lens)
    x = b16(rnd(T, H * (2 * D + V), seed=1)).to(dev).to(dt)
    decay = torch.tensor([0.5, 0.9, 0.99], device=dev)
    start = rnd(4, H, D, V, seed=2).float().to(dev)
    together = start.clone()
    got = S.decay_attention(x, H, D, V, decay, together, seg_meta(lens, pos0, slots, dev), silu=True)
    at = 0
    for n, p0, sl in zip(lens, pos0, slots):
        alone = start.clone()
        w = S.decay_attention(x[at:at + n].contiguous(), H, D, V, decay, alone, seg_meta([n], [p0], [sl], dev), silu=True)
        close(got[at:at + n], w.double().cpu(), torch.float32, scale=5.0)
        close(together[sl], alone[sl].double().cpu(), torch.float32, scale=5.0)
        at += n


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("V", [12, 256, 1000, 2048, 6000])
def test_one_norm_over_the_heads_and_the_gate(backend, V):
    dev, dt = backend
    T, eps = 5, 1e-4
    o, g, w = rnd(T, V, seed=1, std=3.0), b16(rnd(T, V + 3, seed=2)), rnd(V, seed=3) + 1.0
    want = O.unit_rms(o, eps) * w * torch.sigmoid(g[:, 3:])
    for gate in (f32(g, dev), g.to(dev).to(torch.bfloat16)):
        close(S.head_norm_gate(f32(o, dev), gate[:, 3:], f32(w, dev), 1, V, eps, dt), want, dt)
    close(S.head_norm_gate(f32(o, dev), None, None, 1, V, eps, dt), O.unit_rms(o, eps), dt)


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("backend", BACKENDS)
def test_layers_match_after_every_run(backend):
    dev, dt = backend
    d = default_config()
    W = weights(d, 1)
    tokens = toks(45, d["vocab"], 2)
    want = []
    O.forward(W, d, tokens, want)
    eng = engine(d, W, backend)
    sid = eng.new_sequence()
    got = []
    fw = eng.model.forward
    eng.model.forward = lambda *a, **k: fw(*a, layers_out=got, **k)
    eng.feed([(sid, tokens, [])])
    assert len(got) == len(want) == 9
    for i, (g, w) in enumerate(zip(got, want)):
        e = float((g.double().cpu() - w).abs().max() / w.abs().max())
        assert e < (1e-5 if dt == torch.float32 else 0.03), (i, e)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cuts", [(), (70,), (30, 2, 2, 17, 3, 5), (69,), (1, 68), (2,) * 35])
def test_prefill_decode_and_portions_agree_with_oracle(backend, cuts):
    """() = token by token from the first token on; (70,) = one prefill; portions down to two tokens."""
    d = default_config()
    W = weights(d, 3)
    tokens = toks(70, d["vocab"], 4)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    got = feed_all(eng, eng.new_sequence(), tokens, cuts)
    assert agrees(got, want, backend[1]), row_errs(got, want).max()


@pytest.mark.parametrize("backend", BACKENDS)
def test_mixed_batches_equal_each_alone_and_reuse_pages_and_slots(backend):
    """Five requests of unequal length through three slots and a pool that cannot hold them all at once:
    portions of some beside single tokens of others; finished requests give pages and slots back."""
    d = default_config()
    W = weights(d, 5)
    lens = [50, 9, 33, 1, 64]
    reqs = [toks(n, d["vocab"], 10 + i) for i, n in enumerate(lens)]
    want = [O.forward(W, d, r) for r in reqs]
    eng = engine(d, W, backend, num_blocks=5, block_size=32, slots=3)
    got = [[] for _ in reqs]
    at = [0] * len(reqs)
    sid = {}
    plan = [[(0, 20), (1, 2)], [(0, 1), (1, 7), (2, 30)], [(0, 29), (2, 1)], [(2, 2), (3, 1)],       # 0, 1, 3 end
            [(4, 40)], [(4, 1), (2, 0)], [(4, 23)]]
    for step in plan:
        entries, who = [], []
        for i, n in step:
            if n == 0:
                continue
            if i not in sid:
                sid[i] = eng.new_sequence()
            entries.append((sid[i], reqs[i][at[i]:at[i] + n], list(range(n))))
            who.append((i, n))
            at[i] += n
        lg = eng.feed(entries)
        o = 0
        for i, n in who:
            got[i].append(lg[o:o + n])
            o += n
            if at[i] == lens[i]:
                eng.release_sequence(sid.pop(i))
    assert at == lens
    for i in range(len(reqs)):
        assert agrees(torch.cat(got[i]), want[i], backend[1]), i
    assert eng.kv.free_blocks == eng.kv.num_blocks and eng.states.free_slots == 3


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind", ["attention", "latent"])
@pytest.mark.parametrize("window,big", [(1, False), (33, False), (40, True), (64, True)])
def test_a_token_just_outside_the_window_does_not_matter(backend, kind, window, big):
    """One windowed layer: replacing the token window - 1 positions back moves the asker's logits, replacing the one
    before it does not; asked as part of a prompt, of a portion and decoded."""
    mix = (att(heads=2, kv_heads=1, dim=64, vdim=64, rot=64, window=window, scale=0.15) if big else att(window=window, scale=0.5)) \
        if kind == "attention" else \
        (lat(heads=4, dim=32, rot=16, vdim=32, kv_rank=64, window=window) if big else lat(window=window))
    d = config([(mix, 0)])
    W = weights(d, 6)
    i = 90
    base = toks(i + 1, d["vocab"], 7)
    for cuts in [(i + 1,), (60, i - 59), (i,)]:
        def ask(tokens):
            eng = engine(d, W, backend)
            return feed_all(eng, eng.new_sequence(), tokens, cuts)[i].double().cpu()
        ref = ask(base)
        assert agrees(ref[None], O.forward(W, d, base)[i:i + 1], backend[1])
        for back, seen in ((window, False), (window - 1, True)):
            other = list(base)
            other[i - back] = (other[i - back] + 101) % d["vocab"]
            moved = float((ask(other) - ref).abs().max() / ref.abs().max())
            assert (moved > 1e-4) if seen else (moved == 0.0), (back, moved, cuts)


@pytest.mark.parametrize("backend", BACKENDS)
def test_sharp_scores_over_page_borders(backend):
    """Large score scales: nearly all weight on one key, so a key lost at a page border or a sink left out shows in the
    logits.  Pages of 32."""
    d = config([(att(scale=9.0, window=60), 24), (lat(scale=3.0, window=50), 0), (att(scale=9.0, window=0, rot=8), 0)])
    W = weights(d, 6)
    tokens = toks(100, d["vocab"], 7)
    want = O.forward(W, d, tokens)
    for cuts in [(100,), (31, 2, 31, 15, 2, 17), (64,)]:
        eng = engine(d, W, backend)
        assert not eng.stateful and eng.states is None
        got = feed_all(eng, eng.new_sequence(), tokens, cuts)
        assert agrees(got, want, backend[1], mult=2.0 if backend[1] == torch.float32 else 3.5), (cuts, row_errs(got, want).max())


BIG = [(lig(heads=2, dim=64, vdim=64), 0), (att(heads=6, kv_heads=2, dim=64, vdim=64, rot=48, scale=0.3, window=90), 64),
       (lat(heads=5, dim=24, rot=20, vdim=40, q_rank=48, kv_rank=96, window=75), 56)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("layers,loop", [("small", (1, 4, 2)), ("matrix_cores", (1, 3, 2))])
def test_long_portions_then_decoding(backend, layers, loop):
    """Portions long enough for the parallel forms of the recurrence, cut off a block's border, then single tokens;
    far more tokens than any window."""
    d = default_config() if layers == "small" else config(BIG, width=64, loop=loop)
    W = weights(d, 17)
    tokens = toks(330, d["vocab"], 18)
    want = O.forward(W, d, tokens)
    for cuts in [(321,), (150, 2, 168), (63, 1, 64, 190)]:
        eng = engine(d, W, backend)
        got = feed_all(eng, eng.new_sequence(), tokens, cuts)
        assert agrees(got, want, backend[1], mult=1.5), (cuts, row_errs(got, want).max())


@pytest.mark.parametrize("backend", BACKENDS)
def test_first_tokens(backend):
    d = default_config()
    W = weights(d, 8)
    for n in (1, 2, 3):
        tokens = toks(n, d["vocab"], 20 + n)
        eng = engine(d, W, backend)
        assert agrees(feed_all(eng, eng.new_sequence(), tokens, (n,)), O.forward(W, d, tokens), backend[1], mult=1.5), n


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend):
    d = default_config()
    W = weights(d, 9)
    tokens = toks(150, d["vocab"], 10)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    got = feed_all(eng, eng.new_sequence(), tokens, (10,))           # 140 tokens one by one
    assert agrees(got, want, backend[1], mult=1.5)


OTHER = {
    "matrix_core_sizes": (BIG + [(lig(heads=3, dim=128, vdim=32), 128), (lat(heads=18, dim=16, rot=64, vdim=16, kv_rank=128, window=50), 0),
                                 (att(heads=3, kv_heads=1, dim=128, vdim=64, rot=32, scale=0.2, window=40), 0)], (2, 5, 2)),
    "one_head_everywhere": ([(lig(heads=1, dim=4, vdim=4, decay=[0.9]), 8), (att(heads=1, kv_heads=1, dim=4, vdim=4, rot=2), 8),
                             (lat(heads=1, dim=2, rot=2, vdim=2, q_rank=4, kv_rank=4), 8)], (0, 3, 2)),
    "windows_of_one_and_none": ([(att(window=1), 0), (lat(window=1), 16), (att(window=0), 0), (lat(window=0), 16)], None),
    "the_whole_stack_repeated": ([(lig(), 16), (lat(), 0)], (0, 2, 3)),
    "one_layer_repeated_at_the_end": ([(att(), 0), (lig(), 16)], (1, 2, 4)),
    "one_pass_only": ([(att(), 16), (lig(), 0), (lat(), 0)], (1, 2, 1)),
    "nothing_repeated": ([(att(), 16), (lig(), 0), (lat(), 0)], None),
    "no_scaling_of_frequencies": ([(att(scaling=None), 16), (lat(scaling=None), 0), (att(rot=0), 0), (att(rot=8), 0)], (1, 3, 2)),
    "unaligned_sizes": ([(lig(heads=3, dim=7, vdim=5), 13), (att(heads=5, kv_heads=1, dim=10, vdim=3, rot=6), 11),
                         (lat(heads=3, dim=5, rot=10, vdim=9, q_rank=7, kv_rank=11), 9), (lig(heads=5, dim=33, vdim=70), 0)], (1, 4, 2)),
    "decays_of_zero_and_one": ([(lig(heads=3, decay=[0.0, 1.0, 0.7]), 16), (lig(heads=2, dim=64, vdim=64, decay=[1.0, 0.25]), 0)], (0, 1, 2)),
    "constants_of_one": ([(lat(scale=1.0), 16), (att(scale=1.0, heads=3, kv_heads=3), 0)], (0, 2, 2)),
}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(backend, name):
    layers, loop = OTHER[name]
    d = config(layers, width={"unaligned_sizes": 34, "matrix_core_sizes": 64}.get(name, 40), eps=1e-3, loop=loop,
               scale=1.0 if name == "constants_of_one" else 5.0)
    W = weights(d, 11)
    tokens = toks(60, d["vocab"], 12)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    got = feed_all(eng, eng.new_sequence(), tokens, (13, 2, 33))
    assert agrees(got, want, backend[1], mult=1.5), row_errs(got, want).max()


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("stateful", [True, False])
def test_greedy_generation_through_submit_and_scheduler(backend, stateful):
    """``submit`` + ``step``: the scheduler's own batching (two prompts of unequal length, then decode rows)
    must produce the oracle's greedy continuation; a model of attention layers alone has no state slots and runs its
    steps overlapped."""
    d = default_config(vocab=8192) if stateful else config([(att(), 24), (lat(), 0)], vocab=8192, loop=(0, 2, 2))
    W = weights(d, 13)
    eng = engine(d, W, backend, num_blocks=16)
    assert eng.stateful == stateful
    prompts = [toks(37, 2000, 14), toks(6, 2000, 15)]
    outs = {}
    for i, p in enumerate(prompts):
        eng.submit(eng.new_sequence(), p, None, 6, temperature=0.0, on_done=lambda g, st, i=i: outs.__setitem__(i, g))
    eng.run_until_idle()
    for i, p in enumerate(prompts):
        seq, same = list(p), 0
        for t in outs[i][:6]:
            lg = O.forward(W, d, seq)[-1, :eng.vocab]
            if backend[1] == torch.float32:
                assert t == int(lg.argmax()), i
            else:       # bf16: the chosen token is among the best few of thousands, and mostly the best
                assert int((lg > lg[t]).sum()) < 8, i
                same += t == int(lg.argmax())
            seq.append(t)
        assert len(outs[i]) >= 6 and (backend[1] == torch.float32 or same >= 4)


def test_config_round_trip_registry_and_replay(tmp_path):
    """config.json -> configuration -> config.json; the registry picks the class by the file; a recorded
    schedule replayed through the engine gives the oracle's logits."""
    from k8s_llm_rca_amd.engine import trace as TR
    from k8s_llm_rca_amd.models import fikerax as FK
    from k8s_llm_rca_amd.models.registry import checkpoint_arch, get_any_config, load_model
    d = default_config()
    cfg = FikeraxConfig.from_json(d, "x")
    assert FikeraxConfig.from_json(cfg.to_json(), "x") == cfg and cfg.n_layers == 9
    assert get_any_config("tiny-fikerax").arch == "fikerax"
    tiny = FikeraxModel(get_any_config("tiny-fikerax"), "cpu", torch.float32)
    assert tiny.weight_bytes() > 0 and len(tiny.state_spec()) == 4 and len(tiny.cached) == 4
    W = weights(d, 21)
    path = str(tmp_path / "ckpt")
    FK.save_checkpoint(cfg, W, path)
    assert checkpoint_arch(path) == "fikerax"
    assert isinstance(load_model(path, "cpu", torch.float32), FikeraxModel)
    eng = TR.make_engine(path, torch.float32, 128, device="cpu", state_slots=2, block_size=32)
    a, b = toks(40, d["vocab"], 22), toks(21, d["vocab"], 23)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[30:31], "want": [0]}, {"id": "b", "tokens": b[:20], "want": []}],
              "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[20:], "want": [0]}, {"id": "a", "tokens": a[31:], "want": [8]}],
              "end": ["a", "b"]}]
    out = str(tmp_path / "out")
    log = io.StringIO()
    TR.replay(eng, io.StringIO("\n".join(json.dumps(s) for s in steps)), out, log)
    assert log.getvalue().split() == ["done", "0", "done", "1", "done", "2"]
    wa, wb = O.forward(W, d, a), O.forward(W, d, b)
    g0 = torch.from_numpy(np.fromfile(os.path.join(out, "0.f32"), dtype="<f4").reshape(2, -1))
    g2 = torch.from_numpy(np.fromfile(os.path.join(out, "2.f32"), dtype="<f4").reshape(2, -1))
    assert agrees(g0, wa[[0, 29]], torch.float32) and agrees(g2, torch.stack([wb[20], wa[39]]), torch.float32)
    assert eng.kv.free_blocks == eng.kv.num_blocks and eng.states.free_slots == 2


def test_bad_configurations_are_refused():
    bad_rot = lat()
    bad_rot["mixer"]["rot"]["dims"] = 4
    for layers, loop in (([(att(heads=5, kv_heads=2), 0)], None), ([(att(rot=5), 0)], None), ([(att(rot=10), 0)], None),
                         ([(lat(rot=5), 0)], None), ([(bad_rot, 0)], None), ([(lig(heads=2, decay=[0.5]), 0)], None),
                         ([(lig(heads=1, decay=[1.5]), 0)], None), ([(lig(), 0)], (0, 2, 2)), ([(lig(), 0)], (0, 1, 0)),
                         ([({"type": "other", "mixer": {}}, 0)], None)):
        with pytest.raises(ValueError):
            FikeraxModel(FikeraxConfig.from_json(config(layers, loop=loop), "bad"), "cpu", torch.float32, init=False)


def test_trace_run_command_line(tmp_path):
    from k8s_llm_rca_amd.models import fikerax as FK
    d = default_config()
    W = weights(d, 31)
    path = str(tmp_path / "ckpt")
    FK.save_checkpoint(FikeraxConfig.from_json(d, "x"), W, path)
    tokens = toks(12, d["vocab"], 32)
    step = json.dumps({"step": 0, "entries": [{"id": "r", "tokens": tokens, "want": [11]}], "end": ["r"]})
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(tmp_path / "o"), "--max-tokens", "64", "--device", "cpu"], input=step + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0 and "done 0" in r.stdout, r.stderr[-2000:]
    got = torch.from_numpy(np.fromfile(str(tmp_path / "o" / "0.f32"), dtype="<f4").reshape(1, -1))
    assert agrees(got, O.forward(W, d, tokens)[-1:], torch.float32)
