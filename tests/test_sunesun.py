"""Sunesun through the engine against the plain implementation in ``sunesun_oracle.py``:
each mechanism alone, prefill against token-by-token decoding, portions, mixed batches,
reuse and sharing of pages, far keys, page borders and window edges, the first tokens of a
sequence, long decoding, other sizes, and greedy generation through ``submit`` / ``step``.

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

import sunesun_oracle as O
from k8s_llm_rca_amd.engine.engine import EngineConfig, LLMEngine
from k8s_llm_rca_amd.models.sunesun import SunesunConfig, SunesunModel
from k8s_llm_rca_amd.ops import moe as M
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
    """Logits rows against the oracle's: a wrong key, a window one token off or a wrong expert moves a row by 1e-2 and
    more in fp32 terms (the sharp check).  bf16: every sublayer adds its rounding (a few 1e-3 of a row); a router's
    near-tie that goes the other way would move a row a lot, so the bf16 runs use :func:`weights` with clear choices."""
    e = row_errs(got, want)
    print("row errors: median %.2e, 85%% %.2e, largest %.2e" % tuple(float(e.quantile(q)) for q in (0.5, 0.85, 1.0)))
    if dtype == torch.float32:
        return float(e.max()) < 1e-5 * mult
    return float(e.median()) < 0.02 * mult and float(e.max()) < 0.1 * mult


def close(got, want, dtype, scale=1.0):
    """Element-wise check of an op's output against fp64."""
    got, want = got.double().cpu(), want.double().cpu()
    t = (2e-5 if dtype == torch.float32 else 2e-2) * scale
    err = float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))
    assert err < t, err


# ------------------------------------------------------------------ configurations and weights
YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def att(heads=6, kv_heads=3, dim=8, scale=None, cap=9.0, window=21, rot=4, base=300.0, yarn=YARN):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale}
    if cap:
        m["softcap"] = cap
    if window:
        m["mask"] = {"size": window}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
        if yarn:
            m["rot"]["scaling"] = dict(yarn)
    return m


def moe(ff=20, experts=12, top=3, count=4, keep=2):
    r = {"experts": experts, "top": top}
    if count:
        r["groups"] = {"count": count, "keep": keep}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def config(layers, width=48, vocab=512, eps=1e-5, streams=3, mult=0.4, scale=5.0):
    """``layers``: (mixer, feed-forward) of a layer with tensors, or the index of the layer whose tensors it runs."""
    out = []
    for i, L in enumerate(layers):
        if isinstance(L, int):
            out.append(dict(json.loads(json.dumps(out[L])), weights_of=L))
        else:
            out.append({"type": "attention", "mixer": L[0], "mlp": L[1]})
    d = {"architecture": "Sunesun", "vocab": vocab, "width": width, "layers": out, "norm": {"eps": eps},
         "embedding": {"scale": scale}, "residual_mult": mult}
    if streams:
        d["streams"] = streams
    return d


def default_config(**kw):
    return config([(att(), moe()), (att(heads=4, kv_heads=1, dim=12, window=33, rot=12, cap=4.0), moe(experts=6, top=1, count=3)),
                   0, (att(window=0, yarn=None, rot=8), None), 1, 0], **kw)


CLASSES = 6


def weights(d, seed=0, clear=False):
    """Random weights under the checkpoint's names, rounded to bfloat16.  ``clear``: the routers read nothing but the
    token's class (token % CLASSES, in residual entries that no sublayer writes) and rank the experts in even steps,
    so rounding does not turn a choice over."""
    g = torch.Generator().manual_seed(seed)
    W, n = d["width"], d.get("streams", 0)

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    def lin(o, i, mul=1.0):
        return r(o, i, std=mul * i ** -0.5)

    t = {"embed": r(d["vocab"], W, std=0.3), "head": lin(d["vocab"], W), "final.norm": r(W, std=0.2, mean=1.0)}
    for i, L in enumerate(d["layers"]):
        if "weights_of" in L:
            continue
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        t[p + "mix.q"], t[p + "mix.k"] = lin(m["heads"] * m["dim"], W, 1.5), lin(m["kv_heads"] * m["dim"], W, 1.5)
        t[p + "mix.o"] = lin(W, m["heads"] * m["dim"])
        for q in ("1", "2") if f is not None else ("1",):
            t[p + "norm" + q] = r(W, std=0.2, mean=1.0)
            if n:
                t[f"{p}hc{q}.in"], t[f"{p}hc{q}.out"] = r(n, std=0.4, mean=0.5), r(n, std=0.5, mean=1.0)
                t[f"{p}hc{q}.mix"] = r(n, n, std=0.3) + torch.eye(n) * 0.75
        if f is not None:
            t[p + "mlp.router"] = lin(f["router"]["experts"], W, 2.0)
            for e in range(f["router"]["experts"]):
                t[f"{p}mlp.e{e}.up"], t[f"{p}mlp.e{e}.down"] = lin(f["expert"]["ff"], W), lin(W, f["expert"]["ff"])
    if clear:
        C = CLASSES
        t["embed"][:, :C] = torch.nn.functional.one_hot(torch.arange(d["vocab"]) % C, C) * 0.6
        for k in t:
            if k.endswith((".mix.o", ".down")):
                t[k][:C] = 0.0
            elif k.endswith(".router"):
                E = t[k].shape[0]
                r = d["layers"][int(k[1:k.index(".")])]["mlp"]["router"]
                ng = r.get("groups", {}).get("count", 1)
                t[k].zero_()
                for c in range(C):                 # a group's experts hold neighbouring ranks
                    rank = torch.cat([q * (E // ng) + torch.randperm(E // ng, generator=g)
                                      for q in torch.randperm(ng, generator=g).tolist()])
                    t[k][:, c] = torch.linspace(-1.2, 1.3, E)[rank] if E > 1 else 0.5
    return {k: v.to(torch.bfloat16).float() for k, v in t.items()}


def engine(d, W, backend, num_blocks=24, block_size=32, **kw):
    dev, dt = backend
    model = SunesunModel(SunesunConfig.from_json(d, "test"), dev, dt, init=False)
    model.load_tensors(W.__getitem__)
    cfg = dict(model="test", device=dev, dtype=dt, num_blocks=num_blocks, block_size=block_size,
               max_batch_tokens=1024, use_graphs=False, temperature=0.0)
    cfg.update(kw)
    eng = LLMEngine(EngineConfig(**cfg), model=model)
    assert eng.states is None             # pages hold everything
    for c in eng.kv.kc + eng.kv.vc + eng.kv.vt:
        if c is not None:
            c.fill_(STALE)                # stale pages hold finite garbage (a masked key's weight is 0)
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


def seg_meta(lens, pos0, dev, block_tables):
    row0 = [0]
    for n in lens:
        row0.append(row0[-1] + n)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
    row_seg = [s for s, n in enumerate(lens) for _ in range(n)]
    z = [0] * len(lens)
    return S.SegMeta(len(lens), i32(row_seg), i32(row0), i32(pos0), i32(z), i32(block_tables), row0, list(pos0), z,
                     n_single=0)


def rnd(*shape, seed=0, std=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=DT) * std


def f32(z, dev):
    return None if z is None else z.float().to(dev)


def b16(*shape, seed=0, std=1.0):
    """Random numbers that bfloat16 holds exactly, in float64."""
    return rnd(*shape, seed=seed, std=std).to(torch.bfloat16).double()


# ------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("W", [6, 48, 301, 1028, 2048])
def test_streams(backend, n, W):
    """The streams from the embedding, one step with a plain sublayer output, one with the experts' rows joined on the
    way in, one that nothing reads, and the sum at the end; mix is [from][to] and uses the old streams only."""
    dev, dt = backend
    T, eps, K = 5, 1e-3, 3
    emb, nw, inn = b16(20, W, seed=1), rnd(W, seed=2) + 1.0, rnd(n, seed=3) + 0.5
    out, mix = rnd(n, seed=4), rnd(n, n, seed=5)
    ids = torch.tensor([3, 19, 0, 3, 7], dtype=torch.int32)
    x = torch.full((T, n, W), float("nan"), device=dev)
    h = N.hyper_embed(ids.to(dev), emb.to(dev).to(dt), 7.0, x, f32(inn, dev), f32(nw, dev), eps, dt)
    x0 = (emb[ids.long()] * 7.0)[:, None].repeat(1, n, 1)
    close(x, x0, torch.float32)
    close(h, O.unit_rms(torch.einsum("s,tsw->tw", inn, x0), eps) * nw, dt)
    xs, y = rnd(T, n, W, seed=6, std=2.0), rnd(T, W, seed=7, std=3.0)
    new = torch.einsum("sr,tsw->trw", mix, xs) + out[None, :, None] * y[:, None]
    want = O.unit_rms(torch.einsum("s,tsw->tw", inn, new), eps) * nw
    x = f32(xs, dev)
    h = N.hyper_step(x, f32(y, dev), f32(out, dev), f32(mix, dev), inn=f32(inn, dev), nw=f32(nw, dev), eps=eps, out_dtype=dt)
    close(x, new, torch.float32)
    close(h, want, dt)
    x = f32(xs, dev)
    assert N.hyper_step(x, f32(y, dev), f32(out, dev), f32(mix, dev)) is None
    close(x, new, torch.float32)
    yp, ew = b16(T * K, W, seed=8, std=2.0), rnd(T, K, seed=9)
    inv = torch.randperm(T * K, generator=torch.Generator().manual_seed(1)).to(torch.int32)
    y = (yp[inv.long()].view(T, K, W) * ew[:, :, None]).sum(1)
    new = torch.einsum("sr,tsw->trw", mix, xs) + out[None, :, None] * y[:, None]
    x = f32(xs, dev)
    h = N.hyper_step(x, yp.to(dev).to(dt), f32(out, dev), f32(mix, dev), experts=(inv.to(dev), f32(ew, dev)), inn=f32(inn, dev),
                     nw=f32(nw, dev), eps=eps, out_dtype=dt)
    close(x, new, torch.float32)
    close(h, O.unit_rms(torch.einsum("s,tsw->tw", inn, new), eps) * nw, dt)
    rows = torch.tensor([4, 0, 4])
    close(N.hyper_read(f32(xs, dev), rows.to(dev), f32(nw, dev), eps, dt), O.unit_rms(xs[rows].sum(1), eps) * nw, dt)
    close(N.hyper_read(f32(xs, dev), None, f32(nw, dev), eps, dt, inn=f32(inn, dev)),
          O.unit_rms(torch.einsum("s,tsw->tw", inn, xs), eps) * nw, dt)


@pytest.mark.parametrize("backend", BACKENDS)
def test_streams_of_many_rows(backend):
    """Enough rows for the narrower workgroups of prompts."""
    dev, dt = backend
    T, n, W, eps = 300, 4, 1032, 1e-5
    xs, y, mix, out = rnd(T, n, W, seed=1), rnd(T, W, seed=2), rnd(n, n, seed=3), rnd(n, seed=4)
    nw, inn = rnd(W, seed=5), rnd(n, seed=6)
    new = torch.einsum("sr,tsw->trw", mix, xs) + out[None, :, None] * y[:, None]
    x = f32(xs, dev)
    h = N.hyper_step(x, f32(y, dev), f32(out, dev), f32(mix, dev), inn=f32(inn, dev), nw=f32(nw, dev), eps=eps, out_dtype=dt)
    close(x, new, torch.float32)
    close(h, O.unit_rms(torch.einsum("s,tsw->tw", inn, new), eps) * nw, dt)


ROPES = [(8, 300.0, None), (4, 300.0, YARN), (64, 500000.0, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}),
         (2, 50.0, YARN),                                                               # one pair
         (16, 100.0, {"factor": 3.0, "original": 40, "fast": 1.0, "slow": 1.0}),       # both borders in one step
         (32, 1e4, {"factor": 16.0, "original": 8, "fast": 64.0, "slow": 2.0}),        # borders below 0
         (12, 10.0, {"factor": 2.0, "original": 100000, "fast": 30.0, "slow": 0.001}),  # borders past the last pair
         (8, 300.0, {"factor": 1.0, "original": 64, "fast": 8.0, "slow": 1.0})]


@pytest.mark.parametrize("backend", BACKENDS[:2])
@pytest.mark.parametrize("dims,base,sc", ROPES)
def test_rotation_table(backend, dims, base, sc):
    dev = backend[0]
    yarn = tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None
    r = S.make_rope(dims, base, dev, pairs=True, yarn=yarn)
    f, amp = O.yarn(dims, base, sc)
    assert torch.allclose(r.freq.cpu(), f, rtol=1e-12) and abs(r.amp - amp) < 1e-12
    pos = torch.tensor([0, 1, 2, 31, 4095, 70001, 1000003], dtype=torch.int32)
    a = pos.double()[:, None] * f[None]
    cs = S.rope_table(pos.to(dev), r)
    assert float((cs.double().cpu() - amp * torch.cat([a.cos(), a.sin()], 1)).abs().max()) < 1e-6 * amp


def slots_of(order, BS, a, e, dev):
    p = torch.arange(a, e)
    return (torch.tensor(order)[p // BS] * BS + p % BS).to(torch.int32).to(dev)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,G,D,rot,lo,T,twin", [(6, 3, 8, 4, 0, 9, True), (3, 3, 6, 6, 1, 9, True), (2, 1, 16, 0, 0, 9, False),
                                                 (5, 1, 70, 32, 0, 9, True), (16, 2, 128, 64, 0, 9, True), (4, 2, 12, 2, 0, 40, False),
                                                 (4, 2, 16, 6, 3, 1100, True), (2, 2, 8, 8, 0, 1093, False)])
@pytest.mark.parametrize("table", [True, False])
def test_preparation_rotates_neighbouring_pairs(backend, H, G, D, rot, lo, T, twin, table):
    """Entries 2i and 2i + 1 turn together; the values are the keys in front of the rotation.  Rows at column offset
    ``lo`` of something wider (unaligned too), tokens whose slots are not in a row, rows without a slot, values in
    both layouts or in the transposed one alone."""
    dev, dt = backend
    BS = 32
    x = rnd(T, lo + (H + G) * D + 4 - (lo + (H + G) * D) % 4, seed=H + D, std=2.0)
    pos = torch.arange(T) + 70001
    rope = S.make_rope(rot, 777.0, dev, pairs=True, yarn=(4.0, 64.0, 8.0, 1.0)) if rot else None
    orot = {"dims": rot, "base": 777.0, "scaling": YARN} if rot else None
    order = torch.randperm(-(-T // BS) + 2, generator=torch.Generator().manual_seed(3)).tolist()
    sl = slots_of(order, BS, 0, T, dev)
    sl[2] = -1
    if T > 20:
        sl[12:14] = sl[12:14].flip(0)
    n_pages = len(order)
    kc = torch.full((n_pages, BS, G * D), STALE, device=dev, dtype=dt)
    vc = None if twin and table else torch.full((n_pages, BS, G * D), STALE, device=dev, dtype=dt)
    vt = torch.full((n_pages, G * D, BS), STALE, device=dev, dtype=dt) if twin else None
    p32 = pos.to(torch.int32).to(dev)
    got = S.attn_prep(f32(x, dev)[:, lo:lo + (H + G) * D], None, H, G, D, D, p32, sl, kc, vc, dt, rope=rope, vt=vt,
                      v_is_k=True, rope_cs=S.rope_table(p32, rope) if rope is not None and table else None)
    q, k = x[:, lo:lo + H * D].view(T, H, D), x[:, lo + H * D:lo + (H + G) * D].view(T, G, D)
    close(got, O.rotate(q, pos, orot).reshape(T, -1), dt)
    ok = sl >= 0
    s = sl[ok].long()
    okc = ok.cpu()
    close(kc.view(-1, G * D)[s], O.rotate(k, pos, orot).reshape(T, -1)[okc], dt)
    if vc is not None:
        close(vc.view(-1, G * D)[s], k.reshape(T, -1)[okc], dt)
    if vt is not None:
        close(vt[s // BS, :, s % BS], k.reshape(T, -1)[okc], dt)
        assert int((vt == STALE).sum()) >= (n_pages * BS - T + 1) * G * D - 8            # nothing else written
    assert int((kc == STALE).sum()) >= (n_pages * BS - T + 1) * G * D - 8


def attention_case(dev, dt, H, G, D, n, BS, seed, sharp=None, twin=False):
    """Random q and keys (= values) for one sequence in shuffled pages.  ``sharp`` = (i, j): key j stands out for
    query i."""
    q, k, v = rnd(n, H, D, seed=seed), rnd(n, G, D, seed=seed + 1), rnd(n, G, D, seed=seed + 2)
    if sharp is not None:
        i, j = sharp
        q[i] = q[i, 0] / q[i, 0].norm() * 6.0
        k[j] = q[i, 0]
    q, k, v = (z.to(torch.bfloat16).double() for z in (q, k, v))
    n_pages = -(-n // BS)
    order = torch.randperm(n_pages + 2, generator=torch.Generator().manual_seed(seed)).tolist()[:n_pages]
    sl = slots_of(order, BS, 0, n, dev).long()
    kc = torch.full((n_pages + 2, BS, G * D), STALE, device=dev, dtype=dt)
    kc.view(-1, G * D)[sl] = k.reshape(n, -1).to(dev).to(dt)
    vc = vt = None
    if twin:
        vt = torch.full((n_pages + 2, G * D, BS), STALE, device=dev, dtype=dt)
        vt[sl // BS, :, sl % BS] = v.reshape(n, -1).to(dev).to(dt)
    else:
        vc = torch.full((n_pages + 2, BS, G * D), STALE, device=dev, dtype=dt)
        vc.view(-1, G * D)[sl] = v.reshape(n, -1).to(dev).to(dt)
    return q, k, v, kc, vc, vt, [list(order)]


def run_cuts(q, H, G, D, kc, vc, vt, bt, cuts, scale, cap, window, dev):
    n, at, out = q.shape[0], 0, []
    for c in list(cuts) + [n]:
        if at >= n:
            break
        e = min(n, at + c)
        out.append(S.masked_attention(q[at:e].contiguous(), H, G, D, D, kc, vc, seg_meta([e - at], [at], dev, bt), scale,
                                      softcap=cap, window=window, vt=vt))
        at = e
    return torch.cat(out)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("H,G,D,cap,window", [(4, 2, 8, 3.0, 11), (3, 3, 5, 0.0, 1), (6, 1, 32, 5.0, 0), (2, 2, 70, 2.0, 75),
                                              (9, 3, 96, 4.0, 33), (4, 2, 64, 4.0, 16), (4, 4, 128, 0.0, 17)])
def test_window_and_cap_over_shuffled_pages(backend, H, G, D, cap, window):
    dev, dt = backend
    n, BS, scale = 77, 16, 0.6
    q, k, v, kc, vc, _, bt = attention_case(dev, dt, H, G, D, n, BS, seed=H + D)
    want = O.attend(q, k, v, scale, cap, window).reshape(n, -1)
    for cuts in [(n,), (40, 1, 1, 2, 30), (3, 70), (2,) * 38]:
        close(run_cuts(q.reshape(n, -1).to(dev).to(dt), H, G, D, kc, vc, None, bt, cuts, scale, cap, window, dev), want, dt)


@pytest.mark.parametrize("backend", MFMA_BACKEND)
@pytest.mark.parametrize("H,G,D,cap,window", [(9, 3, 96, 4.0, 100), (6, 6, 96, 0.0, 31), (4, 2, 64, 3.0, 32), (3, 1, 128, 5.0, 129),
                                              (10, 2, 96, 2.0, 1), (8, 2, 128, 5.0, 0)])
@pytest.mark.parametrize("split", [True, False])
def test_window_and_cap_on_the_matrix_cores(backend, H, G, D, cap, window, split, monkeypatch):
    """Values in the transposed pages alone; tiles of 16 tokens, portions that start inside a tile's span, single
    tokens, with and without the split of a tile's key blocks over workgroups; two sequences in a step."""
    dev, dt = backend
    if not split:
        monkeypatch.setattr(S, "WINDOW_SPLIT_ITEMS", 0)
    n, BS, scale = 330, 32, 0.3
    q, k, v, kc, vc, vt, bt = attention_case(dev, dt, H, G, D, n, BS, seed=H + D, twin=True)
    assert S.masked_mfma_ok(H, G, D, D, dt, dev) and vc is None
    want = O.attend(q, k, v, scale, cap, window).reshape(n, -1)
    qd = q.reshape(n, -1).to(dev).to(dt)
    for cuts in [(n,), (40, 1, 1, 2, 30, 17), (3, 270), (319,) + (1,) * 11]:
        close(run_cuts(qd, H, G, D, kc, vc, vt, bt, cuts, scale, cap, window, dev), want, dt)
    got = S.masked_attention(torch.cat([qd[n - 5:], qd[100:]]).contiguous(), H, G, D, D, kc, vc,
                             seg_meta([5, n - 100], [n - 5, 100], dev, bt + bt), scale, softcap=cap, window=window, vt=vt)
    close(got, torch.cat([want[n - 5:], want[100:]]), dt)


@pytest.mark.parametrize("backend", MFMA_BACKEND)
@pytest.mark.parametrize("n_seq,window", [(40, 100), (100, 0), (140, 100)])
def test_many_decoding_sequences_on_the_matrix_cores(backend, n_seq, window):
    """Single tokens of many sequences in one step (their key blocks split over workgroups up to a point), each at
    another position."""
    dev, dt = backend
    H, G, D, n, BS = 4, 2, 128, 330, 32
    q, k, v, kc, vc, vt, bt = attention_case(dev, dt, H, G, D, n, BS, seed=5, twin=True)
    want = O.attend(q, k, v, 0.3, 5.0, window).reshape(n, -1)
    at = [(37 * i + 5) % n for i in range(n_seq)]
    got = S.masked_attention(q.reshape(n, -1)[at].to(dev).to(dt).contiguous(), H, G, D, D, kc, vc,
                             seg_meta([1] * n_seq, at, dev, bt * n_seq), 0.3, softcap=5.0, window=window, vt=vt)
    close(got, want[at], dt)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("window,aim", [(0, 1), (70, "in"), (70, "out"), (33, "in"), (33, "out"), (64, "in"), (64, "out"),
                                        (1, "in"), (1, "out"), (0, 255), (0, 256), (0, 301)])
@pytest.mark.parametrize("D", [16, 96, 128])
def test_one_key_stands_out(backend, window, aim, D):
    """One key draws nearly all of query i's weight, so the output shows at once whether it was seen: just inside and
    just outside the window, far back, at both sides of a page border, behind the query.  Query 300 as part of the
    whole prompt, of a portion, and decoded alone."""
    dev, dt = backend
    H, G, n, BS, i = 4, 2, 302, 32, 300
    j = aim if isinstance(aim, int) else i - window + (1 if aim == "in" else 0)
    twin = dt == torch.bfloat16 and D >= 64
    q, k, v, kc, vc, vt, bt = attention_case(dev, dt, H, G, D, n, BS, seed=3, sharp=(i, j), twin=twin)
    want = O.attend(q, k, v, 1.0, 30.0, window)
    seen = float((want[i] - v[j].repeat_interleave(H // G, 0)).abs().max()) < 0.2
    assert seen == (aim != "out" and j <= i)                             # the case is what its name says
    qd = q.reshape(n, -1).to(dev).to(dt)
    for a, e in ((0, n), (290, n), (i, i + 1)):
        got = S.masked_attention(qd[a:e].contiguous(), H, G, D, D, kc, vc, seg_meta([e - a], [a], dev, bt), 1.0, softcap=30.0,
                                 window=window, vt=vt)
        close(got[i - a], want[i].reshape(-1), dt)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("E,top,count,keep,W,T", [(12, 3, 4, 2, 48, 9), (20, 3, 5, 3, 192, 9), (6, 1, 3, 1, 20, 9), (8, 8, 2, 2, 64, 9),
                                                  (5, 2, 5, 3, 7, 9), (64, 6, 8, 4, 512, 33), (256, 8, 8, 3, 128, 17),
                                                  (130, 5, 65, 20, 96, 9), (16, 4, 4, 2, 512, 700), (9, 4, 0, 0, 64, 9),
                                                  (12, 6, 1, 1, 32, 3), (32, 4, 4, 2, 2048, 40)])
def test_router_chooses_groups_first(backend, E, top, count, keep, W, T):
    """Sigmoid scores, the best groups by the sum of their two largest, the top experts inside them; the weights are
    the scores.  On the device in bf16 most of these run on the matrix cores."""
    dev, dt = backend
    h, wr = b16(T, W, seed=E), b16(E, W, seed=2, std=2.0 * W ** -0.5)
    w, ids = M.route_direct(h.to(dev).to(dt), wr.to(dev).to(dt), top, scoring="sigmoid", groups=(count, keep) if count else None)
    s = torch.sigmoid(h @ wr.T)
    want = torch.tensor([O.choose(s[t], top, {"count": count, "keep": keep} if count else None) for t in range(T)])
    same = (ids.cpu().long() == want).all(-1)
    assert float(same.float().mean()) > 0.99, ids[~same.to(ids.device)]   # (a near-tie among hundreds may round over)
    close(w.cpu()[same], torch.gather(s, 1, want)[same], torch.float32)
    assert int(ids.min()) >= 0 and int(ids.max()) < E
    plain = M.route_direct(h.to(dev).to(dt), wr.to(dev).to(dt), top, scoring="sigmoid")[1].cpu().long()
    if keep < count < E:
        assert not torch.equal(plain, ids.cpu().long())                   # the groups matter here


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("E,top,X,W,T", [(5, 2, 1, 64, 9), (30, 3, 2, 256, 20), (16, 2, 1, 1024, 600)])
def test_softmax_router_with_bias_and_gate_rows_at_matrix_core_sizes(backend, E, top, X, W, T):
    """The router's other options on the sizes its matrix-core form takes."""
    dev, dt = backend
    h, wr, bias = b16(T, W, seed=E), b16(E + X, W, seed=2, std=2.0 * W ** -0.5), rnd(E, seed=3, std=0.2)
    w, ids, extra = M.route_direct(h.to(dev).to(dt), wr.to(dev).to(dt), top, scoring="softmax", renorm=True, renorm_eps=1e-20,
                                   scale=1.3, extra_rows=X, choice_bias=f32(bias, dev))
    z = h @ wr.T
    s = torch.softmax(z[:, :E], -1)
    want = torch.sort(s + bias, dim=-1, descending=True, stable=True).indices[:, :top]
    same = (ids.cpu().long() == want).all(-1)
    assert float(same.float().mean()) > 0.99
    ws = torch.gather(s, 1, want)
    close(w.cpu()[same], (ws / ws.sum(-1, keepdim=True) * 1.3)[same], torch.float32)
    close(extra, z[:, E:], torch.float32)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("rows,E,F,W,form", [(37, 5, 20, 24, "any"), (100, 4, 128, 128, "plain"), (100, 4, 128, 256, "split"),
                                             (60, 6, 64, 128, "strips"), (2200, 4, 256, 128, "big"), (2200, 3, 256, 256, "tokens")])
def test_squared_relu_in_the_grouped_products(backend, rows, E, F, W, form):
    """Every grouped kernel with the activation in its epilogue (or behind its split sum); an expert without rows; the
    prefill form also with the tokens' rows read in expert order by the kernel's own loads."""
    dev, dt = backend
    k = 2
    T = rows // k if form == "tokens" else rows
    x, w = b16(T, W, seed=1), b16(E, F, W, seed=2, std=W ** -0.5)
    ids = torch.randint(0, E - 1, (T, k if form == "tokens" else 1), generator=torch.Generator().manual_seed(3))
    ids[ids == 1] = E - 1                                                # expert 1 gets nothing
    order, inv, offsets = M.align(ids.to(torch.int32).to(dev), E)
    of = ids.reshape(-1)[order.cpu().long()]
    xr = x[order.cpu().long() // ids.shape[1]]
    want = torch.relu((w[of] * xr[:, None]).sum(-1)).pow(2)
    xd, wd = x.to(dev).to(dt), w.to(dev).to(dt)
    xp = M.gather_rows(xd, order, ids.shape[1])
    if form == "tokens" and dt == torch.bfloat16:
        got = M.grouped_big(xd, wd, offsets, act="relu_sq", order=order, k=k)
        close(M.grouped_big(xd, wd, offsets, order=order, k=k), (w[of] * xr[:, None]).sum(-1), dt)
    elif form in ("big", "tokens"):
        got = M.grouped_auto(xp, wd, offsets, act="relu_sq")
    else:
        got = M.grouped_gemm(xp, wd, offsets, act="relu_sq", splits=2 if form == "split" else 1,
                             glds=13 if form == "strips" else 0)
    close(got, want, dt)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("T", [1, 7, 16, 17, 32, 33])
@pytest.mark.parametrize("F,W", [(48, 256), (96, 1024), (10, 24)])
def test_projection_with_fp32_result(backend, T, F, W):
    """A few rows on the weight-streaming kernel, more on the library's; sizes that neither splits evenly."""
    from k8s_llm_rca_amd.ops.linear import proj_f32out
    dev, dt = backend
    x, w = b16(T, W, seed=1), b16(F, W, seed=2, std=W ** -0.5)
    got = proj_f32out(x.to(dev).to(dt), w.to(dev).to(dt))
    assert got.dtype == torch.float32
    close(got, x @ w.T, torch.float32)


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("backend", BACKENDS)
def test_streams_match_after_every_layer(backend):
    dev, dt = backend
    d = default_config()
    W = weights(d, 55, clear=backend[1] == torch.bfloat16)
    tokens = toks(45, d["vocab"], 2)
    want = []
    O.forward(W, d, tokens, want)
    eng = engine(d, W, backend)
    sid = eng.new_sequence()
    got = []
    fw = eng.model.forward
    eng.model.forward = lambda *a, **k: fw(*a, layers_out=got, **k)
    eng.feed([(sid, tokens, [])])
    assert len(got) == len(want) == len(d["layers"])
    for i, (g, w) in enumerate(zip(got, want)):
        e = (g.double().cpu() - w).abs().max(-1).values / w.abs().max()       # per token
        if dt == torch.float32:
            assert float(e.max()) < 2e-5, (i, float(e.max()))
        else:
            assert float(e.median()) < 0.01 and float(e.max()) < 0.05, (i, float(e.median()), float(e.max()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cuts", [(), (80,), (30, 2, 2, 17, 3, 5), (79,), (1, 68), (21, 22, 2)])
def test_prefill_decode_and_portions_agree_with_oracle(backend, cuts):
    """() = token by token from the first token on; (80,) = one prefill; portions down to two tokens."""
    d = default_config()
    W = weights(d, 23, clear=backend[1] == torch.bfloat16)
    tokens = toks(80, d["vocab"], 4)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    got = feed_all(eng, eng.new_sequence(), tokens, cuts)
    assert agrees(got, want, backend[1])


@pytest.mark.parametrize("backend", BACKENDS)
def test_mixed_batches_equal_each_alone_and_reuse_pages(backend):
    """Five requests of unequal length through a pool that cannot hold them all at once: portions of some beside
    single tokens of others; finished requests give their pages back."""
    d = default_config()
    W = weights(d, 41, clear=backend[1] == torch.bfloat16)
    lens = [50, 9, 33, 1, 64]
    reqs = [toks(n, d["vocab"], 10 + i) for i, n in enumerate(lens)]
    want = [O.forward(W, d, r) for r in reqs]
    eng = engine(d, W, backend, num_blocks=5, block_size=32)
    got = [[] for _ in reqs]
    at = [0] * len(reqs)
    sid = {}
    plan = [[(0, 20), (1, 2)], [(0, 1), (1, 7), (2, 30)], [(0, 29), (2, 1)], [(2, 2), (3, 1)],       # 0, 1, 3 end
            [(4, 40)], [(4, 1)], [(4, 23)]]
    for step in plan:
        entries, who = [], []
        for i, n in step:
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
        assert agrees(torch.cat(got[i]), want[i], backend[1], mult=1.5), i
    assert eng.kv.free_blocks == eng.kv.num_blocks


def marker_weights(d, seed, marker, asker, clear):
    """Weights under which token ``asker``'s queries find token ``marker``'s keys (scores of about the cap) and hardly
    any other: one direction of the residual is theirs alone."""
    W = weights(d, seed, clear)
    n, wd, m = d["streams"], d["width"], d["layers"][0]["mixer"]
    H, G, D, r = m["heads"], m["kv_heads"], m["dim"], (m.get("rot") or {}).get("dims", 0)
    a, b = CLASSES, CLASSES + 1
    W["embed"][:, a], W["embed"][:, b] = 0.0, 0.0
    W["embed"][marker, a] = 4.0
    W["embed"][asker, b] = 4.0
    q, k = W["l0.mix.q"].view(H, D, wd), W["l0.mix.k"].view(G, D, wd)
    q[:, :, b], k[:, :, a] = 0.0, 0.0
    q[:, r, b], k[:, r, a] = 6.0, 6.0              # entry r of every head is not rotated
    W["l0.hc1.in"] = torch.full((n,), 0.5)
    W["l0.norm1"][a:b + 1] = 1.0
    return {k_: v.to(torch.bfloat16).float() for k_, v in W.items()}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("window", [21, 32, 33, 64])
@pytest.mark.parametrize("dim", [16, 64])
def test_marked_key_at_the_windows_edge(backend, window, dim):
    """One layer: a marked token just inside and just outside the window of an asking one, in a prompt, in portions and
    decoded alone.  Replacing it changes the asker's logits exactly where it is inside."""
    d = config([(att(heads=4, kv_heads=2, dim=dim, window=window, rot=4, cap=15.0, scale=2.0 / dim), moe())])
    marker, asker, other, at = 500, 501, 7, 70
    W = marker_weights(d, 6, marker, asker, backend[1] == torch.bfloat16)
    for back in (window - 1, window):
        tokens = toks(at, 499, 7) + [asker, 3, 4]
        tokens[at - back] = marker
        want = O.forward(W, d, tokens)
        swapped = list(tokens)
        swapped[at - back] = other
        moved = float(row_errs(O.forward(W, d, swapped)[at:at + 1], want[at:at + 1]))
        assert (moved > 0.2) if back < window else (moved < 1e-9)
        for cuts in [(73,), (at,), (at - back + 1, 2, 300), (31, 33)]:
            eng = engine(d, W, backend)
            got = feed_all(eng, eng.new_sequence(), tokens, cuts)
            assert float(row_errs(got[at:at + 1], want[at:at + 1])) < (1e-5 if backend[1] == torch.float32 else 0.05), (back, cuts)
            assert agrees(got, want, backend[1], mult=2.0), (back, cuts)


@pytest.mark.parametrize("backend", BACKENDS)
def test_far_marked_key_without_a_window(backend):
    """A marked token hundreds back, at both sides of a page border, asked for by a decoded token."""
    d = config([(att(heads=4, kv_heads=2, dim=16, window=0, rot=4, cap=15.0, scale=0.1), None)])
    marker, asker = 500, 501
    W = marker_weights(d, 16, marker, asker, backend[1] == torch.bfloat16)
    for place in (0, 31, 32, 255):
        tokens = toks(330, 499, 17) + [asker]
        tokens[place] = marker
        want = O.forward(W, d, tokens)
        eng = engine(d, W, backend)
        got = feed_all(eng, eng.new_sequence(), tokens, (330,))
        assert float(row_errs(got[330:], want[330:])) < (1e-5 if backend[1] == torch.float32 else 0.05), place


@pytest.mark.parametrize("backend", BACKENDS)
def test_first_tokens(backend):
    d = default_config()
    W = weights(d, 50, clear=backend[1] == torch.bfloat16)
    for n in (1, 2, 3):
        tokens = toks(n, d["vocab"], 20 + n)
        eng = engine(d, W, backend)
        assert agrees(feed_all(eng, eng.new_sequence(), tokens, (n,)), O.forward(W, d, tokens), backend[1], mult=2.5), n


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend):
    d = default_config()
    W = weights(d, 53, clear=backend[1] == torch.bfloat16)
    tokens = toks(150, d["vocab"], 10)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    got = feed_all(eng, eng.new_sequence(), tokens, (10,))           # 140 tokens one by one, past every window
    assert agrees(got, want, backend[1], mult=1.5)


OTHER = {
    "matrix_core_sizes": [(att(heads=4, kv_heads=2, dim=64, rot=32, window=17), moe()), (att(heads=9, kv_heads=3, dim=96, rot=40), None),
                          (att(heads=3, kv_heads=1, dim=128, rot=64, window=5, cap=0), moe(count=0)), 0, 1],
    "expert_kernel_sizes": [(att(), moe(ff=128, experts=8, top=2, count=2, keep=1)), (att(), moe(ff=64, experts=4, top=4, count=0)), 0],
    "one_of_everything": [(att(heads=1, kv_heads=1, dim=4, rot=2, window=1), moe(ff=8, experts=1, top=1, count=1, keep=1))],
    "groups_of_one_and_keep_all": [(att(), moe(experts=5, top=2, count=5, keep=3)), (att(), moe(experts=6, top=3, count=2, keep=2))],
    "no_feed_forward": [(att(), None), 0, (att(window=2), None)],
    "no_rotation_no_cap_no_window": [(att(rot=0, cap=0, window=0), moe()), (att(rot=0, window=3), moe(count=0)), 0],
    "whole_head_rotated_no_yarn": [(att(dim=8, rot=8, yarn=None), moe()), (att(dim=10, rot=10, heads=3, kv_heads=3), None)],
    "unaligned_sizes": [(att(heads=5, kv_heads=1, dim=7, rot=2, window=6), moe(ff=11, experts=7, top=2, count=0)),
                        (att(heads=3, kv_heads=3, dim=9, rot=6), moe(ff=3, experts=9, top=3, count=3, keep=1)), 0],
    "reuse_before_and_across": [(att(), moe()), (att(heads=2, kv_heads=2, dim=6, window=9), None), 1, 0, 1, 3],
    "many_streams": [(att(), moe()), 0], "one_stream": [(att(), moe()), 0], "plain_residual": [(att(), moe()), 0, (att(), None)],
    "constants_of_one": [(att(scale=1.0, base=2.0, yarn={"factor": 1.0, "original": 7, "fast": 2.0, "slow": 1.0}), moe()), 0],
}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(backend, name):
    kw = {"unaligned_sizes": dict(width=34, vocab=301), "matrix_core_sizes": dict(width=64, streams=2),
          "expert_kernel_sizes": dict(width=128, streams=4), "many_streams": dict(streams=7, mult=0.2), "one_stream": dict(streams=1),
          "plain_residual": dict(streams=0), "constants_of_one": dict(mult=1.0, scale=1.0)}.get(name, dict(width=40))
    d = config(OTHER[name], eps=1e-3, **kw)
    W = weights(d, 11, clear=backend[1] == torch.bfloat16)
    tokens = toks(40, d["vocab"], 12)
    want = O.forward(W, d, tokens)
    eng = engine(d, W, backend)
    assert agrees(feed_all(eng, eng.new_sequence(), tokens, (13, 2, 9)), want, backend[1], mult=2.0)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("overlap", [True, False])
def test_greedy_generation_through_submit_and_scheduler(backend, overlap):
    """``submit`` + ``step``: the scheduler's own batching (two prompts of unequal length, then decode rows), with the
    next step launched before the host has the last one's tokens and without, must produce the oracle's greedy
    continuation."""
    d = default_config(vocab=8192)
    W = weights(d, 50, clear=backend[1] == torch.bfloat16)
    eng = engine(d, W, backend, num_blocks=16, async_steps=overlap)
    assert eng._async == overlap
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
                assert int((lg > lg[t]).sum()) < 40, i
                same += t == int(lg.argmax())
            seq.append(t)
        assert len(outs[i]) >= 6 and (backend[1] == torch.float32 or same >= 3)


@pytest.mark.parametrize("backend", BACKENDS)
def test_shared_prefix_and_a_thread_that_goes_on_or_diverges(backend):
    """Pages hold all a sequence carries, so a second thread attaches the first one's prompt pages, and a thread whose
    next prompt diverges keeps the common prefix; the tokens are the oracle's."""
    d = default_config(vocab=8192)
    W = weights(d, 52, clear=backend[1] == torch.bfloat16)
    eng = engine(d, W, backend, num_blocks=24)
    common = toks(70, 2000, 24)

    def run(sid, prompt):
        out = []
        eng.submit(sid, prompt, None, 3, temperature=0.0, on_done=lambda g, st: out.extend(g))
        eng.run_until_idle()
        seq = list(prompt)
        for t in out[:3]:
            lg = O.forward(W, d, seq)[-1, :eng.vocab]
            assert t == int(lg.argmax()) if backend[1] == torch.float32 else int((lg > lg[t]).sum()) < 40
            seq.append(t)
        assert len(out) >= 3

    a, b = eng.new_sequence(), eng.new_sequence()
    run(a, common + toks(9, 2000, 25))
    before = eng.stats["prefix_hit_tokens"]
    run(b, common + toks(5, 2000, 26))
    assert eng.stats["prefix_hit_tokens"] - before >= 64                 # two pages of 32 shared
    run(a, common + toks(20, 2000, 27))                                  # diverges behind the common part
    run(b, common[:40] + toks(11, 2000, 28))                             # diverges inside a shared page


def test_config_round_trip_registry_and_replay(tmp_path):
    """config.json -> configuration -> config.json; the registry picks the class by the file; a recorded
    schedule replayed through the engine gives the oracle's logits."""
    from k8s_llm_rca_amd.engine import trace as TR
    from k8s_llm_rca_amd.models import sunesun as SN
    from k8s_llm_rca_amd.models.registry import checkpoint_arch, get_any_config, load_model
    d = default_config()
    cfg = SunesunConfig.from_json(d, "x")
    assert SunesunConfig.from_json(cfg.to_json(), "x") == cfg
    assert cfg.to_json()["layers"] == d["layers"]
    assert get_any_config("tiny-sunesun").arch == "sunesun"
    tiny = SunesunModel(get_any_config("tiny-sunesun"), "cpu", torch.float32)
    assert tiny.weight_bytes() > 0 and len(tiny.weights) == 2 and len(tiny._widths()) == 4
    W = weights(d, 21)
    path = str(tmp_path / "ckpt")
    SN.save_checkpoint(cfg, W, path)
    assert checkpoint_arch(path) == "sunesun"
    assert isinstance(load_model(path, "cpu", torch.float32), SunesunModel)
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
    assert eng.kv.free_blocks == eng.kv.num_blocks


def test_bad_configurations_are_refused():
    def refused(d):
        with pytest.raises(ValueError):
            SunesunModel(SunesunConfig.from_json(d, "bad"), "cpu", torch.float32, init=False)

    for layers in ([(att(heads=4, kv_heads=3), None)], [(att(rot=3), None)], [(att(dim=4, rot=6), None)],
                   [(att(), moe(experts=2, top=3, count=0))], [(att(), moe(experts=10, count=4))],
                   [(att(), moe(experts=12, top=4, count=4, keep=1))]):
        refused(config(layers))
    d = config([(att(), None), 0])
    d["layers"][0]["weights_of"] = 1                                     # a circle
    refused(d)
    d = config([(att(), moe()), 0])
    d["layers"][1]["mixer"]["softcap"] = 1.5                             # an entry that differs from its source's
    refused(d)
    d = config([(att(), None)])
    d["layers"][0]["mixer"]["vdim"] = 4
    refused(d)


def test_trace_run_command_line(tmp_path):
    from k8s_llm_rca_amd.models import sunesun as SN
    d = default_config()
    W = weights(d, 31)
    path = str(tmp_path / "ckpt")
    SN.save_checkpoint(SunesunConfig.from_json(d, "x"), W, path)
    tokens = toks(12, d["vocab"], 32)
    step = json.dumps({"step": 0, "entries": [{"id": "r", "tokens": tokens, "want": [11]}], "end": ["r"]})
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(tmp_path / "o"), "--max-tokens", "64", "--device", "cpu"], input=step + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0 and "done 0" in r.stdout, r.stderr[-2000:]
    got = torch.from_numpy(np.fromfile(str(tmp_path / "o" / "0.f32"), dtype="<f4").reshape(1, -1))
    assert agrees(got, O.forward(W, d, tokens)[-1:], torch.float32)
