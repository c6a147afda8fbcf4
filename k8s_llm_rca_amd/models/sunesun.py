"""Sunesun decoder: hyper-connections around windowed attention whose keys double as values, and a mixture of experts
chosen group-first.

Residual:      ``streams`` fp32 copies x_1 .. x_S of the embedding output.  Around every sublayer
               ``u = sum_s in[s] x_s``, ``y = sublayer(rms(u) w)``, ``x_r <- sum_s mix[s, r] x_s + residual_mult out[r] y``
               with vectors and a matrix of the sublayer's own; at the end x is the sum of the streams.  Without
               ``streams`` it is the plain pre-norm residual ``x <- x + residual_mult sublayer(rms(x) w)``.
``attention``: q = W_q h, k = W_k h; the values are the keys as projected, in front of their rotation (there is no
               value projection); q and k rotated on the first ``rot.dims`` entries of every head, neighbouring
               entries a pair, with YaRN's frequencies and amplitude; scores times ``scale``, soft-capped; a sliding
               window; ordinary softmax.
feed-forward:  experts ``W_down relu(W_up h)^2``; a sigmoid router whose experts form groups of neighbours: only the
               experts of the best groups (by the sum of their two largest scores) can be chosen; the weights are the
               scores themselves.
Weight reuse:  a layer with ``weights_of`` runs another layer's tensors on a cache of its own.
Output:        the final RMS norm, then a head of its own.

What a sequence carries from step to step is keys and values in cache pages alone
(:class:`~..engine.kv_cache.WindowKVPool`): no state slots, so pages can be shared and rewound.  Every size, and
every constant that can differ between checkpoints, comes from the configuration or from a tensor's shape.
"""
from __future__ import annotations

import json
import math
import os
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch

from ..ops import moe as M
from ..ops import norm as N
from ..ops import seq_ops as S
from ..ops.linear import proj_f32out
from ..parallel.groups import ParallelContext, single
from .moe import MoELayerSet


@dataclass(frozen=True)
class AttnSpec:
    """``attention``: keys double as values (``vdim == dim``)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0        # 0: no cap
    window: int = 0             # keys a position sees, itself included; 0: all before it
    rot_dims: int = 0           # 0: no rotation
    rot_base: float = 10000.0
    yarn: Optional[Tuple[float, float, float, float]] = None    # factor, original, fast, slow


@dataclass(frozen=True)
class MoeSpec:
    ff: int
    experts: int
    top: int
    groups: int = 0             # 0: every expert can be chosen
    keep: int = 0


@dataclass(frozen=True)
class LayerSpec:
    attn: AttnSpec
    mlp: Optional[MoeSpec] = None
    weights_of: Optional[int] = None


@dataclass(frozen=True)
class SunesunConfig:
    name: str
    vocab_size: int
    hidden: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float = 1e-5
    embed_scale: float = 1.0
    residual_mult: float = 1.0
    streams: int = 0               # 0: one plain residual, no hyper-connection tensors
    max_position: int = 1 << 20    # no tabulated positions: any length the cache holds
    arch: str = "sunesun"

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_json(cls, d: dict, name: str = "sunesun") -> "SunesunConfig":
        layers = []
        for L in d["layers"]:
            if L["type"] != "attention":
                raise ValueError(f"unknown mixer type {L['type']!r}")
            m, f = L["mixer"], L.get("mlp")
            rot = m.get("rot") or {}
            sc = rot.get("scaling")
            yarn = tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None
            attn = AttnSpec(int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]),
                            int(m.get("vdim", m["dim"])), float(m["scale"]), float(m.get("softcap") or 0.0),
                            int((m.get("mask") or {}).get("size") or 0), int(rot.get("dims", 0)),
                            float(rot.get("base", 10000.0)), yarn)
            mlp = None
            if f is not None:
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"unknown feed-forward kind {f['kind']!r}")
                r = f["router"]
                g = r.get("groups") or {}
                mlp = MoeSpec(int(f["expert"]["ff"]), int(r["experts"]), int(r["top"]), int(g.get("count", 0)),
                              int(g.get("keep", 0)))
            wo = L.get("weights_of")
            layers.append(LayerSpec(attn, mlp, int(wo) if wo is not None else None))
        return cls(name, int(d["vocab"]), int(d["width"]), tuple(layers), norm_eps=float(d["norm"]["eps"]),
                   embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
                   residual_mult=float(d.get("residual_mult", 1.0)), streams=int(d.get("streams") or 0))

    def to_json(self) -> dict:
        layers = []
        for L in self.layers:
            a, f = L.attn, L.mlp
            m: dict = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
            if a.softcap:
                m["softcap"] = a.softcap
            if a.window:
                m["mask"] = {"size": a.window}
            if a.rot_dims:
                m["rot"] = {"dims": a.rot_dims, "base": a.rot_base}
                if a.yarn:
                    m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), a.yarn))
            mlp = None
            if f is not None:
                mlp = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top}}
                if f.groups:
                    mlp["router"]["groups"] = {"count": f.groups, "keep": f.keep}
            d = {"type": "attention", "mixer": m, "mlp": mlp}
            if L.weights_of is not None:
                d["weights_of"] = L.weights_of
            layers.append(d)
        d = {"architecture": "Sunesun", "vocab": self.vocab_size, "width": self.hidden, "layers": layers,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embed_scale},
             "residual_mult": self.residual_mult}
        if self.streams:
            d["streams"] = self.streams
        return d

    def source(self, i: int) -> int:
        """The layer whose tensors layer ``i`` runs."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen or not 0 <= self.layers[i].weights_of < len(self.layers):
                raise ValueError(f"layer {i}: weights_of must lead to a layer with tensors of its own")
            seen.add(i)
            i = self.layers[i].weights_of
        return i


def _stack(n: int, attn: AttnSpec, mlp: MoeSpec) -> Tuple[LayerSpec, ...]:
    """``n`` layer runs over n / 2 sets of weights: every odd run repeats the weights of the one before it."""
    return tuple(LayerSpec(attn, mlp, i - 1 if i % 2 else None) for i in range(n))


PRESETS: Dict[str, SunesunConfig] = {
    "tiny-sunesun": SunesunConfig(
        "tiny-sunesun", 8192, 256, _stack(4, AttnSpec(8, 2, 64, 64, 0.125, 30.0, 128, 32, 10000.0, (4.0, 1024, 32.0, 1.0)),
                                          MoeSpec(128, 8, 2, 4, 2)), embed_scale=16.0, residual_mult=0.4, streams=2),
    # sizes of a ~1B-class decoder's layers (benchmarks; random weights)
    "sunesun-1b": SunesunConfig(
        "sunesun-1b", 32768, 2048, _stack(12, AttnSpec(16, 2, 128, 128, 128 ** -0.5, 30.0, 1024, 64, 500000.0,
                                                       (8.0, 4096, 32.0, 1.0)),
                                          MoeSpec(2048, 16, 2, 4, 2)), embed_scale=45.0, residual_mult=0.25, streams=4),
}


class SunesunModel:
    stateful = False           # pages hold everything: prefixes can be shared, steps overlapped
    step_layout = "segments"   # the engine packs steps as segments (ops.seq_ops.SegStepInputs)
    graph_capturable = False

    def __init__(self, cfg: SunesunConfig, device, dtype=torch.bfloat16, pc: Optional[ParallelContext] = None,
                 seed: int = 0, init: bool = True):
        self.cfg = cfg
        self.device = torch.device(device)
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Sunesun runs in bfloat16 or float32")
        self.dtype = dtype
        self.pc = pc or single()
        if self.pc.tp_size != 1:
            raise ValueError("Sunesun runs on one device per replica (no tensor-parallel sharding of its layers)")
        self.logits_f32 = True
        self.weights: Dict[int, Dict[str, torch.Tensor]] = {}     # layers with tensors of their own
        self.source = [cfg.source(i) for i in range(cfg.n_layers)]
        self.ropes: List[Optional[S.Rope]] = []
        made: Dict[tuple, S.Rope] = {}
        for i, L in enumerate(cfg.layers):
            a, f = L.attn, L.mlp
            src = cfg.layers[self.source[i]]
            if (src.attn, src.mlp) != (a, f):
                raise ValueError(f"layer {i}: its entry must equal that of layer {self.source[i]}, whose tensors it runs")
            if a.heads % a.kv_heads:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
            if a.vdim != a.dim:
                raise ValueError(f"layer {i}: the values are the keys, so vdim must equal dim")
            if a.rot_dims % 2 or not 0 <= a.rot_dims <= a.dim or a.window < 0 or a.softcap < 0:
                raise ValueError(f"layer {i}: an even rot.dims <= dim, a window and a cap that are not negative")
            if f is not None:
                if not 1 <= f.top <= f.experts or f.experts > 256:
                    raise ValueError(f"layer {i}: 1..256 experts and top among them")
                if f.groups and (f.experts % f.groups or not 1 <= f.keep <= f.groups
                                 or f.keep * (f.experts // f.groups) < f.top):
                    raise ValueError(f"layer {i}: equal groups, and the kept ones must hold the top experts")
            key = (a.rot_dims, a.rot_base, a.yarn)
            if a.rot_dims and key not in made:
                made[key] = S.make_rope(a.rot_dims, a.rot_base, self.device, pairs=True, yarn=a.yarn)
            self.ropes.append(made[key] if a.rot_dims else None)
        if init:
            self._random_init(seed)

    # ------------------------------------------------------- what the engine allocates for this model
    def _twins(self) -> List[bool]:
        """Per layer run: whether the matrix-core kernel runs it (then its values are cached transposed, and only so)."""
        return [S.masked_mfma_ok(L.attn.heads, L.attn.kv_heads, L.attn.dim, L.attn.vdim, self.dtype, self.device)
                for L in self.cfg.layers]

    def _widths(self) -> List[Tuple[int, int]]:
        return [(L.attn.kv_heads * L.attn.dim, L.attn.kv_heads * L.attn.vdim) for L in self.cfg.layers]

    def cache_bytes_per_block(self, block_size: int) -> int:
        return max(1, sum(a + b for a, b in self._widths())) * block_size * (2 if self.dtype == torch.bfloat16 else 4)

    def make_cache(self, num_blocks: int, block_size: int):
        from ..engine.kv_cache import WindowKVPool
        return WindowKVPool(self._widths(), num_blocks, block_size, self.device, self.dtype, self._twins(), twin_only=True)

    def workspace_bytes(self, tokens: int) -> int:
        w, widest = self.cfg.hidden, 0
        for L in self.cfg.layers:
            a, f = L.attn, L.mlp
            widest = max(widest, 2 * a.heads * (a.dim + a.vdim) + a.kv_heads * a.dim)
            if f is not None:
                widest = max(widest, f.top * (2 * f.ff + 2 * w))
        return int(tokens * (4 * w * (max(1, self.cfg.streams) + 2) + widest * 4) + (2 << 30))

    # --------------------------------------------------------------- weights
    def _random_init(self, seed: int) -> None:
        t = random_tensors(self.cfg, seed, self.device)
        self.load_tensors(t.__getitem__)

    def load_tensors(self, get, has=None) -> None:
        """Build the fused device layout from checkpoint tensors (``get(name)`` -> tensor; names of the
        safetensors file: ``embed``, ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.hc1.in`` ...)."""
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def put(*names, dtype=dt):
            ts = [get(n) for n in names]
            return (ts[0] if len(ts) == 1 else torch.cat(ts, 0)).to(device=dev, dtype=dtype).contiguous()

        def f32(name):
            return put(name, dtype=torch.float32)

        self.embed, self.head, self.final_norm = put("embed"), put("head"), f32("final.norm")
        one = torch.ones(1, dtype=torch.float32, device=dev)
        self.weights = {}
        for i in sorted(set(self.source)):
            p, f = f"l{i}.", cfg.layers[i].mlp
            L: Dict[str, torch.Tensor] = {"w_in": put(p + "mix.q", p + "mix.k"),      # one fp32-out GEMM: q | k (= v)
                                          "wo": put(p + "mix.o")}
            for q in ("1", "2") if f is not None else ("1",):
                L["norm" + q] = f32(p + "norm" + q)
                if cfg.streams:
                    L["in" + q], L["mix" + q] = f32(f"{p}hc{q}.in"), f32(f"{p}hc{q}.mix")
                    L["out" + q] = f32(f"{p}hc{q}.out") * cfg.residual_mult
                else:                                                                  # one stream that is only added to
                    L["in" + q], L["mix" + q], L["out" + q] = one, one.view(1, 1), one * cfg.residual_mult
            if f is not None:
                m = p + "mlp."
                L["router"] = put(m + "router")
                L["w_up"] = torch.stack([put(f"{m}e{e}.up") for e in range(f.experts)]).contiguous()
                L["w_down"] = torch.stack([put(f"{m}e{e}.down") for e in range(f.experts)]).contiguous()
            self.weights[i] = L

    def weight_bytes(self) -> int:
        ts = [t for L in self.weights.values() for t in L.values()] + [self.embed, self.head, self.final_norm]
        return sum(t.numel() * t.element_size() for t in ts)

    # -------------------------------------------------------------- forward
    def _attention(self, li: int, L, h: torch.Tensor, inp: S.SegStepInputs, tables, kc, vc, vt) -> torch.Tensor:
        a, rope = self.cfg.layers[li].attn, self.ropes[li]
        H, G, D = a.heads, a.kv_heads, a.dim
        x = proj_f32out(h, L["w_in"])                                  # [T, H D + G D] fp32
        if rope is not None and id(rope) not in tables:
            tables[id(rope)] = S.rope_table(inp.positions, rope)
        q = S.attn_prep(x, None, H, G, D, D, inp.positions, inp.slots, kc, vc, self.dtype, rope=rope,
                        rope_cs=tables.get(id(rope)), vt=vt, v_is_k=True)
        o = S.masked_attention(q, H, G, D, D, kc, vc, inp.seg, a.scale, softcap=a.softcap, window=a.window, vt=vt)
        return proj_f32out(o, L["wo"])

    def _moe(self, li: int, L, h: torch.Tensor):
        """The experts' output rows in expert order, and (inv, w) that join them."""
        f = self.cfg.layers[li].mlp
        w, ids = M.route_direct(h, L["router"], f.top, scoring="sigmoid",
                                groups=(f.groups, f.keep) if f.groups else None)
        order, inv, offsets = M.align(ids, f.experts)
        rows = order.numel()
        dev16 = h.is_cuda and h.dtype == torch.bfloat16
        if dev16 and rows > M.BIG_MIN_ROWS and M.grouped_big_ok(rows, f.ff, h.shape[1], False):
            # prefill sizes: the grouped MFMA GEMM reads the tokens' rows in expert order itself
            act = M.grouped_big(h, L["w_up"], offsets, act="relu_sq", order=order, k=f.top)
        elif dev16 and rows <= MoELayerSet.GLDS_MAX_ROWS:
            # decode sizes: the weight-streaming kernels (LDS-DMA strips up; the down projection with its K split)
            act = M.grouped_gemm(M.gather_rows(h, order, f.top), L["w_up"], offsets, glds=MoELayerSet.GLDS_UP[0],
                                 splits=MoELayerSet.GLDS_UP[1], act="relu_sq")
        else:
            act = M.grouped_auto(M.gather_rows(h, order, f.top), L["w_up"], offsets, act="relu_sq")
        if dev16 and rows <= MoELayerSet.SPLIT_MAX_ROWS:
            yp = M.grouped_gemm(act, L["w_down"], offsets, splits=MoELayerSet.DOWN_SPLITS)
        else:
            yp = M.grouped_auto(act, L["w_down"], offsets)
        return yp, (inv, w)

    def forward(self, inp: S.SegStepInputs, kcs: List[torch.Tensor], vcs: List[Optional[torch.Tensor]],
                vts: List[Optional[torch.Tensor]], states: Optional[Dict[str, torch.Tensor]] = None,
                layers_out: Optional[list] = None) -> torch.Tensor:
        """Logits [len(logits_idx), vocab] fp32.  ``kcs`` / ``vcs`` / ``vts``: the paged keys, values and transposed
        values of every layer run.  ``layers_out`` (debugging): receives the sum of the streams after every run."""
        cfg, eps, dt = self.cfg, self.cfg.norm_eps, self.dtype
        T = inp.input_ids.shape[0]
        runs = [self.weights[s] for s in self.source]
        tables: Dict[int, torch.Tensor] = {}       # cos | sin of the step's positions, one per distinct rotation
        x = torch.empty(T, max(1, cfg.streams), cfg.hidden, dtype=torch.float32, device=self.device)
        h = N.hyper_embed(inp.input_ids, self.embed, cfg.embed_scale, x, runs[0]["in1"], runs[0]["norm1"], eps, dt)
        for li, (spec, L) in enumerate(zip(cfg.layers, runs)):
            nxt = runs[li + 1] if li + 1 < len(runs) else None
            into = dict(inn=nxt["in1"], nw=nxt["norm1"], eps=eps, out_dtype=dt) if nxt is not None else {}
            y = self._attention(li, L, h, inp, tables, kcs[li], vcs[li], vts[li])
            if spec.mlp is None:
                h = N.hyper_step(x, y, L["out1"], L["mix1"], **into)
            else:
                h = N.hyper_step(x, y, L["out1"], L["mix1"], inn=L["in2"], nw=L["norm2"], eps=eps, out_dtype=dt)
                yp, join = self._moe(li, L, h)
                h = N.hyper_step(x, yp, L["out2"], L["mix2"], experts=join, **into)
            if layers_out is not None:
                layers_out.append(x.sum(1))
        return proj_f32out(N.hyper_read(x, inp.logits_idx, self.final_norm, eps, dt), self.head)


def random_tensors(cfg: SunesunConfig, seed: int = 0, device="cpu") -> Dict[str, torch.Tensor]:
    """Seeded random weights under the checkpoint's names, bfloat16 (so a bfloat16 and a float32 model
    built from them hold the same numbers)."""
    dev = torch.device(device)
    g = torch.Generator(device=dev)
    g.manual_seed(seed)
    W = cfg.hidden

    def rnd(*shape, std=0.02, mean=0.0):
        return torch.empty(*shape, dtype=torch.float32, device=dev).normal_(mean, std, generator=g).to(torch.bfloat16)

    def lin(n_out, n_in, gain=1.0):
        return rnd(n_out, n_in, std=gain / math.sqrt(n_in))

    t: Dict[str, torch.Tensor] = {"embed": rnd(cfg.vocab_size, W, std=1.0 / cfg.embed_scale), "head": lin(cfg.vocab_size, W),
                                  "final.norm": rnd(W, std=0.1, mean=1.0)}
    n = cfg.streams
    for i, L in enumerate(cfg.layers):
        if L.weights_of is not None:
            continue
        p, a, f = f"l{i}.", L.attn, L.mlp
        t[p + "mix.q"], t[p + "mix.k"] = lin(a.heads * a.dim, W, 1.5), lin(a.kv_heads * a.dim, W, 1.5)
        t[p + "mix.o"] = lin(W, a.heads * a.vdim)
        for q in ("1", "2") if f is not None else ("1",):
            t[p + "norm" + q] = rnd(W, std=0.1, mean=1.0)
            if n:
                t[f"{p}hc{q}.in"], t[f"{p}hc{q}.out"] = rnd(n, std=0.2, mean=1.0 / n), rnd(n, std=0.3, mean=1.0)
                t[f"{p}hc{q}.mix"] = (0.9 * torch.eye(n, device=dev) + rnd(n, n, std=0.05)).to(torch.bfloat16)
        if f is not None:
            m = p + "mlp."
            t[m + "router"] = lin(f.experts, W, 2.0)
            for e in range(f.experts):
                t[f"{m}e{e}.up"], t[f"{m}e{e}.down"] = lin(f.ff, W), lin(W, f.ff)
    return t


def load_checkpoint(path: str, device, dtype, pc=None) -> SunesunModel:
    """A folder with config.json and model.safetensors (bfloat16 weights) -> the model on ``device``."""
    from safetensors import safe_open
    with open(os.path.join(path, "config.json")) as f:
        cfg = SunesunConfig.from_json(json.load(f), name=os.path.basename(os.path.normpath(path)) or "sunesun")
    model = SunesunModel(cfg, device, dtype, pc, init=False)
    with safe_open(os.path.join(path, "model.safetensors"), framework="pt", device="cpu") as h:
        model.load_tensors(h.get_tensor, set(h.keys()).__contains__)
    return model


def save_checkpoint(cfg: SunesunConfig, tensors: Dict[str, torch.Tensor], path: str) -> None:
    """Write config.json + model.safetensors (bfloat16) in the layout :func:`load_checkpoint` reads."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg.to_json(), f, indent=1)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()},
              os.path.join(path, "model.safetensors"))
