"""Fikerax decoder: lightning attention, windowed attention with normed rotated heads, and windowed latent attention with a
sink, in a pre-norm stack of which a part may run several times in a row.

Residual:             ``x = embed[token] * embed_scale`` in fp32; around every sublayer ``x <- x + sublayer(rms(x) (1 + w))``.
Repeats:              layers ``loop.start .. loop.stop - 1`` run ``loop.times`` times with the same tensors, each pass on a
                      cache or state of its own; in front of every pass but the first the embedding output is added to x.
``lightning``:        q, k, v = silu of one projection; per head ``S <- decay_h S + k v^T``, ``o = S^T q``; the heads side by
                      side RMS-normed as one vector, times ``sigmoid(W_g h)``, then W_o.
``attention``:        q, k, v with biases; q and k rotated (entry i with i + dims / 2, long wavelengths stretched by a
                      factor), then each head divided by its root mean square; scores times ``scale``; sliding window.
``latent_attention``: queries through a normed latent; keys and values from a normed latent c per token plus one rotated key
                      part shared by the heads (neighbouring entries a pair, YaRN).  The cache holds c and that part; the
                      query moves into latent space (``qa[h] = W_uk[h]^T q[h]``), attention runs over the latents, W_uv and
                      W_o follow.  Sliding window; the softmax's denominator also holds ``exp(sink_h)``.
feed-forward:         ``W_down (silu(W_gate h) * W_up h)``, or none.
Output:               the final norm, then a head of its own.

What a sequence carries from step to step: keys, values and latents in cache pages (:class:`~..engine.kv_cache.WindowKVPool`),
and per run of a lightning layer its state in the sequence's slot (fp32).  Every size, and every constant that can differ
between checkpoints, comes from the configuration or from a tensor's shape.
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
from ..ops.linear import linear, proj_f32out, swiglu_gemm
from ..parallel.groups import ParallelContext, single

TAIL_ALIGN = 32     # the rotated key part of a latent cache row is filled up to a multiple of this
Scaling = Optional[Tuple[float, float, float, float]]
STRETCH_KEYS = ("factor", "low", "high", "original")
YARN_KEYS = ("factor", "original", "fast", "slow")


@dataclass(frozen=True)
class LightningSpec:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class AttnSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0             # keys a position sees, itself included; 0: all before it
    rot_dims: int = 0           # 0: no rotation
    rot_base: float = 10000.0
    stretch: Scaling = None     # factor, low, high, original


@dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int                    # unrotated query / key entries per head
    rot_dim: int                # rotated ones (the key's are shared by the heads)
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int = 0
    rot_base: float = 10000.0
    yarn: Scaling = None        # factor, original, fast, slow

    @property
    def tail(self) -> int:
        """Numbers of a cache row behind the latent."""
        return -(-self.rot_dim // TAIL_ALIGN) * TAIL_ALIGN


@dataclass(frozen=True)
class LayerSpec:
    kind: str                   # 'lightning' | 'attention' | 'latent_attention'
    mix: object                 # the kind's spec
    ff: int = 0                 # feed-forward width; 0: none


@dataclass(frozen=True)
class FikeraxConfig:
    name: str
    vocab_size: int
    hidden: int
    layers: Tuple[LayerSpec, ...]
    norm_eps: float = 1e-5
    embed_scale: float = 1.0
    loop: Optional[Tuple[int, int, int]] = None     # start, stop, times
    max_position: int = 1 << 20    # no tabulated positions: any length the cache holds
    arch: str = "fikerax"

    @property
    def n_layers(self) -> int:
        return len(self.runs)

    @property
    def runs(self) -> Tuple[Tuple[int, bool], ...]:
        """(layer, whether the embedding output is added in front of it) in the order they run."""
        n = len(self.layers)
        start, stop, times = self.loop if self.loop is not None else (0, n, 1)
        out = [(i, False) for i in range(start)]
        for turn in range(times):
            out += [(i, turn > 0 and i == start) for i in range(start, stop)]
        return tuple(out + [(i, False) for i in range(stop, n)])

    @classmethod
    def from_json(cls, d: dict, name: str = "fikerax") -> "FikeraxConfig":
        def scaling(m, keys):
            sc = (m.get("rot") or {}).get("scaling")
            return tuple(float(sc[k]) for k in keys) if sc else None

        def window(m):
            return int((m.get("mask") or {}).get("size") or 0)

        layers = []
        for L in d["layers"]:
            m, f, kind = L["mixer"], L.get("mlp"), L["type"]
            rot = m.get("rot") or {}
            if kind == "lightning":
                mix = LightningSpec(int(m["heads"]), int(m["dim"]), int(m.get("vdim", m["dim"])),
                                    tuple(float(v) for v in m["decay"]))
            elif kind == "attention":
                mix = AttnSpec(int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]),
                               int(m.get("vdim", m["dim"])), float(m["scale"]), window(m), int(rot.get("dims", 0)),
                               float(rot.get("base", 10000.0)), scaling(m, STRETCH_KEYS))
            elif kind == "latent_attention":
                mix = LatentSpec(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m.get("vdim", m["dim"])),
                                 int(m["q_rank"]), int(m["kv_rank"]), float(m["scale"]), window(m),
                                 float(rot.get("base", 10000.0)), scaling(m, YARN_KEYS))
                if int(rot.get("dims", mix.rot_dim)) != mix.rot_dim:
                    raise ValueError("latent_attention rotates its rot_dim part: rot.dims must equal rot_dim")
            else:
                raise ValueError(f"unknown mixer type {kind!r}")
            if f is not None and f.get("kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {f['kind']!r}")
            layers.append(LayerSpec(kind, mix, int(f["ff"]) if f is not None else 0))
        lp = d.get("loop")
        return cls(name, int(d["vocab"]), int(d["width"]), tuple(layers), norm_eps=float(d["norm"]["eps"]),
                   embed_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
                   loop=(int(lp["start"]), int(lp["stop"]), int(lp.get("times", 1))) if lp else None)

    def to_json(self) -> dict:
        layers = []
        for L in self.layers:
            c = L.mix
            if L.kind == "lightning":
                m: dict = {"heads": c.heads, "dim": c.dim, "vdim": c.vdim, "decay": list(c.decay)}
            elif L.kind == "attention":
                m = {"heads": c.heads, "kv_heads": c.kv_heads, "dim": c.dim, "vdim": c.vdim, "scale": c.scale}
                if c.rot_dims:
                    m["rot"] = {"dims": c.rot_dims, "base": c.rot_base}
                    if c.stretch:
                        m["rot"]["scaling"] = dict(zip(STRETCH_KEYS, c.stretch))
            else:
                m = {"heads": c.heads, "dim": c.dim, "rot_dim": c.rot_dim, "vdim": c.vdim, "q_rank": c.q_rank,
                     "kv_rank": c.kv_rank, "scale": c.scale, "rot": {"dims": c.rot_dim, "base": c.rot_base}}
                if c.yarn:
                    m["rot"]["scaling"] = dict(zip(YARN_KEYS, c.yarn))
            if L.kind != "lightning" and c.window:
                m["mask"] = {"size": c.window}
            layers.append({"type": L.kind, "mixer": m, "mlp": {"kind": "dense", "ff": L.ff} if L.ff else None})
        d = {"architecture": "Fikerax", "vocab": self.vocab_size, "width": self.hidden, "layers": layers,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embed_scale}}
        if self.loop is not None:
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return d


def _decays(heads: int) -> Tuple[float, ...]:
    """Half-lives from one token to some hundreds, evenly spread over the heads on a log scale."""
    return tuple(math.exp(-(2.0 ** (-8.0 * h / max(1, heads - 1)))) for h in range(heads))


def _stack(heads: int, kv_heads: int, dim: int, q_rank: int, kv_rank: int, rot_dim: int, window: int, ff: int):
    """One lightning layer, a group (attention, latent attention, lightning) to be repeated, one lightning layer."""
    lin = LightningSpec(heads, dim, dim, _decays(heads))
    att = AttnSpec(heads, kv_heads, dim, dim, dim ** 0.5, window, dim, 500000.0, (8.0, 1.0, 4.0, 8192.0))
    lat = LatentSpec(heads, dim, rot_dim, dim, q_rank, kv_rank, (dim + rot_dim) ** -0.5, window, 500000.0,
                     (8.0, 8192.0, 32.0, 1.0))
    return (LayerSpec("lightning", lin), LayerSpec("attention", att, ff), LayerSpec("latent_attention", lat, ff),
            LayerSpec("lightning", lin, ff), LayerSpec("lightning", lin))


PRESETS: Dict[str, FikeraxConfig] = {
    "tiny-fikerax": FikeraxConfig("tiny-fikerax", 8192, 384, _stack(6, 3, 64, 80, 96, 32, 160, 640), embed_scale=18.0,
                                  loop=(1, 4, 2)),
    # sizes of a ~1B-class decoder's layers (benchmarks; random weights): 1 + 3 x 3 + 1 layer runs
    "fikerax-1b": FikeraxConfig("fikerax-1b", 32768, 2048, _stack(16, 2, 128, 768, 256, 64, 1024, 8192),
                                embed_scale=45.0, loop=(1, 4, 3)),
}


class FikeraxModel:
    step_layout = "segments"   # the engine packs steps as segments (ops.seq_ops.SegStepInputs)
    graph_capturable = False

    def __init__(self, cfg: FikeraxConfig, device, dtype=torch.bfloat16, pc: Optional[ParallelContext] = None,
                 seed: int = 0, init: bool = True):
        self.cfg = cfg
        self.device = torch.device(device)
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Fikerax runs in bfloat16 or float32")
        self.dtype = dtype
        self.pc = pc or single()
        if self.pc.tp_size != 1:
            raise ValueError("Fikerax runs on one device per replica (no tensor-parallel sharding of its mixers)")
        self.logits_f32 = True
        self.layers: List[Dict[str, torch.Tensor]] = []
        self.ropes: List[Optional[S.Rope]] = []
        made: Dict[tuple, S.Rope] = {}
        for i, L in enumerate(cfg.layers):
            self._check(i, L)
            c, key, kw = L.mix, None, {}
            if L.kind == "attention" and c.rot_dims:
                key, kw = (False, c.rot_dims, c.rot_base, c.stretch), dict(stretch=c.stretch)
            elif L.kind == "latent_attention" and c.rot_dim:
                key, kw = (True, c.rot_dim, c.rot_base, c.yarn), dict(pairs=True, yarn=c.yarn)
            if key is not None and key not in made:
                made[key] = S.make_rope(key[1], key[2], self.device, **kw)
            self.ropes.append(made.get(key))
        if cfg.loop is not None:
            start, stop, times = cfg.loop
            if not 0 <= start <= stop <= len(cfg.layers) or times < 0:
                raise ValueError("loop: 0 <= start <= stop <= layers, and times not negative")
        # every run of a layer has pages (attention kinds) or a state (lightning) of its own
        self.runs = cfg.runs
        if not self.runs:
            raise ValueError("a model needs at least one layer run")
        self.cache_of: List[Optional[int]] = []
        self.state_of: List[Optional[int]] = []
        self.cached: List[LayerSpec] = []
        n_states = 0
        for i, _ in self.runs:
            lin = cfg.layers[i].kind == "lightning"
            self.state_of.append(n_states if lin else None)
            self.cache_of.append(None if lin else len(self.cached))
            if lin:
                n_states += 1
            else:
                self.cached.append(cfg.layers[i])
        # per-sequence state slots besides cache pages forbid rewinding and page sharing
        self.stateful = n_states > 0
        if init:
            self._random_init(seed)

    @staticmethod
    def _check(i: int, L: LayerSpec) -> None:
        c = L.mix
        if L.kind == "lightning":
            if len(c.decay) != c.heads or any(not 0.0 <= v <= 1.0 for v in c.decay):
                raise ValueError(f"layer {i}: one decay from 0 to 1 per head")
            return
        if c.window < 0:
            raise ValueError(f"layer {i}: a window that is not negative")
        if L.kind == "attention" and (c.heads % c.kv_heads or c.rot_dims % 2 or not 0 <= c.rot_dims <= c.dim):
            raise ValueError(f"layer {i}: heads a multiple of kv_heads, an even rot.dims <= dim")
        if L.kind == "latent_attention" and (c.rot_dim < 0 or c.rot_dim % 2):
            raise ValueError(f"layer {i}: an even rot_dim")

    # ------------------------------------------------------- what the engine allocates for this model
    def _mfma(self, L: LayerSpec) -> bool:
        """Whether the matrix-core kernels run this attention (then its values are also cached transposed)."""
        c = L.mix
        if L.kind == "attention":
            return S.masked_mfma_ok(c.heads, c.kv_heads, c.dim, c.vdim, self.dtype, self.device)
        return bool(S.mfma_tiles(c.kv_rank, self.dtype, self.device, c.tail))

    def _widths(self) -> List[Tuple[int, int]]:
        return [(L.mix.kv_heads * L.mix.dim, L.mix.kv_heads * L.mix.vdim) if L.kind == "attention"
                else (L.mix.kv_rank + L.mix.tail, L.mix.kv_rank) for L in self.cached]

    def cache_bytes_per_block(self, block_size: int) -> int:
        per = sum(k + (v if L.kind == "attention" or self._mfma(L) else 0)
                  for L, (k, v) in zip(self.cached, self._widths()))
        return max(1, per) * block_size * (2 if self.dtype == torch.bfloat16 else 4)

    def make_cache(self, num_blocks: int, block_size: int):
        from ..engine.kv_cache import WindowKVPool
        return WindowKVPool(self._widths(), num_blocks, block_size, self.device, self.dtype,
                            [self._mfma(L) for L in self.cached], twin_only=True,
                            in_keys=[L.kind == "latent_attention" for L in self.cached])

    def state_spec(self) -> Dict[str, Tuple[int, ...]]:
        """Per-slot fp32 state tensors: name -> shape behind the slot dimension."""
        spec: Dict[str, Tuple[int, ...]] = {}
        for (i, _), j in zip(self.runs, self.state_of):
            if j is not None:
                c = self.cfg.layers[i].mix
                spec[f"mem{j}"] = (c.heads, c.dim, c.vdim)
        return spec

    def workspace_bytes(self, tokens: int) -> int:
        w, widest = self.cfg.hidden, 0
        for L in self.cfg.layers:
            c = L.mix
            if L.kind == "lightning":
                n = 4 * c.heads * (c.dim + c.vdim)
            elif L.kind == "attention":
                n = 2 * c.heads * (c.dim + c.vdim) + c.kv_heads * (c.dim + c.vdim)
            else:
                n = 2 * (c.q_rank + c.kv_rank) + c.heads * (c.dim + 2 * c.tail + 2 * c.kv_rank + c.vdim)
            widest = max(widest, n, 3 * L.ff)
        return int(tokens * (4 * w * 4 + widest * 4) + (2 << 30))

    # --------------------------------------------------------------- weights
    def _random_init(self, seed: int) -> None:
        t = random_tensors(self.cfg, seed, self.device)
        self.load_tensors(t.__getitem__)

    def load_tensors(self, get, has=None) -> None:
        """Build the fused device layout from checkpoint tensors (``get(name)`` -> tensor; names of the
        safetensors file: ``embed``, ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.mlp.gate`` ...)."""
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def put(*names, dtype=dt):
            ts = [get(n) for n in names]
            return (ts[0] if len(ts) == 1 else torch.cat(ts, 0)).to(device=dev, dtype=dtype).contiguous()

        def f32(*names):
            return put(*names, dtype=torch.float32)

        def norm(name):                                   # stored around zero
            return 1.0 + f32(name)

        self.embed, self.head, self.final_norm = put("embed"), put("head"), norm("final.norm")
        self.one = torch.ones(1, dtype=torch.float32, device=dev)      # one stream that is only added to
        self.layers = []
        for i, spec in enumerate(cfg.layers):
            p, c = f"l{i}.mix.", spec.mix
            L: Dict[str, torch.Tensor] = {"norm1": norm(f"l{i}.norm1"), "wo": put(p + "o")}
            if spec.kind == "lightning":
                L["w_in"] = put(p + "q", p + "k", p + "v", p + "g")           # one GEMM: q | k | v | gate
                L["decay"] = torch.tensor(c.decay, dtype=torch.float32, device=dev)
                L["mem_norm"] = f32(p + "norm")
            elif spec.kind == "attention":
                L["w_in"] = put(p + "q", p + "k", p + "v")                    # one fp32-out GEMM: q | k | v
                L["b_in"] = f32(p + "q.b", p + "k.b", p + "v.b")
            else:
                H, D, V, KR = c.heads, c.dim, c.vdim, c.kv_rank
                L["w_in"] = put(p + "dq", p + "dkv")                          # query latent | latent | rotated key part
                L["dq_norm"], L["dkv_norm"] = put(p + "dq.norm"), put(p + "dkv.norm")
                L["w_uq"] = put(p + "uq")
                # absorbed forms, per head [D, KR] and [KR, V]
                L["uk"] = put(p + "uk").view(H, D, KR).contiguous()
                L["uv_t"] = put(p + "uv").view(H, V, KR).transpose(1, 2).contiguous()
                L["sink"] = f32(p + "sink")
            if spec.ff:
                L["norm2"] = norm(f"l{i}.norm2")
                L["w13"], L["w2"] = put(f"l{i}.mlp.gate", f"l{i}.mlp.up"), put(f"l{i}.mlp.down")
            self.layers.append(L)

    def weight_bytes(self) -> int:
        ts = [t for L in self.layers for t in L.values()] + [self.embed, self.head, self.final_norm]
        return sum(t.numel() * t.element_size() for t in ts)

    # -------------------------------------------------------------- forward
    def _table(self, i: int, inp: S.SegStepInputs, tables) -> Optional[torch.Tensor]:
        """cos | sin of the step's positions for layer ``i``'s rotation, made once per distinct rotation."""
        rope = self.ropes[i]
        if rope is None:
            return None
        if id(rope) not in tables:
            tables[id(rope)] = S.rope_table(inp.positions, rope)
        return tables[id(rope)]

    def _lightning(self, i: int, h: torch.Tensor, inp: S.SegStepInputs, state: torch.Tensor) -> torch.Tensor:
        L, c = self.layers[i], self.cfg.layers[i].mix
        HV = c.heads * c.vdim
        x = linear(h, L["w_in"])                                             # q | k | v | gate as activations
        o = S.decay_attention(x, c.heads, c.dim, c.vdim, L["decay"], state, inp.seg, silu=True)
        y = S.head_norm_gate(o, x[:, x.shape[1] - HV:], L["mem_norm"], 1, HV, self.cfg.norm_eps, self.dtype)
        return proj_f32out(y, L["wo"])

    def _attention(self, i: int, h: torch.Tensor, inp: S.SegStepInputs, tables, kc, vc, vt) -> torch.Tensor:
        L, c = self.layers[i], self.cfg.layers[i].mix
        x = proj_f32out(h, L["w_in"])
        q = S.attn_prep(x, L["b_in"], c.heads, c.kv_heads, c.dim, c.vdim, inp.positions, inp.slots, kc, vc, self.dtype,
                        norm="head", eps=self.cfg.norm_eps, rope=self.ropes[i], rope_cs=self._table(i, inp, tables), vt=vt)
        o = S.masked_attention(q, c.heads, c.kv_heads, c.dim, c.vdim, kc, vc, inp.seg, c.scale, window=c.window, vt=vt)
        return proj_f32out(o, L["wo"])

    def _latent_attention(self, i: int, h: torch.Tensor, inp: S.SegStepInputs, tables, cache, cache_t) -> torch.Tensor:
        L, c = self.layers[i], self.cfg.layers[i].mix
        T, H, D, R, V, KR = h.shape[0], c.heads, c.dim, c.rot_dim, c.vdim, c.kv_rank
        cs = self._table(i, inp, tables)
        dn = proj_f32out(h, L["w_in"])                                        # [T, q_rank + KR + R] fp32
        cq = S.latent_norm(dn, L["dq_norm"], L["dkv_norm"], inp.slots, cache, c.q_rank, KR, self.cfg.norm_eps, self.dtype,
                           cache_t=cache_t, tail=R, tail_cs=cs)
        q = linear(cq, L["w_uq"])                                             # [T, H (D + R)]
        qr = S.rotated_tail(q, cs, H, D, c.tail) if R else None
        qa = torch.bmm(q.view(T, H, D + R)[:, :, :D].transpose(0, 1), L["uk"]).transpose(0, 1)    # [T, H, KR], head-major
        kw = dict(window=c.window, sink=L["sink"], head_major=True)
        if cache_t is not None:
            o = S.latent_attention_mfma(qa, cache, cache_t, None, inp.seg, inp.positions, c.scale, qr=qr, **kw)
        else:
            o = S.latent_attention(qa.float(), cache, None, inp.seg, c.scale, self.dtype,
                                   qr=qr.float() if qr is not None else None, **kw)
        ov = torch.empty(T, H, V, dtype=self.dtype, device=h.device)
        torch.bmm(o.transpose(0, 1), L["uv_t"], out=ov.transpose(0, 1))       # written token-major: W_o reads it as it is
        return proj_f32out(ov.view(T, H * V), L["wo"])

    def _dense(self, i: int, h: torch.Tensor) -> torch.Tensor:
        L = self.layers[i]
        a = swiglu_gemm(h, L["w13"])                                          # one launch where a fused kernel takes the shape
        if a is None:
            a = M.glu_clamp(linear(h, L["w13"]), 1.0, math.inf, 0.0)          # silu(gate) * up
        return proj_f32out(a, L["w2"])

    def forward(self, inp: S.SegStepInputs, kcs: List[torch.Tensor], vcs: List[Optional[torch.Tensor]],
                vts: List[Optional[torch.Tensor]], states: Optional[Dict[str, torch.Tensor]] = None,
                layers_out: Optional[list] = None) -> torch.Tensor:
        """Logits [len(logits_idx), vocab] fp32.  ``kcs`` / ``vcs`` / ``vts``: the paged keys (latent rows), values and
        transposed values (latents) of every run of an attention layer; ``states``: the per-slot tensors of
        :meth:`state_spec`.  ``layers_out`` (debugging): receives the residual after every layer run."""
        cfg, eps, dt = self.cfg, self.cfg.norm_eps, self.dtype
        T, one = inp.input_ids.shape[0], self.one
        mix1 = one.view(1, 1)
        tables: Dict[int, torch.Tensor] = {}
        again = (inp.input_ids, self.embed, cfg.embed_scale)
        x = torch.empty(T, 1, cfg.hidden, dtype=torch.float32, device=self.device)
        h = N.hyper_embed(inp.input_ids, self.embed, cfg.embed_scale, x, one, self.layers[self.runs[0][0]]["norm1"], eps, dt)
        for r, (i, _) in enumerate(self.runs):
            spec, L, ci = cfg.layers[i], self.layers[i], self.cache_of[r]
            # the write-back of the run's last sublayer also reads the next run's input
            into: dict = {}
            if r + 1 < len(self.runs):
                j, add = self.runs[r + 1]
                into = dict(inn=one, nw=self.layers[j]["norm1"], eps=eps, out_dtype=dt, again=again if add else None)
            if spec.kind == "lightning":
                y = self._lightning(i, h, inp, states[f"mem{self.state_of[r]}"])
            elif spec.kind == "attention":
                y = self._attention(i, h, inp, tables, kcs[ci], vcs[ci], vts[ci])
            else:
                y = self._latent_attention(i, h, inp, tables, kcs[ci], vts[ci])
            if spec.ff:
                h = N.hyper_step(x, y, one, mix1, inn=one, nw=L["norm2"], eps=eps, out_dtype=dt)
                y = self._dense(i, h)
            if layers_out is not None:
                layers_out.append(x[:, 0] + y)
            h = N.hyper_step(x, y, one, mix1, **into)
        return proj_f32out(N.hyper_read(x, inp.logits_idx, self.final_norm, eps, dt), self.head)


def random_tensors(cfg: FikeraxConfig, seed: int = 0, device="cpu") -> Dict[str, torch.Tensor]:
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
                                  "final.norm": rnd(W, std=0.1)}
    for i, L in enumerate(cfg.layers):
        p, c = f"l{i}.mix.", L.mix
        t[f"l{i}.norm1"] = rnd(W, std=0.1)
        if L.kind == "lightning":
            for n, rows in (("q", c.heads * c.dim), ("k", c.heads * c.dim), ("v", c.heads * c.vdim), ("g", c.heads * c.vdim)):
                t[p + n] = lin(rows, W)
            t[p + "norm"], t[p + "o"] = rnd(c.heads * c.vdim, std=0.1, mean=1.0), lin(W, c.heads * c.vdim)
        elif L.kind == "attention":
            for n, rows in (("q", c.heads * c.dim), ("k", c.kv_heads * c.dim), ("v", c.kv_heads * c.vdim)):
                t[p + n], t[p + n + ".b"] = lin(rows, W), rnd(rows, std=0.2)
            t[p + "o"] = lin(W, c.heads * c.vdim)
        else:
            H, KR = c.heads, c.kv_rank
            t[p + "dq"], t[p + "dq.norm"] = lin(c.q_rank, W), rnd(c.q_rank, std=0.1, mean=1.0)
            t[p + "uq"] = lin(H * (c.dim + c.rot_dim), c.q_rank)
            t[p + "dkv"], t[p + "dkv.norm"] = lin(KR + c.rot_dim, W), rnd(KR, std=0.1, mean=1.0)
            t[p + "uk"], t[p + "uv"] = lin(H * c.dim, KR), lin(H * c.vdim, KR)
            t[p + "sink"], t[p + "o"] = rnd(H, std=1.0), lin(W, H * c.vdim)
        if L.ff:
            t[f"l{i}.norm2"] = rnd(W, std=0.1)
            t[f"l{i}.mlp.gate"], t[f"l{i}.mlp.up"], t[f"l{i}.mlp.down"] = lin(L.ff, W), lin(L.ff, W), lin(W, L.ff)
    return t


def load_checkpoint(path: str, device, dtype, pc=None) -> FikeraxModel:
    """A folder with config.json and model.safetensors (bfloat16 weights) -> the model on ``device``."""
    from safetensors import safe_open
    with open(os.path.join(path, "config.json")) as f:
        cfg = FikeraxConfig.from_json(json.load(f), name=os.path.basename(os.path.normpath(path)) or "fikerax")
    model = FikeraxModel(cfg, device, dtype, pc, init=False)
    with safe_open(os.path.join(path, "model.safetensors"), framework="pt", device="cpu") as h:
        model.load_tensors(h.get_tensor, set(h.keys()).__contains__)
    return model


def save_checkpoint(cfg: FikeraxConfig, tensors: Dict[str, torch.Tensor], path: str) -> None:
    """Write config.json + model.safetensors (bfloat16) in the layout :func:`load_checkpoint` reads."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg.to_json(), f, indent=1)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()},
              os.path.join(path, "model.safetensors"))
