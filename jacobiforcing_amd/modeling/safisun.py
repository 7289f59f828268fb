"""Safisun: a decoder with a float residual stream, a norm in front of AND behind every sublayer — x + norm1b(mixer(norm1 x)), then
x + norm2b(ff(norm2 x)) — mostly recurrent mixers, and a span of layers that runs several times with the same weights: in front of every pass
the stream is formed anew from itself and the embedding output, x <- W_in [x; x0] + step[pass], and every pass has caches and states of its
own.

* mixer ``lightning``: linear attention with a fixed decay per head (q, k, v through silu), the heads RMS-normed together, gated by a sigmoid.
* mixer ``mamba2``: the state-space duality — one product for z, x, B, C and dt; x, B, C through a short causal convolution with a bias and silu; a
  step size softplus(dt + bias) and a decay exp(-exp(A_log) dt) per head and token, B and C shared by groups of heads, a skip D x; gated by
  silu(z) BEFORE a norm over equal parts.
* mixer ``parallel``: attention and lightning side by side on the same input, left_scale * left + right_scale * right.  The attention: grouped
  heads with biases, q and k normed over the whole projection, rotation of neighbouring dimensions, tanh-capped scores, positions that see
  their own chunk of the sequence only, one added to the softmax's denominator, a sigmoid gate per head.
* feed-forward ``dense``: down(silu(gate h) * up h); or none.

The forward runs one ragged batch (``layer_ops.RaggedBatch``): portions of prompts and single decoded tokens side by side, over
``engine.state_cache.PagedStateCache``.  Dense products are torch's (hipBLASLt / rocBLAS); everything else is a launch of
``libjf_layers.so`` / ``libjf_layers_seq.so``.  A sublayer's output norm, the residual update and the next sublayer's norm are one launch.
With float32 weights every product is a true 32-bit one."""
from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path
from typing import Any, Dict, List, Optional, Tuple

import torch
import torch.nn.functional as F

from . import read_tensors
from .. import layer_ops as LO
from ..engine.state_cache import PagedStateCache, RunSpec

MIXERS = ("lightning", "mamba2", "parallel")
MAX_TAPS, MAX_STATE_ROWS = 8, 256      # what the convolution and the recurrence kernels take


def _lightning_sizes(m: Dict[str, Any]):
    return int(m["heads"]), int(m["dim"]), int(m["vdim"])


def _attention_sizes(m: Dict[str, Any]):
    return int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])


def _mamba_sizes(m: Dict[str, Any]):
    """heads, groups, state rows, head width, taps, columns of the convolution"""
    H, G, N, Dv = int(m["heads"]), int(m["groups"]), int(m["state"]), int(m["vdim"])
    return H, G, N, Dv, int(m["conv"]), H * Dv + 2 * G * N


def _rot_key(m: Dict[str, Any]):
    rot = m.get("rot") or {}
    return int(rot.get("dims", 0)), float(rot.get("base", 10000.0))


@dataclass
class SafisunConfig:
    vocab_size: int
    hidden_size: int
    layers: List[Dict[str, Any]]
    loop: Optional[Tuple[int, int, int]] = None     # (start, stop, times); None: every layer runs once, nothing in front of it
    norm_eps: float = 1e-5
    max_position_embeddings: int = 1 << 20          # the design has no limit of its own: the engine's max_model_len decides
    eos_token_id: int = -1
    pad_token_id: int = 0
    family: str = "ragged"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "SafisunConfig":
        n, loop = len(d["layers"]), None
        if d.get("loop"):
            loop = tuple(int(d["loop"][k]) for k in ("start", "stop", "times"))
            if not 0 <= loop[0] < loop[1] <= n or loop[2] < 1:
                raise ValueError(f"loop {d['loop']} does not fit {n} layers")

        def lightning(i, m):
            H, D, _ = _lightning_sizes(m)
            if len(m["decay"]) != H:
                raise ValueError(f"layer {i}: {len(m['decay'])} decays for {H} heads")
            if D > MAX_STATE_ROWS:
                raise ValueError(f"layer {i}: a state of {D} rows (up to {MAX_STATE_ROWS} are served)")

        for i, L in enumerate(d["layers"]):
            m = L["mixer"]
            if L["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
            if L["type"] == "lightning":
                lightning(i, m)
            elif L["type"] == "mamba2":
                H, G, N, Dv, taps, _ = _mamba_sizes(m)
                if H % G or (H * Dv) % int(m["norm_groups"]):
                    raise ValueError(f"layer {i}: {H} heads over {G} groups, {H * Dv} channels in {m['norm_groups']} norm parts")
                if not 1 <= taps <= MAX_TAPS or N > MAX_STATE_ROWS:
                    raise ValueError(f"layer {i}: {taps} taps (1 .. {MAX_TAPS} are served), a state of {N} rows (up to {MAX_STATE_ROWS})")
            else:
                a = m["left"]
                H, G, D, _ = _attention_sizes(a)
                dims = _rot_key(a)[0]
                if H % G:
                    raise ValueError(f"layer {i}: {H} heads over {G} key/value heads")
                if dims % 2 or dims > D:
                    raise ValueError(f"layer {i}: rot.dims {dims} must be even and at most dim {D}")
                if int((a.get("mask") or {}).get("size", 0)) < 0:
                    raise ValueError(f"layer {i}: a chunk of {a['mask']['size']} positions")
                lightning(i, m["right"])
            f = L.get("mlp")
            if f is not None and f.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {f.get('kind')!r}")
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=d["layers"], loop=loop, norm_eps=float(d["norm"]["eps"]),
                   eos_token_id=int(d.get("eos_token_id", -1)), pad_token_id=int(d.get("pad_token_id", 0)))

    @classmethod
    def from_json(cls, path) -> "SafisunConfig":
        return cls.from_dict(json.loads(Path(path).read_text()))

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer index, the pass that begins in front of it or None) in execution order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b, times = self.loop
        out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(a)]
        for t in range(times):
            out += [(a, t)] + [(i, None) for i in range(a + 1, b)]
        return out + [(i, None) for i in range(b, n)]


class SafisunWeights:
    """Tensors by their checkpoint names (``embed``, ``loop.in``, ``loop.step``, ``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b``, ``l<i>.mix.*``,
    ``l<i>.mlp.*``, ``final.norm``, ``head``), regrouped per layer for the forward: a mixer's input projections stacked into one matrix (of a
    parallel mixer both sides', with one bias vector), ending with zero rows up to a multiple of eight so that the product's rows start at
    16-byte borders; a parallel mixer's two output projections side by side, so that one product adds both sides; gate and up stacked;
    norm weights, decays and the recurrence's constants in float."""

    def __init__(self, cfg: SafisunConfig, tensors: Dict[str, torch.Tensor], device, dtype=torch.bfloat16):
        dev = torch.device(device)
        W = cfg.hidden_size

        def act(key, *shape):
            t = tensors[key]
            if tuple(t.shape) != shape:
                raise ValueError(f"{key} is {tuple(t.shape)}, the config's sizes give {shape}")
            return t.to(device=dev, dtype=dtype).contiguous()

        def f32(key, *shape):
            t = tensors[key]
            if tuple(t.shape) != shape:
                raise ValueError(f"{key} is {tuple(t.shape)}, the config's sizes give {shape}")
            return t.to(device=dev, dtype=torch.float32).contiguous()

        def stack(mats):
            rows = sum(t.shape[0] for t in mats)
            return torch.cat([*mats, torch.zeros(((-rows) % 8, *mats[0].shape[1:]), dtype=dtype, device=dev)], 0).contiguous()

        self.device, self.dtype = dev, dtype
        self.embed, self.final_norm, self.head = act("embed", cfg.vocab_size, W), f32("final.norm", W), act("head", cfg.vocab_size, W)
        if cfg.loop is not None:
            self.loop_in, self.loop_step = act("loop.in", W, 2 * W), f32("loop.step", cfg.loop[2], W)
        self.layers = []

        def lightning(p, m):
            """input projections q, k, v, gate; their columns; the constants"""
            H, D, Dv = _lightning_sizes(m)
            mats = [act(p + "q", H * D, W), act(p + "k", H * D, W), act(p + "v", H * Dv, W), act(p + "g", H * Dv, W)]
            return mats, (0, H * D, 2 * H * D, 2 * H * D + H * Dv), dict(decay=torch.tensor([float(x) for x in m["decay"]], dtype=torch.float32, device=dev),
                                                                         out_norm=f32(p + "norm", H * Dv)), act(p + "o", W, H * Dv)

        for i, L in enumerate(cfg.layers):
            p, m = f"l{i}.", L["mixer"]
            w: Dict[str, Any] = dict(norm1=f32(p + "norm1", W), norm1b=f32(p + "norm1b", W))
            if L["type"] == "lightning":
                mats, w["cols"], consts, w["w_o"] = lightning(p + "mix.", m)
                w.update(consts, w_in=stack(mats))
            elif L["type"] == "mamba2":
                H, G, N, Dv, taps, C_ = _mamba_sizes(m)
                inner = H * Dv
                w.update(w_in=stack([act(p + "mix.in", inner + C_ + H, W)]), conv=act(p + "mix.conv", C_, taps), conv_b=act(p + "mix.conv.b", C_),
                         dt_bias=f32(p + "mix.dt_bias", H), a_log=f32(p + "mix.A_log", H), skip=f32(p + "mix.D", H), out_norm=f32(p + "mix.norm", inner),
                         w_o=act(p + "mix.o", W, inner))
            else:
                H, G, D, Dv = _attention_sizes(m["left"])
                q = p + "mix.left."
                mats = [act(q + "q", H * D, W), act(q + "k", G * D, W), act(q + "v", G * Dv, W)]
                bias = [act(q + "q.b", H * D), act(q + "k.b", G * D), act(q + "v.b", G * Dv)]
                rows = H * D + G * D + G * Dv
                r_mats, r_cols, consts, r_o = lightning(p + "mix.right.", m["right"])
                # left q | k | v, right q | k | v | gate, the left side's head gates last (their number need not be a multiple of anything)
                w_in = stack(mats + r_mats + [act(q + "g", H, W)])
                g_col = rows + sum(t.shape[0] for t in r_mats)
                w.update(consts, w_in=w_in, b_in=torch.cat(bias + [torch.zeros(w_in.shape[0] - rows, dtype=dtype, device=dev)]), cols=tuple(rows + c for c in r_cols),
                         a_cols=(0, H * D, H * D + G * D, g_col), q_norm=act(q + "q.norm", H * D), k_norm=act(q + "k.norm", G * D),
                         sink=torch.zeros(H, dtype=torch.float32, device=dev), w_o=torch.cat([act(q + "o", W, H * Dv), r_o], 1).contiguous())
            if L.get("mlp") is not None:
                ff = int(L["mlp"]["ff"])
                w.update(norm2=f32(p + "norm2", W), norm2b=f32(p + "norm2b", W), w_gu=torch.cat([act(p + "mlp.gate", ff, W), act(p + "mlp.up", ff, W)], 0),
                         w_down=act(p + "mlp.down", W, ff))
            self.layers.append(w)

    @classmethod
    def from_safetensors(cls, cfg: SafisunConfig, model_dir, device, dtype=torch.bfloat16) -> "SafisunWeights":
        return cls(cfg, read_tensors(model_dir), device, dtype)

    @classmethod
    def random(cls, cfg: SafisunConfig, device, dtype=torch.bfloat16, seed: int = 0) -> "SafisunWeights":
        return cls(cfg, random_tensors(cfg, seed), device, dtype)


def random_tensors(cfg: SafisunConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random tensors under the checkpoint's names (benchmarks and tests; bf16-representable float32 values)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg.hidden_size
    rnd = lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16).float()
    uni = lambda *s, lo=0.0, hi=1.0: (lo + (hi - lo) * torch.rand(*s, generator=g)).to(torch.bfloat16).float()
    lin = lambda o, i: rnd(o, i, std=i ** -0.5)
    one = lambda *s: (1 + torch.randn(*s, generator=g) * 0.1).to(torch.bfloat16).float()
    t = {"embed": rnd(cfg.vocab_size, W), "final.norm": one(W), "head": lin(cfg.vocab_size, W)}
    if cfg.loop is not None:
        t.update({"loop.in": lin(W, 2 * W), "loop.step": rnd(cfg.loop[2], W, std=0.5)})

    def lightning(p, m):
        H, D, Dv = _lightning_sizes(m)
        t.update({p + "q": lin(H * D, W), p + "k": lin(H * D, W), p + "v": lin(H * Dv, W), p + "g": lin(H * Dv, W), p + "o": lin(W, H * Dv), p + "norm": one(H * Dv)})

    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.", L["mixer"]
        t.update({p + "norm1": one(W), p + "norm1b": one(W)})
        if L["type"] == "lightning":
            lightning(p + "mix.", m)
        elif L["type"] == "mamba2":
            H, G, N, Dv, taps, C_ = _mamba_sizes(m)
            t.update({p + "mix.in": lin(H * Dv + C_ + H, W), p + "mix.conv": rnd(C_, taps, std=0.5), p + "mix.conv.b": rnd(C_, std=0.2), p + "mix.dt_bias": rnd(H),
                      p + "mix.A_log": uni(H, lo=-3.0, hi=1.0), p + "mix.D": rnd(H), p + "mix.norm": one(H * Dv), p + "mix.o": lin(W, H * Dv)})
        else:
            H, G, D, Dv = _attention_sizes(m["left"])
            q = p + "mix.left."
            t.update({q + "q": lin(H * D, W), q + "k": lin(G * D, W), q + "v": lin(G * Dv, W), q + "q.b": rnd(H * D, std=0.2), q + "k.b": rnd(G * D, std=0.2),
                      q + "v.b": rnd(G * Dv, std=0.2), q + "q.norm": one(H * D), q + "k.norm": one(G * D), q + "g": lin(H, W), q + "o": lin(W, H * Dv)})
            lightning(p + "mix.right.", m["right"])
        if L.get("mlp") is not None:
            ff = int(L["mlp"]["ff"])
            t.update({p + "norm2": one(W), p + "norm2b": one(W), p + "mlp.gate": lin(ff, W), p + "mlp.up": lin(ff, W), p + "mlp.down": lin(W, ff)})
    return t


class SafisunModel:
    def __init__(self, cfg: SafisunConfig, weights: SafisunWeights, max_positions: int = 8192):
        self.cfg, self.w = cfg, weights
        self.device, self.dtype = weights.device, weights.dtype
        self.runs = cfg.runs()
        self._angles: Dict[tuple, tuple] = {}
        self.max_positions = 0
        self.reserve_positions(max_positions)

    # ---- what the cache must hold, one entry per layer run (a repeated layer has a state, and a pool, per pass) --------------------------
    def cache_specs(self) -> List[RunSpec]:
        specs = []
        for li, _ in self.runs:
            L, m = self.cfg.layers[li], self.cfg.layers[li]["mixer"]
            if L["type"] == "lightning":
                specs.append(RunSpec("state", state_shape=_lightning_sizes(m)))
            elif L["type"] == "mamba2":                 # the float state per head, and the convolution's last inputs
                H, G, N, Dv, taps, C_ = _mamba_sizes(m)
                specs.append(RunSpec("state", state_shape=(H, N, Dv), tails={"conv": (taps - 1, C_)}))
            else:                                       # a pool for the left side, a state for the right
                H, G, D, Dv = _attention_sizes(m["left"])
                specs.append(RunSpec("kv+state", k_width=G * D, v_width=G * Dv, state_shape=_lightning_sizes(m["right"])))
        return specs

    def new_cache(self, num_pages: int, page_size: int, num_slots: int) -> PagedStateCache:
        return PagedStateCache(self.cache_specs(), num_pages, page_size, num_slots, self.device, self.dtype)

    # ---- rotation angles for every position the engine can reach: position * frequency, cosine and sine, all in float32 -----------------
    def reserve_positions(self, n: int) -> None:
        if n <= self.max_positions:
            return
        self.max_positions = int(n)
        self._angles.clear()
        for L in self.cfg.layers:
            if L["type"] != "parallel":
                continue
            key = _rot_key(L["mixer"]["left"])
            if key[0] and key not in self._angles:
                dims, base = key
                f = torch.tensor([base ** (-2.0 * k / dims) for k in range(dims // 2)], dtype=torch.float32, device=self.device)
                a = torch.arange(n, dtype=torch.float32, device=self.device).view(n, 1) * f.view(1, -1)
                self._angles[key] = (a.cos().contiguous(), a.sin().contiguous())

    # ---- mixers: from the norm's output to the mixer's result (behind its output projection) ----------------------------------------------
    def _linear_attention(self, m, w, proj: torch.Tensor, run: int, batch: LO.RaggedBatch, cache: PagedStateCache, scale: float, out: Optional[torch.Tensor]) -> torch.Tensor:
        """Lightning attention on the columns ``w["cols"]`` of a product, up to (not with) its output projection."""
        H, D, Dv = _lightning_sizes(m)
        cols = w["cols"]
        raw = LO.linear_scan(proj, cols[:3], batch, H, H, D, Dv, cache.state[run], act=LO.ACT_SILU, decay=w["decay"])
        return LO.gated_norm(raw, proj[:, cols[3]:cols[3] + H * Dv], w["out_norm"], self.cfg.norm_eps, LO.ACT_SIGMOID, False, scale=scale, out=out)

    def _lightning(self, run: int, li: int, h: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache) -> torch.Tensor:
        w = self.w.layers[li]
        return F.linear(self._linear_attention(self.cfg.layers[li]["mixer"], w, F.linear(h, w["w_in"]), run, batch, cache, 1.0, None), w["w_o"])

    def _mamba2(self, run: int, li: int, h: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache) -> torch.Tensor:
        m, w = self.cfg.layers[li]["mixer"], self.w.layers[li]
        H, G, N, Dv, taps, C_ = _mamba_sizes(m)
        inner = H * Dv
        proj = F.linear(h, w["w_in"])                   # z | x | B | C | dt
        xbc = LO.short_conv(proj, inner, C_, w["conv"], batch, cache.tails[run].get("conv"), LO.ACT_SILU, bias=w["conv_b"], out_dtype=self.dtype)
        y = LO.linear_scan(xbc, (inner + G * N, inner, 0), batch, H, G, N, Dv, cache.state[run], dt=proj[:, inner + C_:inner + C_ + H], a_log=w["a_log"],
                           dt_bias=w["dt_bias"], skip=w["skip"])
        return F.linear(LO.gated_norm(y, proj[:, :inner], w["out_norm"], self.cfg.norm_eps, LO.ACT_SILU, True, parts=int(m["norm_groups"])), w["w_o"])

    def _attention(self, m, w, proj: torch.Tensor, run: int, batch: LO.RaggedBatch, cache: PagedStateCache, scale: float, out: torch.Tensor) -> torch.Tensor:
        """The parallel mixer's left side on its columns of the product, up to (not with) its output projection."""
        H, G, D, Dv = _attention_sizes(m)
        key, kp, vp, cols = _rot_key(m), cache.k[run], cache.v[run], w["a_cols"]
        cos, sin = self._angles[key] if key[0] else (None, None)
        q = LO.qk_norm_append(proj, cols[:3], H, G, D, Dv, w["q_norm"], w["k_norm"], self.cfg.norm_eps, kp, vp, batch.kv_slot, rot_dims=key[0],
                              pairing=LO.ROT_NEIGHBOURS, batch=batch, cos=cos, sin=sin)
        kw = dict(sink=w["sink"], gate_per_head=True, chunk=int((m.get("mask") or {}).get("size", 0)), softcap=float(m.get("softcap") or 0.0), out_scale=scale, out=out)
        gate = proj[:, cols[3]:cols[3] + H]
        if LO.attn_sweep_tile_rows(self.dtype, H, G, D, Dv, kp, vp) > 0:      # bfloat16, head sizes the one-sweep matrix-core kernel takes
            return LO.attn_sweep(q, kp, vp, batch, H, G, D, Dv, float(m["scale"]), 0, gate=gate, **kw)
        return LO.attn_window(q, gate, kp, vp, batch, H, G, D, Dv, float(m["scale"]), 0, 0, None, None, None, **kw)

    def _parallel(self, run: int, li: int, h: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache) -> torch.Tensor:
        m, w = self.cfg.layers[li]["mixer"], self.w.layers[li]
        H, _, _, Dv = _attention_sizes(m["left"])
        n, left, width = h.shape[0], H * Dv, w["w_o"].shape[1]
        proj = F.linear(h, w["w_in"], w["b_in"])
        # both sides write their columns of one matrix, scaled; the output product over all of them is the weighted sum.  Rows start at
        # 16-byte borders; the right side starts where the left one ends
        both = torch.empty((n, width + (-width) % 8), dtype=h.dtype, device=h.device)[:, :width]
        self._attention(m["left"], w, proj, run, batch, cache, float(m["left_scale"]), both[:, :left])
        self._linear_attention(m["right"], w, proj, run, batch, cache, float(m["right_scale"]), both[:, left:])
        return F.linear(both, w["w_o"])

    # ---- one step ----------------------------------------------------------------------------------------------------------------------
    @torch.inference_mode()
    def forward(self, ids: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache, logit_rows: Optional[torch.Tensor] = None,
                trace: Optional[list] = None) -> torch.Tensor:
        """ids int64 [N] (the batch's rows).  Returns float logits [N, vocab], or of the rows in ``logit_rows``.  ``trace``, when a
        list, receives the residual stream after every layer run (debugging and tests)."""
        cfg, w, eps, dt = self.cfg, self.w, self.cfg.norm_eps, self.dtype
        if batch.max_pos > self.max_positions:
            raise ValueError(f"position {batch.max_pos - 1} is beyond the {self.max_positions} positions the tables were reserved for")
        x, _ = LO.embed_scale(w.embed, ids, 1.0, False)
        n, W = x.shape
        again = None
        if cfg.loop is not None:                         # [x; x0] in the products' dtype: the right half stays, the left is written in front of each pass
            again = torch.empty((n, 2 * W), dtype=dt, device=self.device)
            again[:, W:] = x
        pending = None                                   # the last sublayer's output and its norm's weight, folded into the next norm's launch

        def norm(w_next, add_row=None):
            nonlocal pending
            y, wb = pending or (None, None)
            pending = None
            return LO.sandwich_norm(x, y, wb, eps, w_next, dt, add_row=add_row)

        for run, (li, begins) in enumerate(self.runs):
            L, lw = cfg.layers[li], w.layers[li]
            step = None
            if begins is not None:
                y, wb = pending or (None, None)
                pending = None
                LO.sandwich_norm(x, y, wb, eps, out=again[:, :W], plain=True)
                x, step = LO.product_f32(again, w.loop_in), w.loop_step[begins]
            h = norm(lw["norm1"], step)
            mixer = self._lightning if L["type"] == "lightning" else self._mamba2 if L["type"] == "mamba2" else self._parallel
            pending = (mixer(run, li, h, batch, cache), lw["norm1b"])
            if L.get("mlp") is not None:
                ff = int(L["mlp"]["ff"])
                h = norm(lw["norm2"])
                pending = (F.linear(LO.gated_act(F.linear(h, lw["w_gu"]), 0, ff, ff, LO.ACT_SILU), lw["w_down"]), lw["norm2b"])
            if trace is not None:
                LO.sandwich_norm(x, *pending, eps)
                pending = None
                trace.append(x.clone())
        hl = norm(w.final_norm)
        if logit_rows is not None:
            hl = hl.index_select(0, logit_rows)
        return F.linear(hl, w.head).float()


def load_model_directory(model_dir, device, dtype=torch.bfloat16, max_positions: int = 8192):
    cfg = SafisunConfig.from_json(Path(model_dir) / "config.json")
    return cfg, SafisunModel(cfg, SafisunWeights.from_safetensors(cfg, model_dir, device, dtype), max_positions)


def random_model(cfg: SafisunConfig, device, dtype=torch.bfloat16, max_positions: int = 8192, seed: int = 0) -> SafisunModel:
    return SafisunModel(cfg, SafisunWeights.random(cfg, device, dtype, seed), max_positions)
