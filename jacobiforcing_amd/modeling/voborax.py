"""Voborax: a decoder with a float residual stream in which each sublayer reads the stream itself and a LAYER norm sits on its output —
x += m * norm(sublayer(x)), m one number, the norm centred with a weight per channel — and whose mixers are all latent attention: queries,
keys and values go through low-rank latents, and the pool keeps only the normalised key/value latent (and, where there is one, a rotary key
part shared by the heads).

* mixer ``latent_attention``: a rotary part beside the latent (neighbouring dimensions form the rotation's pairs), a sliding window, a sigmoid
  gate per head on the outputs.  A layer with ``kv_from`` has no key/value latent and no pool of its own: it attends over the pool of that
  earlier layer with its own queries, up-projections, window and gate.
* mixer ``latent_attention_2``: no positions at all, plain causal, a learned sink per head in the softmax's denominator.
* feed-forward ``dense``: down(gelu_tanh(up x)), both with biases; ``moe``: softmax router over experts and identity experts (which hand
  their input through), the largest scores + correction chosen, weights = the chosen scores renormalised; experts down(silu(gate x) * up x); a
  shared expert of the same form for every token; or none.
* output: the same layer norm, then an untied head.

The forward runs one ragged batch (``layer_ops.RaggedBatch``): portions of prompts and single decoded tokens side by side, over
``engine.state_cache.PagedStateCache``.  Dense products are torch's (hipBLASLt / rocBLAS); everything else is a launch of
``libjf_layers.so`` / ``libjf_layers_seq.so``.  The query is multiplied by the key up-projection, so attention runs over the pool with one
key/value head and the value up-projection follows it.  A sublayer's output norm, the residual update, the identity experts' share and what the
next sublayer reads are one launch.  With float32 weights every product is a true 32-bit one."""
from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path
from typing import Any, Dict, List, Optional

import torch
import torch.nn.functional as F

from . import read_tensors
from .. import layer_ops as LO
from ..engine.state_cache import PagedStateCache, RunSpec

WINDOWED, CAUSAL = "latent_attention", "latent_attention_2"
ROUTER_RENORM_EPS = 1e-20            # a constant of the design's router


@dataclass
class VoboraxConfig:
    vocab_size: int
    hidden_size: int
    layers: List[Dict[str, Any]]
    norm_eps: float = 1e-5
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    max_position_embeddings: int = 1 << 20          # the design has no limit of its own: the engine's max_model_len decides
    eos_token_id: int = -1
    pad_token_id: int = 0
    family: str = "ragged"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def pool_layer(self, i: int) -> int:
        """The layer whose pool layer i attends over: itself, or the one it borrows from."""
        j = self.layers[i]["mixer"].get("kv_from")
        return i if j is None else int(j)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "VoboraxConfig":
        layers = d["layers"]
        for i, L in enumerate(layers):
            if L["type"] not in (WINDOWED, CAUSAL):
                raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
            m = L["mixer"]
            dims, rd = _rot_key(m)[0], _rot_dim(L)
            if dims % 2 or dims > rd:
                raise ValueError(f"layer {i}: rot.dims {dims} must be even and at most rot_dim {rd}")
            j = m.get("kv_from")
            if j is not None:
                o = layers[int(j)] if 0 <= int(j) < i else None
                if (o is None or L["type"] != WINDOWED or o["type"] != WINDOWED or o["mixer"].get("kv_from") is not None or
                        int(o["mixer"]["kv_rank"]) != int(m["kv_rank"]) or _rot_dim(o) != rd or _rot_key(o["mixer"]) != _rot_key(m)):
                    raise ValueError(f"layer {i}: kv_from must name an earlier {WINDOWED} layer with latents of its own, of the same kv_rank, rot_dim and rotation")
            f = L.get("mlp")
            if f is not None and f.get("kind", "dense") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward {f.get('kind')!r}")
            if f is not None and f.get("kind") == "moe" and not 1 <= int(f["router"]["top"]) <= sum(_experts(f)):
                raise ValueError(f"layer {i}: top {f['router']['top']} of {sum(_experts(f))} experts")
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers, norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)), residual_mult=float(d.get("residual_mult", 1.0)),
                   eos_token_id=int(d.get("eos_token_id", -1)), pad_token_id=int(d.get("pad_token_id", 0)))

    @classmethod
    def from_json(cls, path) -> "VoboraxConfig":
        return cls.from_dict(json.loads(Path(path).read_text()))


def _rot_key(m: Dict[str, Any]):
    rot = m.get("rot") or {}
    return int(rot.get("dims", 0)), float(rot.get("base", 10000.0))


def _rot_dim(L: Dict[str, Any]) -> int:
    return int(L["mixer"]["rot_dim"]) if L["type"] == WINDOWED else 0


def _experts(f: Dict[str, Any]):
    """(experts with weights, identity experts)."""
    return int(f["router"]["experts"]), int(f["router"].get("identity", 0))


class VoboraxWeights:
    """Tensors by their checkpoint names (``embed``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``, ``head``), regrouped per
    layer for the forward: a mixer's input projections (query latent, key/value latent with the rotary key, head gate) stacked into one matrix
    that ends with zero rows up to a multiple of eight, the latent up-projections per head ([H, D, R] for keys, [H, R, Dv] for values), every
    expert's gate rows on its up rows ([E, 2*ff, W]), the shared expert's likewise; stream norms, sinks, router and correction in float."""

    def __init__(self, cfg: VoboraxConfig, tensors: Dict[str, torch.Tensor], device, dtype=torch.bfloat16):
        dev = torch.device(device)

        def take(name, shape, dt):
            t = tensors[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name} is {tuple(t.shape)}, the config's sizes give {tuple(shape)}")
            return t.to(device=dev, dtype=dt).contiguous()

        act = lambda name, *shape: take(name, shape, dtype)
        f32 = lambda name, *shape: take(name, shape, torch.float32)
        self.device, self.dtype = dev, dtype
        W = cfg.hidden_size
        self.embed, self.head, self.final_norm = act("embed", cfg.vocab_size, W), act("head", cfg.vocab_size, W), f32("final.norm", W)
        self.layers = []
        for i, L in enumerate(cfg.layers):
            p, m = f"l{i}.", L["mixer"]
            H, D, Dv, R, Rq = (int(m[k]) for k in ("heads", "dim", "vdim", "kv_rank", "q_rank"))
            rd, own = _rot_dim(L), cfg.pool_layer(i) == i
            rows = [act(p + "mix.dq", Rq, W)]
            if own:
                rows.append(act(p + "mix.dkv", R + rd, W))
            if L["type"] == WINDOWED:
                rows.append(act(p + "mix.g", H, W))
            n = sum(r.shape[0] for r in rows)
            rows.append(torch.zeros(((-n) % 8, W), dtype=dtype, device=dev))
            w = dict(norm1=f32(p + "norm1", W), w_in=torch.cat(rows, 0), kv_col=Rq, g_col=Rq + (R + rd if own else 0), dq_norm=act(p + "mix.dq.norm", Rq),
                     dkv_norm=act(p + "mix.dkv.norm", R) if own else None, w_uq=act(p + "mix.uq", H * (D + rd), Rq),
                     w_uk=act(p + "mix.uk", H * D, R).view(H, D, R), w_uv=act(p + "mix.uv", H * Dv, R).view(H, Dv, R).transpose(1, 2).contiguous(),
                     w_o=act(p + "mix.o", W, H * Dv), sink=f32(p + "mix.sink", H) if L["type"] == CAUSAL else None)
            f = L.get("mlp")
            if f is not None:
                w["norm2"] = f32(p + "norm2", W)
            if f is not None and f.get("kind", "dense") == "dense":
                ff = int(f["ff"])
                w.update(w_up=act(p + "mlp.up", ff, W), b_up=act(p + "mlp.up.b", ff), w_down=act(p + "mlp.down", W, ff), b_down=act(p + "mlp.down.b", W))
            elif f is not None:
                (E, ident), ff = _experts(f), int(f["expert"]["ff"])
                w.update(router=f32(p + "mlp.router", E + ident, W), correction=f32(p + "mlp.correction", E + ident),
                         w_gu=torch.stack([torch.cat([act(p + f"mlp.e{e}.gate", ff, W), act(p + f"mlp.e{e}.up", ff, W)], 0) for e in range(E)]).contiguous(),
                         w_down=torch.stack([act(p + f"mlp.e{e}.down", W, ff) for e in range(E)]).contiguous())
                if f.get("shared") is not None:
                    fs = int(f["shared"]["ff"])
                    w.update(w_sh=torch.cat([act(p + "mlp.shared.gate", fs, W), act(p + "mlp.shared.up", fs, W)], 0), w_sh_down=act(p + "mlp.shared.down", W, fs))
            self.layers.append(w)

    @classmethod
    def from_safetensors(cls, cfg: VoboraxConfig, model_dir, device, dtype=torch.bfloat16) -> "VoboraxWeights":
        return cls(cfg, read_tensors(model_dir), device, dtype)

    @classmethod
    def random(cls, cfg: VoboraxConfig, device, dtype=torch.bfloat16, seed: int = 0) -> "VoboraxWeights":
        return cls(cfg, random_tensors(cfg, seed), device, dtype)


def random_tensors(cfg: VoboraxConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random tensors under the checkpoint's names (benchmarks and tests; bf16-representable float32 values)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg.hidden_size
    rnd = lambda *s, std=1.0: (torch.randn(*s, generator=g) * std).to(torch.bfloat16).float()
    lin = lambda o, i: rnd(o, i, std=i ** -0.5)
    one = lambda *s: (1 + torch.randn(*s, generator=g) * 0.1).to(torch.bfloat16).float()
    t = {"embed": rnd(cfg.vocab_size, W, std=W ** -0.5), "final.norm": one(W), "head": lin(cfg.vocab_size, W)}
    for i, L in enumerate(cfg.layers):
        p, m = f"l{i}.", L["mixer"]
        H, D, Dv, R, Rq = (int(m[k]) for k in ("heads", "dim", "vdim", "kv_rank", "q_rank"))
        rd = _rot_dim(L)
        t.update({p + "norm1": one(W), p + "mix.dq": lin(Rq, W), p + "mix.dq.norm": one(Rq), p + "mix.uq": lin(H * (D + rd), Rq),
                  p + "mix.uk": lin(H * D, R), p + "mix.uv": lin(H * Dv, R), p + "mix.o": lin(W, H * Dv)})
        if cfg.pool_layer(i) == i:
            t.update({p + "mix.dkv": lin(R + rd, W), p + "mix.dkv.norm": one(R)})
        if L["type"] == WINDOWED:
            t[p + "mix.g"] = lin(H, W)
        else:
            t[p + "mix.sink"] = rnd(H)
        f = L.get("mlp")
        if f is None:
            continue
        t[p + "norm2"] = one(W)
        if f.get("kind", "dense") == "dense":
            ff = int(f["ff"])
            t.update({p + "mlp.up": lin(ff, W), p + "mlp.up.b": rnd(ff, std=0.1), p + "mlp.down": lin(W, ff), p + "mlp.down.b": rnd(W, std=0.1)})
            continue
        (E, ident), ff = _experts(f), int(f["expert"]["ff"])
        t.update({p + "mlp.router": lin(E + ident, W) * 2, p + "mlp.correction": rnd(E + ident, std=0.05)})
        for e in range(E):
            t.update({p + f"mlp.e{e}.gate": lin(ff, W), p + f"mlp.e{e}.up": lin(ff, W), p + f"mlp.e{e}.down": lin(W, ff)})
        if f.get("shared") is not None:
            fs = int(f["shared"]["ff"])
            t.update({p + "mlp.shared.gate": lin(fs, W), p + "mlp.shared.up": lin(fs, W), p + "mlp.shared.down": lin(W, fs)})
    return t


class VoboraxModel:
    def __init__(self, cfg: VoboraxConfig, weights: VoboraxWeights, max_positions: int = 8192):
        self.cfg, self.w = cfg, weights
        self.device, self.dtype = weights.device, weights.dtype
        self._angles: Dict[tuple, tuple] = {}
        self.max_positions = 0
        self.reserve_positions(max_positions)

    # ---- what the cache must hold, one entry per layer: a layer that attends over another's latents holds nothing ------------------------
    def cache_specs(self) -> List[RunSpec]:
        return [RunSpec("kv", k_width=int(L["mixer"]["kv_rank"]) + _rot_dim(L), v_width=0) if self.cfg.pool_layer(i) == i else RunSpec(None)
                for i, L in enumerate(self.cfg.layers)]

    def new_cache(self, num_pages: int, page_size: int, num_slots: int) -> PagedStateCache:
        return PagedStateCache(self.cache_specs(), num_pages, page_size, num_slots, self.device, self.dtype)

    # ---- rotation angles for every position the engine can reach: position * frequency, cosine and sine, all in float32 -----------------
    def reserve_positions(self, n: int) -> None:
        if n <= self.max_positions:
            return
        self.max_positions = int(n)
        self._angles.clear()
        for L in self.cfg.layers:
            key = _rot_key(L["mixer"])
            if L["type"] == WINDOWED and key[0] and key not in self._angles:
                dims, base = key
                f = torch.tensor([base ** (-2.0 * k / dims) for k in range(dims // 2)], dtype=torch.float32, device=self.device)
                a = torch.arange(n, dtype=torch.float32, device=self.device).view(n, 1) * f.view(1, -1)
                self._angles[key] = (a.cos().contiguous(), a.sin().contiguous())

    # ---- mixer: both kinds; what one of them has not (rotation, window, gate; sink) is absent from its launches ---------------------------
    def _mixer(self, li: int, h: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache) -> torch.Tensor:
        L, w, eps = self.cfg.layers[li], self.w.layers[li], self.cfg.norm_eps
        m, rd = L["mixer"], _rot_dim(L)
        H, D, Dv, R, Rq = (int(m[k]) for k in ("heads", "dim", "vdim", "kv_rank", "q_rank"))
        windowed, src = L["type"] == WINDOWED, self.cfg.pool_layer(li)
        key = _rot_key(m) if windowed else (0, 0.0)
        cos, sin = self._angles[key] if key[0] else (None, None)
        n, pool = h.shape[0], cache.k[src]
        proj = F.linear(h, w["w_in"])
        cq = LO.latent_prep(proj, 0, Rq, w["kv_col"], R, rd, key[0], w["dq_norm"], w["dkv_norm"], eps, batch, cos, sin, pool if src == li else None,
                            pairing=LO.ROT_NEIGHBOURS)
        q = F.linear(cq, w["w_uq"])
        qa = torch.bmm(q.view(n, H, D + rd)[:, :, :D].transpose(0, 1), w["w_uk"])                  # [H, N, R]: query . (W_uk c) = (W_uk^T query) . c
        qf = LO.latent_q_pack(qa, q, H, D, R, rd, key[0], batch, cos, sin, pairing=LO.ROT_NEIGHBOURS)
        gate = proj[:, w["g_col"]:w["g_col"] + H] if windowed else None
        window = int((m.get("mask") or {}).get("size", 0)) if windowed else 0
        ov = LO.latent_attend(qf, pool, w["w_uv"], batch, H, R, rd, float(m["scale"]), window, sink=w["sink"], gate=gate)
        return F.linear(LO.heads_gate(ov, None), w["w_o"])

    # ---- feed-forward: the addends of its output, and the choices among which there are identity experts ----------------------------------
    def _feed_forward(self, li: int, h: torch.Tensor, x: torch.Tensor):
        """``h`` the stream in the products' dtype, ``x`` the stream itself (float): the router and the identity experts read that."""
        f, w = self.cfg.layers[li]["mlp"], self.w.layers[li]
        if f.get("kind", "dense") == "dense":
            z = F.linear(h, w["w_up"], w["b_up"])
            return [(F.linear(LO.gated_act(z, 0, -1, z.shape[1], LO.ACT_GELU_TANH), w["w_down"], w["b_down"]), None)], None
        E, ident = _experts(f)
        y = LO.moe_experts(h, F.linear(x, w["router"]), w["correction"], int(f["router"]["top"]), 1.0, w["w_gu"], w["w_down"], route="softmax_renorm",
                           renorm_eps=ROUTER_RENORM_EPS, gated=(LO.ACT_SILU, 0.0, 1.0, 0.0), identity=ident)
        y, choices = (y[0], (y[1], y[2], E)) if ident else (y, None)
        out = [(y, None)]
        if f.get("shared") is not None:
            fs = int(f["shared"]["ff"])
            out.append((F.linear(LO.gated_act(F.linear(h, w["w_sh"]), 0, fs, fs, LO.ACT_SILU), w["w_sh_down"]), None))
        return out, choices

    # ---- one step ----------------------------------------------------------------------------------------------------------------------
    @torch.inference_mode()
    def forward(self, ids: torch.Tensor, batch: LO.RaggedBatch, cache: PagedStateCache, logit_rows: Optional[torch.Tensor] = None,
                trace: Optional[list] = None) -> torch.Tensor:
        """ids int64 [N] (the batch's rows).  Returns float logits [N, vocab], or of the rows in ``logit_rows``.  ``trace``, when a
        list, receives the residual stream after every layer (debugging and tests)."""
        cfg, w, eps, dt = self.cfg, self.w, self.cfg.norm_eps, self.dtype
        if batch.max_pos > self.max_positions:
            raise ValueError(f"position {batch.max_pos - 1} is beyond the {self.max_positions} positions the tables were reserved for")
        wide = dt == torch.float32                       # float products read the stream itself, 16-bit ones a rounded copy of it
        x, h = LO.embed_scale(w.embed, ids, cfg.embedding_scale, not wide, copy_dtype=dt)
        steps = [(li, norm) for li, L in enumerate(cfg.layers) for norm in (("norm1", "norm2") if L.get("mlp") is not None else ("norm1",))]
        for k, (li, norm) in enumerate(steps):
            h = x if wide else h
            y, choices = ([(self._mixer(li, h, batch, cache), None)], None) if norm == "norm1" else self._feed_forward(li, h, x)
            last = k == len(steps) - 1                   # behind the last sublayer comes the model's own norm
            h = LO.output_norm(x, y, w.layers[li][norm], eps, LO.NORM_LAYER, cfg.residual_mult, w.final_norm if last else None, None if wide and not last else dt,
                               choices=choices)
            if trace is not None and (last or steps[k + 1][0] != li):
                trace.append(x.clone())
        if not steps:
            h = LO.output_norm(x, [], None, eps, LO.NORM_LAYER, w_next=w.final_norm, out_dtype=dt)
        if logit_rows is not None:
            h = h.index_select(0, logit_rows)
        return F.linear(h, w.head).float()


def load_model_directory(model_dir, device, dtype=torch.bfloat16, max_positions: int = 8192):
    cfg = VoboraxConfig.from_json(Path(model_dir) / "config.json")
    return cfg, VoboraxModel(cfg, VoboraxWeights.from_safetensors(cfg, model_dir, device, dtype), max_positions)


def random_model(cfg: VoboraxConfig, device, dtype=torch.bfloat16, max_positions: int = 8192, seed: int = 0) -> VoboraxModel:
    return VoboraxModel(cfg, VoboraxWeights.random(cfg, device, dtype, seed), max_positions)
