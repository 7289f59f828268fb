"""Voborax through the package (HIP layer kernels, paged pools, borrowed latents, ragged step, scheduler, LLM.generate, trace replay) against
the plain oracle ``oracle/voborax_oracle.py``, which shares no code with it.  Small random models of several shapes; where random weights
would hide a fault (a far key among hundreds, a key at a window's or page's edge, the sink) the weights and inputs are chosen so that it
shows, and the test checks on the oracle that it does.

CPU tests cover the oracle's own pieces, the config reader and the cache layout; everything that launches a kernel is marked ``gpu``."""
import copy
import importlib.machinery
import importlib.util
import io
import json
import random
from pathlib import Path

import numpy as np
import pytest
import torch

from oracle import voborax_oracle as O
from jacobiforcing_amd.modeling import MODEL_REGISTRY, read_model_config, read_tensors
from jacobiforcing_amd.modeling import voborax as VB

gpu = pytest.mark.gpu


# ---- model shapes -----------------------------------------------------------------------------------------------------------------
def win(heads=3, dim=16, rot=8, vdim=24, rank=40, qrank=28, size=11, base=300.0, scale=0.25, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": qrank, "scale": scale, "mask": {"size": size},
         "rot": {"dims": rot, "base": base}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def cau(heads=4, dim=24, vdim=20, rank=48, qrank=36, scale=0.2):
    return {"type": "latent_attention_2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "q_rank": qrank, "scale": scale}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, identity=2, top=3, ff=24, shared=40):
    f = {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top}, "expert": {"ff": ff}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def make_cfg(layers, width=96, vocab=131, eps=1e-5, emb=3.0, mult=0.6):
    return {"architecture": "Voborax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "embedding": {"scale": emb}, "residual_mult": mult}


def shape_a():
    """Both mixers; two layers borrow from one owner that lies further back, with other head counts, head sizes, query ranks, scales and
    windows than the owner; dense and expert feed-forwards and a layer without one."""
    return make_cfg([dict(win(), mlp=dense()), dict(cau(), mlp=moe()), dict(win(heads=5, dim=12, vdim=16, qrank=44, size=5, scale=0.3, kv_from=0), mlp=moe(top=2)),
                     dict(win(heads=2, rank=24, rot=6, size=30, base=1e4), mlp=None),
                     dict(win(heads=1, dim=20, vdim=40, qrank=20, size=19, kv_from=0), mlp=dense(24)), dict(cau(heads=1, dim=8, vdim=8, rank=20, qrank=12), mlp=None)])


def shape_b():
    """Windows of one and of more than any sequence; one expert chosen, every expert chosen, no identity expert, no shared expert; sizes that
    are no multiples of eight; multipliers of one; a causal layer first and a borrowing layer last."""
    return make_cfg([dict(cau(heads=7, dim=10, vdim=6, rank=33, qrank=15), mlp=moe(3, 1, 1, 20, 0)), dict(win(heads=2, dim=6, rot=10, vdim=14, rank=18, qrank=9, size=1), mlp=moe(4, 3, 7, 33, 10)),
                     dict(win(heads=3, dim=9, rot=2, vdim=5, rank=26, qrank=31, size=5000), mlp=moe(6, 0, 2, 12, 18)),
                     dict(win(heads=4, dim=4, rot=2, vdim=11, rank=26, qrank=8, size=7, kv_from=2), mlp=None)], width=66, vocab=77, eps=1e-6, emb=1.0, mult=1.0)


def shape_c():
    """Latents the one-sweep matrix-core kernel takes in bfloat16, many heads; a borrower in the very next layer."""
    return make_cfg([dict(win(heads=8, dim=32, rot=16, vdim=48, rank=64, qrank=96, size=40, base=1e6, scale=0.14), mlp=moe(9, 3, 4, 16, 32)),
                     dict(win(heads=16, dim=16, rot=16, vdim=16, rank=64, qrank=64, size=21, base=1e6, scale=0.17, kv_from=0), mlp=dense(48)),
                     dict(cau(heads=12, dim=48, vdim=32, rank=96, qrank=80, scale=0.15), mlp=dense(64))], width=128, vocab=50, mult=0.4, emb=7.0)


SHAPES = {"a": shape_a, "b": shape_b, "c": shape_c}


def tensors_for(cfg_dict, seed):
    return VB.random_tensors(VB.VoboraxConfig.from_dict(cfg_dict), seed)


def layer_tensors(t, i, dtype=torch.float64):
    return {k[len(f"l{i}."):]: v.to(dtype) for k, v in t.items() if k.startswith(f"l{i}.")}


def rel_err(got, want):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    return float(np.sqrt(((got - want) ** 2).mean()) / max(np.sqrt((want ** 2).mean()), 1e-30))


F32_TOL, BF16_TOL = 2e-4, 6e-2


def rows_off(got, want, tol):
    """Fraction of rows (positions) whose own relative error is above ``tol``.  In bfloat16 a router's close call may go the other way for a
    token, and a norm behind a sublayer divides by that sublayer's size, so a test over random models bounds how many rows differ."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    err = np.sqrt(((got - want) ** 2).mean(-1)) / np.maximum(np.sqrt((want ** 2).mean(-1)), 1e-30)
    return float((err > tol).mean())


def toks(n, vocab, seed):
    return [random.Random(seed * 7919 + i).randrange(vocab) for i in range(n)]


# =====================================================================================================================================
# CPU: oracle pieces, config reader, cache layout
# =====================================================================================================================================
def test_registry_reads_the_architecture_key(tmp_path):
    assert MODEL_REGISTRY["Voborax"][2] == "ragged"
    (tmp_path / "config.json").write_text(json.dumps(shape_a()))
    cfg = read_model_config(tmp_path)
    assert isinstance(cfg, VB.VoboraxConfig) and cfg.family == "ragged" and cfg.num_hidden_layers == 6
    assert (cfg.embedding_scale, cfg.residual_mult, cfg.norm_eps, cfg.vocab_size, cfg.hidden_size) == (3.0, 0.6, 1e-5, 131, 96)
    assert [cfg.pool_layer(i) for i in range(6)] == [0, 1, 0, 3, 0, 5]


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0].update(type="attention"), lambda c: c["layers"][0]["mlp"].update(kind="polynomial"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=8), lambda c: c["layers"][1]["mlp"]["router"].update(top=0),
    lambda c: c["layers"][2]["mixer"].update(kv_from=2), lambda c: c["layers"][2]["mixer"].update(kv_from=3), lambda c: c["layers"][2]["mixer"].update(kv_from=1),
    lambda c: c["layers"][4]["mixer"].update(kv_from=2), lambda c: c["layers"][2]["mixer"].update(kv_rank=41), lambda c: c["layers"][2]["mixer"].update(rot_dim=10),
    lambda c: c["layers"][2]["mixer"]["rot"].update(base=301.0), lambda c: c["layers"][2]["mixer"].update(kv_from=-1)])
def test_config_rejects_what_the_design_does_not_have(change):
    bad = copy.deepcopy(shape_a())
    change(bad)
    with pytest.raises(ValueError):
        VB.VoboraxConfig.from_dict(bad)


def test_cache_layout_and_stacked_weights():
    cfg = VB.VoboraxConfig.from_dict(shape_a())
    t = tensors_for(shape_a(), 1)
    assert "l2.mix.dkv" not in t and "l2.mix.g" in t and "l1.mix.sink" in t and "l1.mix.g" not in t and "l3.norm2" not in t
    w = VB.VoboraxWeights(cfg, t, "cpu", torch.float32)
    specs = VB.VoboraxModel(cfg, w, max_positions=16).cache_specs()
    assert [s.kind for s in specs] == ["kv", "kv", None, "kv", None, "kv"] and [s.k_width for s in specs] == [48, 48, 0, 30, 0, 20]
    assert all(s.v_width == 0 for s in specs)
    l0, l1, l2 = w.layers[:3]
    assert tuple(l0["w_in"].shape) == (80, 96) and (l0["kv_col"], l0["g_col"]) == (28, 76) and not l0["w_in"][79:].any()       # 28 + 48 + 3 rows, one of zeros
    assert tuple(l1["w_in"].shape) == (88, 96) and l1["sink"].dtype == torch.float32 and l0["sink"] is None
    assert tuple(l2["w_in"].shape) == (56, 96) and l2["g_col"] == 44 and l2["dkv_norm"] is None
    assert tuple(l0["w_uk"].shape) == (3, 16, 40) and tuple(l0["w_uv"].shape) == (3, 40, 24) and torch.equal(l0["w_uv"][1].T, t["l0.mix.uv"][24:48])
    assert tuple(l1["w_gu"].shape) == (5, 48, 96) and tuple(l1["w_sh"].shape) == (80, 96) and l1["router"].dtype == torch.float32 and l1["correction"].numel() == 7
    assert "w_sh" not in VB.VoboraxWeights(VB.VoboraxConfig.from_dict(shape_b()), tensors_for(shape_b(), 1), "cpu").layers[0]
    for name in ("l0.mix.dkv", "l1.mlp.e2.up", "l1.mlp.correction", "l0.mlp.up.b", "head"):
        bad = dict(t)
        bad[name] = bad[name][:-1]
        with pytest.raises(ValueError):
            VB.VoboraxWeights(cfg, bad, "cpu")
    from jacobiforcing_amd.engine.state_cache import PagedStateCache
    cache = PagedStateCache(specs, 4, 8, 3, "cpu", torch.float32)
    assert cache.k[2] is None and cache.v == [None] * 6 and cache.bytes() == 4 * 32 * (48 + 48 + 30 + 20)


def test_reading_tensors_needs_a_file(tmp_path):
    from safetensors.torch import save_file
    with pytest.raises(FileNotFoundError):
        read_tensors(tmp_path)
    save_file({"a": torch.ones(2)}, str(tmp_path / "x.safetensors"))
    save_file({"b": torch.zeros(3)}, str(tmp_path / "y.safetensors"))
    assert sorted(read_tensors(tmp_path)) == ["a", "b"]


def test_oracle_pieces():
    g = torch.Generator().manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    z = torch.tensor([-3.0, 0.0, 0.5, 2.0], dtype=torch.float64)
    F = torch.nn.functional
    assert torch.allclose(O.gelu_tanh(z), F.gelu(z, approximate="tanh")) and torch.allclose(O.silu(z), F.silu(z))
    x, w = rn(4, 9) + 5, rn(9)
    assert torch.allclose(O.layer_norm(x, w, 1e-5), F.layer_norm(x, (9,), w, None, 1e-5)) and torch.allclose(O.rms_norm(x, w, 1e-5), F.rms_norm(x, (9,), w, 1e-5))
    r = rn(5, 2, 6)
    t = O.rotate(r, 50.0)
    assert torch.allclose(t[0], r[0]) and torch.allclose((t * t).sum(-1), (r * r).sum(-1))
    a = 3 * torch.tensor(50.0, dtype=torch.float64) ** (-2 / 6)
    assert abs(float(t[3, 1, 2] - (r[3, 1, 2] * a.cos() - r[3, 1, 3] * a.sin()))) < 1e-12 and abs(float(t[3, 1, 3] - (r[3, 1, 3] * a.cos() + r[3, 1, 2] * a.sin()))) < 1e-12
    see = O.visible(5, 2)
    assert see.sum(-1).tolist() == [1, 2, 2, 2, 2] and see[3].tolist() == [False, False, True, True, False] and O.visible(5).sum(-1).tolist() == [1, 2, 3, 4, 5]
    s, sink = rn(2, 4, 4), torch.tensor([0.5, -30.0], dtype=torch.float64)
    wt = O.masked_softmax(s, O.visible(4), sink)
    e = torch.exp(s[0, 2, :3])
    assert torch.allclose(wt[0, 2, :3], e / (e.sum() + torch.exp(sink[0]))) and torch.allclose(wt[1], O.masked_softmax(s, O.visible(4))[1])
    # the correction moves the choice, the weights come from the scores alone and sum to one
    zr, corr = torch.tensor([[2.0, 1.0, 0.5, 0.0]], dtype=torch.float64), torch.tensor([-1.0, 0.0, 0.0, 1.0], dtype=torch.float64)
    idx, wr = O.route(zr, corr, 2)
    sc = torch.softmax(zr, -1)[0]
    assert idx.tolist() == [[3, 1]] and torch.allclose(wr[0], torch.stack([sc[3], sc[1]]) / (sc[3] + sc[1]))
    # a token whose every choice is an identity expert passes through
    cfg = moe(2, 2, 2, 4, 0)
    P = {k: v.double() for k, v in layer_tensors(tensors_for(make_cfg([dict(win(), mlp=cfg)], width=8), 3), 0).items()}
    P["mlp.correction"] = torch.tensor([0.0, 0.0, 5.0, 5.0], dtype=torch.float64)
    h = rn(3, 8)
    assert torch.allclose(O.routed_feed_forward(h, P, cfg), h)


# =====================================================================================================================================
# GPU: the package against the oracle
# =====================================================================================================================================
class Rig:
    """A model on the GPU with a pool of shuffled pages; runs steps of (request, tokens) and keeps the bookkeeping a test needs."""

    def __init__(self, cfg_dict, seed=0, dtype=torch.float32, page=8, pages=64, slots=4, tensors=None, max_positions=1024):
        from jacobiforcing_amd import layer_ops as LO
        self.LO = LO
        self.cfg_dict = cfg_dict
        self.cfg = VB.VoboraxConfig.from_dict(cfg_dict)
        self.tensors = tensors or tensors_for(cfg_dict, seed)
        self.model = VB.VoboraxModel(self.cfg, VB.VoboraxWeights(self.cfg, self.tensors, "cuda", dtype), max_positions=max_positions)
        self.page = page
        self.cache = self.model.new_cache(pages, page, slots)
        self.free_pages = list(range(pages))
        random.Random(seed).shuffle(self.free_pages)
        self.free_slots = list(range(slots))[::-1]
        self.req = {}

    def poison(self):
        """Fill the pools with large values: whatever a kernel reads without having written it shows."""
        for t in self.cache.k:
            if t is not None:
                t.fill_(1e4)

    def batch(self, entries):
        counts, starts, slots, tables, ids = [], [], [], [], []
        for key, tk in entries:
            r = self.req.setdefault(key, {"n": 0, "pages": [], "slot": None})
            if r["slot"] is None:
                r["slot"] = self.free_slots.pop()
            while len(r["pages"]) * self.page < r["n"] + len(tk):
                r["pages"].append(self.free_pages.pop())
            counts.append(len(tk)); starts.append(r["n"]); slots.append(r["slot"]); tables.append(r["pages"])
            ids += list(tk)
            r["n"] += len(tk)
        return self.LO.RaggedBatch.build(counts, starts, slots, tables, self.page, "cuda"), ids

    def step(self, entries, trace=None):
        """entries = [(key, tokens)]; returns logits [sum of tokens, vocab] (float, on the CPU)."""
        b, ids = self.batch(entries)
        return self.model.forward(torch.tensor(ids, device="cuda"), b, self.cache, None, trace).cpu()

    def run(self, key, tokens, cuts):
        """One request in portions of the given sizes; the rest, if any, token by token."""
        got, at = [], 0
        for n in list(cuts) + [1] * (len(tokens) - sum(cuts)):
            got.append(self.step([(key, tokens[at:at + n])]))
            at += n
        return torch.cat(got)

    def end(self, key):
        r = self.req.pop(key)
        self.free_pages += r["pages"][::-1]
        self.free_slots.append(r["slot"])

    def oracle(self, tokens, trace=None):
        return O.forward(self.cfg_dict, self.tensors, list(tokens), torch.float64, trace)


# ---- mechanisms alone -----------------------------------------------------------------------------------------------------------------
@gpu
@pytest.mark.parametrize("W", [50, 96, 200, 1000, 2052, 4096, 8000, 9001])
@pytest.mark.parametrize("kind", ["rms", "layer"])
def test_output_norm_update_and_what_comes_next(W, kind):
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(W)
    rn = lambda *s: torch.randn(*s, generator=g)
    code, norm = (LO.NORM_RMS, O.rms_norm) if kind == "rms" else (LO.NORM_LAYER, O.layer_norm)
    n, E, top = 5, 3, 4
    x, y1, y2, ye, w, wn, sc = rn(n, W), rn(n, W) * 3 + 2, rn(n, 2, W).to(torch.bfloat16), rn(n, top, W), rn(W), rn(W), rn(W)
    xd = x.double()
    # one addend, a rounded one and a scaled one with several rows; the stream itself, its norm, or nothing behind the update
    want = xd + 0.7 * norm(y1.double(), w.double(), 1e-5)
    xg = x.cuda()
    assert LO.output_norm(xg, [(y1.cuda(), None)], w.cuda(), 1e-5, code, 0.7) is None and rel_err(xg.cpu(), want) < 1e-6
    xg = x.cuda()
    o = LO.output_norm(xg, [(y1.cuda(), None)], w.cuda(), 1e-5, code, 0.7, None, torch.bfloat16)
    assert rel_err(xg.cpu(), want) < 1e-6 and torch.equal(o, xg.to(torch.bfloat16))
    want = xd + 0.3 * norm(y1.double() + sc.double() * y2.double().sum(1), w.double(), 1e-6)
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 6e-3)):
        xg = x.cuda()
        o = LO.output_norm(xg, [(y1.cuda(), None), (y2.cuda(), sc.cuda())], w.cuda(), 1e-6, code, 0.3, wn.cuda(), dtype)
        assert rel_err(xg.cpu(), want) < 1e-6 and rel_err(o.float().cpu(), norm(want, wn.double(), 1e-6)) < tol
    # choices among identity experts: their rows are not read (here: not a number), weight * x stands in for them
    ids = torch.tensor([[0, 1, 2, 0], [3, 1, 4, 0], [4, 3, 5, 6], [2, 2, 2, 3], [9, 0, 1, 2]], dtype=torch.int32)
    wts = torch.rand(n, top, generator=g)
    dead = (ids >= E).unsqueeze(-1)
    experts = torch.where(dead, wts.double().unsqueeze(-1) * xd.unsqueeze(1), ye.double()).sum(1)
    xg = x.cuda()
    LO.output_norm(xg, [(ye.masked_fill(dead, float("nan")).cuda(), None), (y1.cuda(), None)], w.cuda(), 1e-5, code, 1.0, choices=(ids.cuda(), wts.cuda(), E))
    assert rel_err(xg.cpu(), xd + norm(experts + y1.double(), w.double(), 1e-5)) < 1e-6
    # no addend: nothing is updated; eps sits inside the root; a row far from zero keeps its deviations
    keep = xg.clone()
    assert rel_err(LO.output_norm(xg, [], None, 1e-5, code, w_next=wn.cuda(), out_dtype=torch.float32).cpu(), norm(keep.cpu().double(), wn.double(), 1e-5)) < 2e-6
    assert torch.equal(LO.output_norm(xg, [], None, 1e-5, code, out_dtype=torch.float32), keep) and torch.equal(xg, keep)
    tiny = torch.zeros(1, W)
    tiny[0, ::2] = 2e-3
    assert rel_err(LO.output_norm(tiny.cuda(), [], None, 1e-5, code, w_next=wn.cuda(), out_dtype=torch.float32).cpu(), norm(tiny.double(), wn.double(), 1e-5)) < 2e-6
    far = (rn(2, W) + 1000.0)
    got = LO.output_norm(far.cuda(), [], None, 1e-5, code, w_next=wn.cuda(), out_dtype=torch.float32).cpu()
    assert rel_err(got, norm(far.double(), wn.double(), 1e-5)) < (2e-4 if kind == "layer" else 1e-6)
    with pytest.raises(ValueError):
        LO.output_norm(xg, [(y1.cuda(), None)], None, 1e-5, code)
    with pytest.raises(ValueError):
        LO.output_norm(xg, [(y1.cuda(), None)], w.cuda(), 1e-5, code, choices=(ids.cuda(), wts.cuda(), E))


@gpu
def test_embedding_with_a_rounded_copy():
    from jacobiforcing_amd import layer_ops as LO
    e = torch.randn(11, 37)
    ids = torch.tensor([3, 0, 10, 3]).cuda()
    for dtype in (torch.float32, torch.bfloat16):
        x, c = LO.embed_scale(e.to(dtype).cuda(), ids, 2.5, True, copy_dtype=torch.bfloat16)
        assert torch.equal(x, e.to(dtype).float().cuda()[ids] * 2.5) and torch.equal(c, x.to(torch.bfloat16))
    assert LO.embed_scale(e.cuda(), ids, 2.5, False)[1] is None and torch.equal(*LO.embed_scale(e.cuda(), ids, 2.5, True))


ROUTED = [(5, 2, 3, 24), (1, 1, 1, 8), (7, 0, 2, 33), (3, 6, 9, 16), (16, 4, 4, 40), (2, 30, 5, 16), (70, 30, 66, 8), (2, 1100, 6, 8), (1, 4000, 3, 8)]


@gpu
@pytest.mark.parametrize("E,ident,top,ff", ROUTED)
@pytest.mark.parametrize("n", [1, 70, 300])
def test_router_experts_and_identity_experts(E, ident, top, ff, n):
    """The router's choice with its correction, the grouped products over the experts that have weights, and the sum with the identity
    experts' share inside the norm's launch — up to thousands of router outputs (several per lane of the router's wavefront)."""
    from jacobiforcing_amd import layer_ops as LO
    W, n = 48, min(n, 20 if top > 60 else n)
    f = moe(E, ident, top, ff, 0)
    t = tensors_for(make_cfg([dict(win(), mlp=f)], width=W), 7)
    t["l0.mlp.correction"] = torch.randn(E + ident, generator=torch.Generator().manual_seed(2)) * 0.2
    P = layer_tensors(t, 0)
    x = torch.randn(n, W, generator=torch.Generator().manual_seed(n))
    want_ids, want_w = O.route(x.double() @ P["mlp.router"].T, P["mlp.correction"], top)
    if E + ident > 2 and top < E + ident and n > 1:
        plain, _ = O.route(x.double() @ P["mlp.router"].T, torch.zeros(E + ident, dtype=torch.float64), top)
        assert not torch.equal(plain.sort(-1)[0], want_ids.sort(-1)[0])                          # the correction decides some choices
    want = x.double() + 0.5 * O.layer_norm(O.routed_feed_forward(x.double(), P, f), P["norm2"], 1e-5)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        w = VB.VoboraxWeights(VB.VoboraxConfig.from_dict(make_cfg([dict(win(), mlp=f)], width=W)), t, "cuda", dtype).layers[0]
        xg = x.cuda()
        res = LO.moe_experts(xg.to(dtype), torch.nn.functional.linear(xg, w["router"]), w["correction"], top, 1.0, w["w_gu"], w["w_down"], route="softmax_renorm",
                             renorm_eps=1e-20, gated=(LO.ACT_SILU, 0.0, 1.0, 0.0), identity=ident)
        y, ids, wts = res if ident else (res, None, None)
        if ident:
            assert torch.equal(ids.cpu().long().sort(-1)[0], want_ids.sort(-1)[0])
            assert torch.allclose(wts.cpu().double().sort(-1)[0], want_w.sort(-1)[0], rtol=1e-5) and torch.allclose(wts.sum(-1).cpu(), torch.ones(n))
        LO.output_norm(xg, [(y, None)], w["norm2"], 1e-5, LO.NORM_LAYER, 0.5, choices=(ids, wts, E) if ident else None)
        assert rel_err(xg.cpu(), want) < tol, dtype


@gpu
def test_a_correction_does_not_enter_the_weights_and_ties_go_to_the_lowest_index():
    from jacobiforcing_amd import layer_ops as LO
    W, E = 16, 4
    gu, dn = torch.zeros(E, 16, W, device="cuda"), torch.zeros(E, W, 8, device="cuda")
    z = torch.tensor([[1.0, 1.0, 1.0, 1.0, 1.0, 1.0]], device="cuda")
    run = lambda c: LO.moe_experts(torch.zeros(1, W, device="cuda"), z, torch.tensor(c, device="cuda"), 2, 1.0, gu, dn, route="softmax_renorm", renorm_eps=1e-20,
                                   gated=(LO.ACT_SILU, 0.0, 1.0, 0.0), identity=2)[1:]
    ids, w = run([0.0] * 6)
    assert ids.tolist() == [[0, 1]] and torch.allclose(w.cpu(), torch.full((1, 2), 0.5))
    ids, w = run([0.0, 0.0, 0.0, 0.5, 0.0, 0.9])
    assert ids.tolist() == [[5, 3]] and torch.allclose(w.cpu(), torch.full((1, 2), 0.5))


@gpu
@pytest.mark.parametrize("H,R,rd,Rq", [(3, 40, 8, 28), (1, 33, 0, 15), (5, 24, 6, 600), (8, 512, 64, 96), (40, 16, 16, 20)])
def test_latent_stages(H, R, rd, Rq):
    """Norms, rotation and append; the query latent alone (a layer that borrows); query packing — with a rotated part and without one."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(R)
    n, D, base = 9, 12, 70.0
    ld = Rq + R + rd + 3
    proj, wq, wk = torch.randn(n, ld, generator=g), torch.randn(Rq, generator=g), torch.randn(R, generator=g)
    start = 5
    b = LO.RaggedBatch.build([n], [start], [0], [[2, 0, 3]], 8, "cuda")
    ang = torch.arange(64, dtype=torch.float32).view(-1, 1) * torch.tensor([base ** (-2.0 * k / max(rd, 1)) for k in range(rd // 2)]).view(1, -1)
    cos, sin = (ang.cos().cuda().contiguous(), ang.sin().cuda().contiguous()) if rd else (None, None)
    turn = lambda v: O.rotate(torch.cat([torch.zeros(start, *v.shape[1:], dtype=torch.float64), v]), base)[start:] if rd else v
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        p_, q_, k_ = proj.to(dtype), wq.to(dtype), wk.to(dtype)
        pool = torch.full((32, R + rd), 7.0, dtype=dtype, device="cuda")
        cq = LO.latent_prep(p_.cuda(), 0, Rq, Rq, R, rd, rd, q_.cuda(), k_.cuda(), 1e-5, b, cos, sin, pool, pairing=LO.ROT_NEIGHBOURS)
        d = p_.double()
        want_q = O.rms_norm(d[:, :Rq], q_.double(), 1e-5)
        want = torch.cat([O.rms_norm(d[:, Rq:Rq + R], k_.double(), 1e-5), turn(d[:, Rq + R:Rq + R + rd].unsqueeze(1))[:, 0]], -1)
        where = b.kv_slot.cpu()
        assert rel_err(cq.float().cpu(), want_q) < tol and rel_err(pool.float().cpu()[where], want) < tol
        rest = torch.ones(32, dtype=torch.bool)
        rest[where] = False
        assert bool((pool.cpu()[rest] == 7.0).all())
        alone = LO.latent_prep(p_.cuda(), 0, Rq, Rq, R, rd, rd, q_.cuda(), None, 1e-5, b, cos, sin, None, pairing=LO.ROT_NEIGHBOURS)
        assert rel_err(alone.float().cpu(), want_q) < tol
        qa, q = torch.randn(H, n, R, generator=g).to(dtype), torch.randn(n, H * (D + rd), generator=g).to(dtype)
        qf = LO.latent_q_pack(qa.cuda(), q.cuda(), H, D, R, rd, rd, b, cos, sin, pairing=LO.ROT_NEIGHBOURS).float().cpu().view(n, H, R + rd)
        assert torch.equal(qf[..., :R], qa.float().transpose(0, 1)) and (rd == 0 or rel_err(qf[..., R:], turn(q.double().view(n, H, D + rd)[..., D:])) < tol)
    with pytest.raises(ValueError):
        LO.latent_prep(proj.cuda(), 0, 0, 0, R, rd, rd, None, wk.cuda(), 1e-5, b, cos, sin, None)


ATTEND = [(3, 40, 8), (5, 33, 4), (8, 64, 16), (16, 128, 32), (6, 144, 16), (12, 200, 0), (4, 512, 64), (40, 96, 0), (64, 512, 64), (20, 80, 24)]


@gpu
@pytest.mark.parametrize("H,R,rd", ATTEND)
@pytest.mark.parametrize("window", [0, 1, 17, 500])
def test_attention_over_the_latents_at_every_kind_of_size(H, R, rd, window):
    """``latent_attend`` — whichever launches the sizes lead to — with a window, a sink and a gate per head against the sums written out: a long
    portion, a short one and single tokens whose keys are shared out over workgroups (each must count the sink once)."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(H * 1000 + R + rd)
    page, Dv, scale = 16, 8, 0.9 / (R + rd) ** 0.5
    starts, counts = [0, 180, 399], [37, 2, 1]
    per = 26
    order = torch.randperm(3 * per, generator=g).tolist()
    tables = [order[b * per:(b + 1) * per] for b in range(3)]
    n = sum(counts)
    pool, q = torch.randn(3 * per * page, R + rd, generator=g), torch.randn(n, H * (R + rd), generator=g)
    gate, sink, w_uv = torch.randn(n, H + 3, generator=g), torch.randn(H, generator=g) + 3, torch.randn(H, R, Dv, generator=g) * R ** -0.5
    b = LO.RaggedBatch.build(counts, starts, [0, 1, 2], tables, page, "cuda")
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        pd, qd, gd, wd = (t.to(dtype) for t in (pool, q, gate, w_uv))
        for use_sink, use_gate in ((True, False), (False, True), (True, True)):
            got = LO.latent_attend(qd.cuda(), pd.cuda(), wd.cuda(), b, H, R, rd, scale, window, sink=sink.cuda() if use_sink else None,
                                   gate=gd.cuda()[:, 1:1 + H] if use_gate else None).float().cpu()
            want, r = torch.zeros(H, n, Dv, dtype=torch.float64), 0
            for bb in range(3):
                rows = torch.tensor([tables[bb][p // page] * page + p % page for p in range(starts[bb] + counts[bb])])
                kv = pd[rows].double()
                for t in range(counts[bb]):
                    i = starts[bb] + t
                    lo = max(0, i - window + 1) if window else 0
                    s = (qd[r].double().view(H, R + rd) @ kv[lo:i + 1].T) * scale
                    if use_sink:
                        s = torch.cat([s, sink.double().view(H, 1)], 1)
                    p = torch.softmax(s, -1)[:, :i + 1 - lo]
                    o = p @ kv[lo:i + 1, :R]
                    if use_gate:
                        o = o * torch.sigmoid(gd[r, 1:1 + H].double()).view(H, 1)
                    want[:, r] = torch.bmm(o.unsqueeze(1), wd.double())[:, 0]
                    r += 1
            assert rel_err(got, want) < tol, (dtype, use_sink, use_gate)
            assert rel_err(got[:, -1], want[:, -1]) < 2 * tol


@gpu
@pytest.mark.parametrize("H,R,rd", [(16, 64, 16), (12, 128, 32), (40, 96, 0)])
@pytest.mark.parametrize("window", [0, 90])
def test_long_portions_take_the_wide_tiles(H, R, rd, window):
    """Hundreds of tokens per request in bfloat16: the 128-row form of the one-sweep kernel over the latents, with sink and gate, beside a portion
    that starts inside a sequence."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(H)
    page, Dv, scale, bf = 64, 8, 0.9 / (R + rd) ** 0.5, torch.bfloat16
    starts, counts = [0, 300], [700, 410]
    tables = [list(range(12))[::-1], list(range(12, 24))]
    pool, q = torch.randn(24 * page, R + rd, generator=g).to(bf), torch.randn(sum(counts), H * (R + rd), generator=g).to(bf)
    gate, sink, w_uv = torch.randn(sum(counts), H, generator=g).to(bf), torch.randn(H, generator=g) + 3, (torch.randn(H, R, Dv, generator=g) * R ** -0.5).to(bf)
    b = LO.RaggedBatch.build(counts, starts, [0, 1], tables, page, "cuda")
    tq = LO.attn_sweep_tile_rows(bf, H, 1, R + rd, R, pool.cuda(), pool.cuda()[:, :R])
    assert b.tiles(tq).shape[0] * -(-H // 32) >= LO.SWEEP_SPLIT_BELOW_GROUPS                        # what makes the launch choose the wide form
    got = LO.latent_attend(q.cuda(), pool.cuda(), w_uv.cuda(), b, H, R, rd, scale, window, sink=sink.cuda(), gate=gate.cuda()).float().cpu()
    r = 0
    for bb in range(2):
        n, T = counts[bb], starts[bb] + counts[bb]
        kv = pool[torch.tensor([tables[bb][p // page] * page + p % page for p in range(T)])].double()
        s = torch.einsum("ihd,jd->hij", q[r:r + n].double().view(n, H, R + rd), kv) * scale
        w = O.masked_softmax(s, O.visible(T, window or None)[starts[bb]:], sink.double())
        o = torch.einsum("hij,jr->hir", w, kv[:, :R]) * torch.sigmoid(gate[r:r + n].double()).T.unsqueeze(-1)
        want = torch.bmm(o, w_uv.double())
        assert rel_err(got[:, r:r + n], want) < 2e-2
        err = ((got[:, r:r + n].double() - want) ** 2).mean((0, 2)).sqrt() / (want ** 2).mean((0, 2)).sqrt()
        assert float(err.max()) < 6e-2
        r += n


MIXER_SIZES = [win(), win(1, 20, 6, 10, 33, 17, 1), win(5, 12, 2, 16, 40, 44, 9), win(8, 32, 32, 32, 64, 96, 30, 1e4, 0.125), win(16, 64, 16, 64, 128, 64, 64, scale=0.1),
               win(2, 8, 24, 40, 96, 20, 33), win(3, 16, 16, 8, 144, 24, 70, scale=0.2), win(12, 48, 64, 48, 512, 160, 50, scale=0.1),
               cau(), cau(1, 8, 8, 20, 12), cau(7, 10, 6, 33, 15), cau(8, 32, 48, 64, 96), cau(12, 64, 32, 96, 80, 0.12), cau(20, 16, 16, 200, 40), cau(33, 8, 8, 32, 24)]


def mixer_name(L):
    return ("w" if "rot_dim" in L["mixer"] else "c") + "-".join(str(v) for v in L["mixer"].values() if not isinstance(v, (dict, float)))


@gpu
@pytest.mark.parametrize("layer", MIXER_SIZES, ids=mixer_name)
def test_each_mixer_alone_in_portions_and_single_tokens(layer):
    """One mixer on the oracle's own inputs, float32 and bfloat16: a prompt's first part in one step, a second part that starts inside a page,
    two tokens, single tokens, then a long portion, on shuffled poisoned pages."""
    W, T = 64, 84
    cfg = make_cfg([dict(layer, mlp=None)], width=W, vocab=40)
    t = tensors_for(cfg, 5)
    P, m = layer_tensors(t, 0), layer["mixer"]
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(7))
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        rig = Rig(cfg, tensors=t, dtype=dtype, pages=16)
        rig.poison()
        hd = h.cuda().to(dtype)
        ho = hd.cpu().double()
        want = O.windowed_latent_attention(ho, P, m, 1e-5, O.latents(ho, P, m, 1e-5)) if "rot_dim" in m else O.causal_latent_attention(ho, P, m, 1e-5)
        got, at = [], 0
        for n in (19, 14, 2, 1, 1, 1, 5, 41):
            b, _ = rig.batch([("r", [0] * n)])
            got.append(rig.model._mixer(0, hd[at:at + n].contiguous(), b, rig.cache).float().cpu())
            at += n
        assert rel_err(torch.cat(got), want) < tol, dtype


@gpu
@pytest.mark.parametrize("f", [dense(), dense(33), moe(), moe(3, 1, 1, 20, 0), moe(4, 0, 4, 32, 16), moe(2, 5, 3, 12, 30)], ids=str)
def test_each_feed_forward_alone(f):
    W = 48
    cfg = make_cfg([dict(win(), mlp=f)], width=W, mult=0.8)
    t = tensors_for(cfg, 9)
    P = layer_tensors(t, 0)
    x = torch.randn(40, W, generator=torch.Generator().manual_seed(3)) * 2
    y = O.dense_feed_forward(x.double(), P) if f["kind"] == "dense" else O.routed_feed_forward(x.double(), P, f)
    want = x.double() + 0.8 * O.layer_norm(y, P["norm2"], 1e-5)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        rig = Rig(cfg, tensors=t, dtype=dtype)
        xg = x.cuda()
        ys, choices = rig.model._feed_forward(0, xg.to(dtype), xg)
        rig.LO.output_norm(xg, ys, rig.model.w.layers[0]["norm2"], 1e-5, rig.LO.NORM_LAYER, 0.8, choices=choices)
        assert rel_err(xg.cpu(), want) < tol, dtype


# ---- whole models ---------------------------------------------------------------------------------------------------------------------
@gpu
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompt_and_every_layer(name):
    rig = Rig(SHAPES[name](), seed=3)
    t = toks(37, rig.cfg.vocab_size, 1)
    tr_o, tr_g = [], []
    want = rig.oracle(t, tr_o)
    got = rig.step([("r", t)], tr_g)
    assert len(tr_g) == len(tr_o) == rig.cfg.num_hidden_layers
    for li, (g_, o_) in enumerate(zip(tr_g, tr_o)):
        assert rel_err(g_.cpu(), o_) < F32_TOL, li
    assert rel_err(got, want) < F32_TOL


@gpu
@pytest.mark.parametrize("name,tol,share", [("a", 0.1, 0.1), ("b", 0.15, 0.25), ("c", 0.1, 0.1)])
def test_whole_prompt_in_bfloat16(name, tol, share):
    rig = Rig(SHAPES[name](), seed=3, dtype=torch.bfloat16)
    rig.poison()
    t = toks(150, rig.cfg.vocab_size, 1)
    want = rig.oracle(t)
    assert rows_off(rig.step([("r", t)]), want, tol) <= share
    assert rows_off(rig.run("s", t, [60, 2, 71]), want, tol) <= share


@gpu
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_prefill_equals_token_by_token_decoding(name):
    rig = Rig(SHAPES[name](), seed=5)
    rig.poison()
    t = toks(45, rig.cfg.vocab_size, 2)
    want = rig.oracle(t)
    assert rel_err(rig.run("r", t, []), want) < F32_TOL
    assert rel_err(rig.step([("p", t)]), want) < F32_TOL


@gpu
@pytest.mark.parametrize("cuts", [[2] * 20, [1, 2, 3, 5, 8, 13, 7, 1], [7, 9, 8, 16], [39, 1], [3, 37], [8, 8, 8, 8, 8], [11, 1, 10, 11, 7]])
def test_portions_of_any_size(cuts):
    """Portions down to two tokens, at and beside the edges of pages (8) and windows (11, 5, 1)."""
    for name in ("a", "b"):
        rig = Rig(SHAPES[name](), seed=7)
        rig.poison()
        t = toks(sum(cuts), rig.cfg.vocab_size, 3)
        assert rel_err(rig.run("r", t, cuts), rig.oracle(t)) < F32_TOL, name


@gpu
def test_unequal_requests_in_one_batch_equal_each_alone():
    for name in ("a", "b", "c"):
        rig = Rig(SHAPES[name](), seed=11, pages=96)
        V = rig.cfg.vocab_size
        seqs = {"x": toks(41, V, 4), "y": toks(3, V, 5), "z": toks(18, V, 6), "w": toks(70, V, 7)}
        plan = [[("x", 17), ("y", 1), ("w", 33)], [("x", 1), ("y", 2), ("z", 18), ("w", 1)], [("x", 23), ("w", 36)]]
        at, got = {k: 0 for k in seqs}, {k: [] for k in seqs}
        for step in plan:
            out = rig.step([(k, seqs[k][at[k]:at[k] + n]) for k, n in step])
            r0 = 0
            for k, n in step:
                got[k].append(out[r0:r0 + n]); r0 += n; at[k] += n
        for k, s in seqs.items():
            assert at[k] == len(s) and rel_err(torch.cat(got[k]), rig.oracle(s)) < F32_TOL, (name, k)


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, 0.15)])
def test_freed_pages_and_slots_are_used_again(dtype, tol):
    """Two slots, a pool that holds two requests: requests end, their pages and slots go to new ones; old latents must not leak."""
    rig = Rig(shape_a(), seed=17, pages=12, slots=2, dtype=dtype)
    V = rig.cfg.vocab_size
    rig.poison()
    for rnd in range(4):
        a, b = toks(40 + rnd, V, 20 + rnd), toks(17 + 3 * rnd, V, 30 + rnd)
        ga = rig.step([("a", a[:25]), ("b", b[:1])])
        gb = rig.step([("a", a[25:]), ("b", b[1:])])
        for got, s in ((torch.cat([ga[:25], gb[:len(a) - 25]]), a), (torch.cat([ga[25:], gb[len(a) - 25:]]), b)):
            if dtype == torch.float32:
                assert rel_err(got, rig.oracle(s)) < tol, rnd
            else:
                assert rows_off(got, rig.oracle(s), tol) <= 0.1, rnd
        used = set(rig.req["a"]["pages"]) | set(rig.req["b"]["pages"])
        rig.end("b"); rig.end("a")
        assert len(rig.free_pages) == 12 and len(used) >= 8


# ---- keys that stand out ----------------------------------------------------------------------------------------------------------------
V_HOT, W_HOT = 40, 32


def hot_model(kind, size=19, owner_size=19, sink=0.0):
    """A sharp softmax without a feed-forward, and a rotation that hardly turns.  ``kind`` "own": one windowed layer; "borrowed": an owner whose
    output is switched off in front of a layer that attends over its latents with a window of its own; "causal".  Returns (cfg, tensors,
    query token, key token, tokens the query ignores)."""
    kw = dict(heads=2, dim=16, rot=4, vdim=16, rank=32, qrank=24, base=1e9, scale=3.0)
    layers = {"own": [win(size=size, **kw)], "borrowed": [win(size=owner_size, **kw), win(size=size, kv_from=0, **dict(kw, qrank=20, scale=6.0))],
              "causal": [cau(heads=2, dim=16, vdim=16, rank=32, qrank=24, scale=3.0)]}[kind]
    cfg = make_cfg([dict(L, mlp=None) for L in layers], width=W_HOT, vocab=V_HOT, emb=5.0, mult=1.0)
    t = tensors_for(cfg, 23)
    last = len(layers) - 1
    for i in range(len(layers)):
        if kind != "causal":                                  # the rotated part carries nothing: the window is the only thing that depends on places
            t[f"l{i}.mix.uq"] = t[f"l{i}.mix.uq"].clone()
            t[f"l{i}.mix.uq"].view(2, 20, -1)[:, 16:] = 0
            t[f"l{i}.mix.g"] = torch.zeros_like(t[f"l{i}.mix.g"])                                # gates of a half: none hides its head
    if kind == "borrowed":
        t["l0.norm1"] = torch.zeros(W_HOT)
    if kind == "causal":
        t["l0.mix.sink"] = torch.full((2,), float(sink))
    h = t["embed"].double() * 5.0
    P, P0 = layer_tensors(t, last), layer_tensors(t, 0)
    q = O.latent_queries(h, P, 2, 1e-5)[:, 0, :16]
    c = O.rms_norm((h @ P0["mix.dkv"].T)[:, :32], P0["mix.dkv.norm"], 1e-5)
    s = q @ (c @ P["mix.uk"].T).view(V_HOT, 2, 16)[:, 0].T
    qi, kj = divmod(int((s - s.diagonal().view(-1, 1)).argmax()), V_HOT)                         # the reader sees itself as well: the key stands out from that
    dull = [x for x in np.argsort(s[qi].numpy())[:12].tolist() if x not in (kj, qi)]
    return cfg, t, qi, kj, dull


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
@pytest.mark.parametrize("place", [16, 23, 24, 0, 127, 128])
def test_a_far_key_among_hundreds(dtype, tol, place):
    """Causal attention over many pages: the hot key sits up to 300 tokens back — at a page's first place, its last place, the next page's
    first, and position 0 — and is read by a prompt's portion and by a single decoded token."""
    cfg, t, qi, kj, dull = hot_model("causal")
    T = 300
    seq = [dull[i % len(dull)] for i in range(T)]
    seq[place], seq[T - 1], seq[T - 9] = kj, qi, qi
    rig = Rig(cfg, tensors=t, pages=64, dtype=dtype)
    got = rig.run("r", seq, [121, T - 123])
    want = rig.oracle(seq)
    assert rel_err(got[-1], want[-1]) < tol and rel_err(got[T - 9], want[T - 9]) < tol and rel_err(got, want) < tol
    seq2 = list(seq)
    seq2[place] = dull[0]
    other = rig.oracle(seq2)
    assert rel_err(other[-1], want[-1]) > 0.05 and rel_err(other[T - 9], want[T - 9]) > 0.05     # the test would see the key missing


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
@pytest.mark.parametrize("kind,size", [("own", 1), ("own", 2), ("own", 8), ("own", 19), ("own", 64), ("own", 130), ("borrowed", 7), ("borrowed", 33)])
def test_keys_just_inside_and_just_outside_a_window(kind, size, dtype, tol):
    """The hot key at the window's last place and one further back, read in a prompt's portion and by decoded tokens; the oracle with a window one
    longer or shorter gives other logits.  A borrowing layer's window is its own, not the owner's."""
    cfg, t, qi, kj, dull = hot_model(kind, size=size, owner_size=12)
    T = 2 * size + 60
    for back, inside in ((size - 1, True), (size, False)):
        if back == 0:
            continue
        for reader in (T - 20, T - 2):                       # in the second portion, and decoded
            seq = [dull[i % len(dull)] for i in range(T)]
            seq[reader], seq[reader - back] = qi, kj
            rig = Rig(cfg, tensors=t, pages=64, dtype=dtype)
            got = rig.run("r", seq, [31, T - 36])
            want = rig.oracle(seq)
            assert rel_err(got[reader], want[reader]) < tol and rel_err(got, want) < tol, (back, reader)
            wrong = copy.deepcopy(cfg)
            wrong["layers"][-1]["mixer"]["mask"]["size"] = size - 1 if inside else size + 1
            if wrong["layers"][-1]["mixer"]["mask"]["size"]:
                assert rel_err(O.forward(wrong, t, seq, torch.float64)[reader], want[reader]) > 3 * BF16_TOL, (back, reader)


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
def test_the_sink_counts_once_in_prompts_and_in_decoding(dtype, tol):
    """A sink as large as all keys together: left out, or counted once more, it changes the logits — at the first token, in portions, and in
    decoding over hundreds of keys (shared out over workgroups)."""
    cfg, t, qi, kj, dull = hot_model("causal")
    t["l0.mix.uq"] = t["l0.mix.uq"] * 0.05                   # flat scores: the denominator is about the number of keys
    for T, sink in ((3, 0.5), (40, 3.0), (400, 6.0)):
        t["l0.mix.sink"] = torch.tensor([sink, sink - 1.0])
        seq = toks(T, V_HOT, T)
        rig = Rig(cfg, tensors=t, pages=64, dtype=dtype)
        got, want = rig.run("r", seq, [T - 3] if T > 3 else []), rig.oracle(seq)
        assert rel_err(got, want) < tol and rel_err(got[-1], want[-1]) < tol and rel_err(got[0], want[0]) < tol
    # a sublayer output's size cancels in its norm: look at the mixer itself for the sink's weight
    P = layer_tensors(t, 0)
    h = torch.randn(400, W_HOT, generator=torch.Generator().manual_seed(1))
    rig = Rig(cfg, tensors=t, pages=64, dtype=dtype)
    hd = h.cuda().to(dtype)
    m = cfg["layers"][0]["mixer"]
    got = torch.cat([rig.model._mixer(0, hd[a:z].contiguous(), rig.batch([("r", [0] * (z - a))])[0], rig.cache).float().cpu() for a, z in ((0, 1), (1, 397), (397, 398), (398, 400))])
    want = O.causal_latent_attention(hd.cpu().double(), P, m, 1e-5)
    for i in (0, 200, 397, 399):
        assert rel_err(got[i], want[i]) < tol / 2, i
    for shift in (-30.0, float(np.log(2.0))):                  # no sink; the sink twice
        other = O.causal_latent_attention(hd.cpu().double(), dict(P, **{"mix.sink": P["mix.sink"] + shift}), m, 1e-5)
        assert min(rel_err(other[i], want[i]) for i in (0, 200, 397, 399)) > 3 * BF16_TOL


@gpu
def test_what_would_be_hidden_shows():
    """Planted in the oracle: each mechanism of the design changes the logits by far more than the tolerance the other tests use."""
    cfg, seq = shape_a(), toks(60, 131, 12)
    t = tensors_for(cfg, 3)
    want = O.forward(cfg, t, seq, torch.float64)
    base = Rig(cfg, tensors=t)
    assert rel_err(base.step([("r", seq)]), want) < F32_TOL

    def off(change=None, tens=None):
        c, tt = copy.deepcopy(cfg), dict(t)
        if change:
            change(c)
        tt.update(tens or {})
        return rel_err(O.forward(c, tt, seq, torch.float64), want)
    assert off(lambda c: c.update(residual_mult=0.5)) > 50 * F32_TOL and off(lambda c: c["embedding"].update(scale=2.0)) > 50 * F32_TOL
    assert off(lambda c: c["layers"][2]["mixer"]["mask"].update(size=11)) > 50 * F32_TOL and off(lambda c: c["layers"][3]["mixer"]["rot"].update(base=300.0)) > 50 * F32_TOL
    assert off(lambda c: c["layers"][2]["mixer"].update(scale=0.25)) > 50 * F32_TOL
    for name in ("l0.mlp.up.b", "l0.mlp.down.b", "l1.mlp.correction", "l1.mix.sink", "l0.mix.g", "l2.mix.g", "l1.mlp.shared.down", "l0.mix.dq.norm", "l3.mix.dkv.norm"):
        assert off(tens={name: torch.zeros_like(t[name]) if "norm" not in name else torch.ones_like(t[name])}) > 25 * F32_TOL, name


@gpu
def test_the_first_tokens_of_a_sequence():
    """One, two and three tokens in a slot and on pages that hold another request's latents."""
    for name in ("a", "b"):
        rig = Rig(SHAPES[name](), seed=19, slots=1, pages=16)
        V = rig.cfg.vocab_size
        rig.step([("old", toks(30, V, 1))])
        rig.end("old")
        for n in (1, 2, 3):
            t = toks(n + 1, V, 50 + n)
            assert rel_err(rig.run("new", t, [n]), rig.oracle(t)) < F32_TOL, (name, n)
            rig.end("new")


@gpu
@pytest.mark.parametrize("name", ["a", "b"])
def test_long_decoding(name):
    rig = Rig(SHAPES[name](), seed=29, pages=64)
    t = toks(220, rig.cfg.vocab_size, 8)
    want = rig.oracle(t)
    got = rig.run("r", t, [40])
    assert rel_err(got, want) < F32_TOL and rel_err(got[-1], want[-1:]) < F32_TOL


def random_cfg(r):
    layers, owners = [], []
    for i in range(r.choice([1, 2, 3, 4, 5])):
        size = lambda: r.choice([1, 2, 5, 8, 13, 20, 64])
        if r.random() < 0.3:
            L = cau(r.choice([1, 2, 4, 7, 18]), r.choice([8, 10, 24, 64]), r.choice([6, 16, 40]), r.choice([16, 20, 33, 64, 96, 160]), r.choice([9, 24, 64]), r.choice([0.1, 0.3]))
        elif owners and r.random() < 0.5:
            j = r.choice(owners)
            o = layers[j]["mixer"]
            L = win(r.choice([1, 3, 6]), r.choice([8, 12, 32]), o["rot_dim"], r.choice([6, 16, 24]), o["kv_rank"], r.choice([9, 32]), size(), o["rot"]["base"], r.choice([0.1, 0.3]), j)
        else:
            L = win(r.choice([1, 2, 5, 8, 17]), r.choice([8, 12, 32]), r.choice([2, 4, 8, 16, 32]), r.choice([6, 16, 40]), r.choice([16, 20, 33, 64, 96, 160]), r.choice([9, 24, 64]), size(),
                    r.choice([50.0, 1e4]), r.choice([0.1, 0.3]))
            owners.append(i)
        k, E, ident = r.random(), r.choice([1, 3, 8]), r.choice([0, 1, 4])
        L["mlp"] = None if k < 0.2 else dense(r.choice([24, 57, 100])) if k < 0.5 else moe(E, ident, r.randint(1, E + ident), r.choice([12, 16, 33]), r.choice([0, 10, 24]))
        layers.append(L)
    return make_cfg(layers, width=r.choice([32, 50, 64, 100]), vocab=r.choice([30, 77, 131]), eps=r.choice([1e-5, 1e-6]), emb=r.choice([1.0, 3.0, 8.0]), mult=r.choice([0.25, 0.5, 1.0]))


@gpu
@pytest.mark.parametrize("seed", range(14))
def test_random_configurations_in_a_mixed_schedule(seed):
    """Random layer orders, borrowings, head counts, sizes and constants; two requests of unequal length in a random schedule of portions and
    single tokens, float32 and bfloat16."""
    r = random.Random(3000 + seed)
    cfg = random_cfg(r)
    t = tensors_for(cfg, seed)
    V = cfg["vocab"]
    seqs = {"x": toks(r.choice([9, 31, 60]), V, seed), "y": toks(r.choice([2, 17, 45]), V, seed + 100)}
    plan, at = [], {k: 0 for k in seqs}
    while any(at[k] < len(s) for k, s in seqs.items()):
        step = []
        for k, s in seqs.items():
            if at[k] < len(s) and r.random() < 0.8:
                n = min(len(s) - at[k], r.choice([1, 1, 2, 3, 7, 8, 9, 20, 40]))
                step.append((k, at[k], n)); at[k] += n
        if step:
            plan.append(step)
    want = {k: O.forward(cfg, t, s, torch.float64) for k, s in seqs.items()}
    for dtype in (torch.float32, torch.bfloat16):
        rig = Rig(cfg, tensors=t, dtype=dtype, pages=32, seed=seed)
        rig.poison()
        got = {k: [] for k in seqs}
        for step in plan:
            out = rig.step([(k, seqs[k][a:a + n]) for k, a, n in step])
            r0 = 0
            for k, a, n in step:
                got[k].append(out[r0:r0 + n]); r0 += n
        for k in seqs:
            if dtype == torch.float32:
                assert rel_err(torch.cat(got[k]), want[k]) < F32_TOL, (cfg, k)
            else:
                assert rows_off(torch.cat(got[k]), want[k], 0.15) <= 0.25, (cfg, k)


# ---- the engine -------------------------------------------------------------------------------------------------------------------------
def _write_model(tmp_path, cfg_dict, tensors):
    from safetensors.torch import save_file
    (tmp_path / "config.json").write_text(json.dumps(cfg_dict))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()}, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


def _oracle_greedy(cfg_dict, tensors, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(O.forward(cfg_dict, tensors, seq, torch.float64)[-1].argmax()))
    return seq[len(prompt):]


@gpu
def test_greedy_generation_through_the_engine_and_its_scheduler(tmp_path):
    """LLM.generate on a checkpoint directory: registry -> loader -> scheduler (prompts cut to the token budget, admissions limited by two
    slots, pages reused) -> ragged step -> argmax.  float32 so that the greedy choice is the oracle's."""
    from jacobiforcing_amd import LLM, SamplingParams
    cfg_dict = shape_a()
    tensors = tensors_for(cfg_dict, 31)
    path = _write_model(tmp_path, cfg_dict, tensors)
    V = cfg_dict["vocab"]
    prompts = [toks(n, V, 40 + n) for n in (70, 5, 33, 1)]
    llm = LLM(path, tokenizer_path="none", dtype="float32", kvcache_block_size=64, num_kvcache_blocks=4, max_num_seqs=2, max_model_len=128,
              max_num_batched_tokens=128, device="cuda")
    out = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True), use_tqdm=False)
    for p, o in zip(prompts, out):
        assert o["token_ids"] == _oracle_greedy(cfg_dict, tensors, p, 6)
    assert len(llm.scheduler.block_manager.free_block_ids) == 4 and len(llm.model_runner.free_rows) == 2
    # the same engine replays a given schedule: portions beside single tokens, requests that end, logits where asked
    a, b = prompts[0], prompts[2]
    l1 = llm.replay_step([("a", a[:40], [0, 39]), ("b", b[:2], [])])
    l2 = llm.replay_step([("a", a[40:], [29]), ("b", b[2:], [len(b) - 3])], end=["a"])
    l3 = llm.replay_step([("c", a, [len(a) - 1])], end=["b", "c"])
    wa, wb = O.forward(cfg_dict, tensors, a, torch.float64), O.forward(cfg_dict, tensors, b, torch.float64)
    assert tuple(l1.shape) == (2, V) and rel_err(l1.cpu(), wa[[0, 39]]) < F32_TOL
    assert rel_err(l2.cpu(), torch.stack([wa[69], wb[len(b) - 1]])) < F32_TOL and rel_err(l3.cpu(), wa[-1:]) < F32_TOL
    assert len(llm.scheduler.block_manager.free_block_ids) == 4 and len(llm.model_runner.free_rows) == 2


@gpu
def test_a_preempted_request_starts_again(tmp_path):
    """Three pages for two requests that need five: the newer one is preempted while it decodes, gives its pages back and is prefilled again."""
    from jacobiforcing_amd import LLM, SamplingParams
    cfg_dict = shape_a()
    tensors = tensors_for(cfg_dict, 43)
    path = _write_model(tmp_path, cfg_dict, tensors)
    prompts = [toks(100, 131, 61), toks(60, 131, 62)]
    llm = LLM(path, tokenizer_path="none", dtype="float32", kvcache_block_size=64, num_kvcache_blocks=3, max_num_seqs=2, max_model_len=192,
              max_num_batched_tokens=192, device="cuda")
    preempted = []
    keep = llm.scheduler.preempt
    llm.scheduler.preempt = lambda seq: (preempted.append(seq.seq_id), keep(seq))[1]
    out = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=30, ignore_eos=True), use_tqdm=False)
    assert preempted, "the pool was meant to run out"
    for p, o in zip(prompts, out):
        assert o["token_ids"] == _oracle_greedy(cfg_dict, tensors, p, 30)


@gpu
def test_sampling_through_the_engine_follows_the_distribution(tmp_path):
    from jacobiforcing_amd import LLM, SamplingParams
    cfg_dict = shape_b()
    tensors = tensors_for(cfg_dict, 37)
    path = _write_model(tmp_path, cfg_dict, tensors)
    prompt = toks(9, cfg_dict["vocab"], 50)
    llm = LLM(path, tokenizer_path="none", dtype="float32", kvcache_block_size=64, num_kvcache_blocks=16, max_num_seqs=16, max_model_len=64,
              max_num_batched_tokens=64, device="cuda")
    torch.manual_seed(0)
    out = llm.generate([prompt] * 800, SamplingParams(temperature=1.0, max_tokens=1, ignore_eos=True), use_tqdm=False)
    p = torch.softmax(O.forward(cfg_dict, tensors, prompt, torch.float64)[-1], 0).numpy()
    counts = np.bincount([o["token_ids"][0] for o in out], minlength=len(p)) / 800.0
    assert 0.5 * np.abs(counts - p).sum() < 0.2                                                 # total variation of 800 draws over 77 ids


@gpu
def test_the_command_lines_serve_the_design(tmp_path, monkeypatch, capsys):
    """bin/trace_run on a schedule with two live requests and pages used again, and the generation driver, on a checkpoint directory."""
    cfg_dict = shape_c()
    tensors = tensors_for(cfg_dict, 51)
    (tmp_path / "m").mkdir()
    path = _write_model(tmp_path / "m", cfg_dict, tensors)
    a, b = toks(90, 50, 1), toks(20, 50, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [0, 69]}, {"id": "b", "tokens": b[:1], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[1:], "want": [18]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[70:], "want": [19]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": a, "want": [89]}], "end": ["c"]}]
    loader = importlib.machinery.SourceFileLoader("trace_run_script", str(Path(__file__).resolve().parents[1] / "bin" / "trace_run"))
    script = importlib.util.module_from_spec(importlib.util.spec_from_loader("trace_run_script", loader))
    loader.exec_module(script)
    monkeypatch.setattr("sys.argv", ["trace_run", "--model", path, "--dtype", "float32", "--out", str(tmp_path / "o"), "--max-tokens", "192"])
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    assert script.main() == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == [f"done {k}" for k in range(4)]
    wa, wb = O.forward(cfg_dict, tensors, a, torch.float64), O.forward(cfg_dict, tensors, b, torch.float64)
    for k, want in enumerate((wa[[0, 69]], wb[-1:], wa[-1:], wa[-1:])):
        got = np.fromfile(str(tmp_path / "o" / f"{k}.f32"), "<f4").reshape(-1, 50)
        assert got.shape == tuple(want.shape) and rel_err(got, want) < F32_TOL
    from jacobiforcing_amd.drivers import generate
    (tmp_path / "p.json").write_text(json.dumps([a[:30], b]))
    assert generate.main(["--model", path, "--prompts", str(tmp_path / "p.json"), "--max-tokens", "4", "--dtype", "float32", "--max-model-len", "128", "--max-num-seqs", "2"]) == 0
    lines = [json.loads(x) for x in capsys.readouterr().out.splitlines() if x.startswith("{")]
    assert [x["token_ids"] for x in lines if "token_ids" in x] == [_oracle_greedy(cfg_dict, tensors, p, 4) for p in (a[:30], b)]
