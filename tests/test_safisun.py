"""Safisun through the package (HIP layer kernels, paged pools beside state slots, ragged step, scheduler, LLM.generate) against the plain
oracle ``oracle/safisun_oracle.py``, which shares no code with it.  Small random models of several shapes; where random weights would hide a
fault (a far key among hundreds, a key at a page's or a chunk's border, an old write in a recurrent state, the one in the softmax's
denominator) the weights and inputs are chosen so that it shows.

CPU tests cover the oracle's own pieces, the config reader, the weights and the cache layout; everything that launches a kernel is marked
``gpu``."""
import json
import random

import numpy as np
import pytest
import torch

from oracle import safisun_oracle as O
from jacobiforcing_amd.modeling import MODEL_REGISTRY, read_model_config
from jacobiforcing_amd.modeling import safisun as SF

gpu = pytest.mark.gpu


# ---- model shapes -----------------------------------------------------------------------------------------------------------------
def decays(n):
    return [round(0.3 + 0.69 * (i + 1) / n, 4) for i in range(n)]


def lightning(heads=3, dim=16, vdim=24, decay=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay or decays(heads)}}


def mamba(heads=6, groups=2, state=20, vdim=12, conv=3, parts=3):
    return {"type": "mamba2", "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": parts}}


def parallel(heads=6, kv=2, dim=24, vdim=20, dims=16, base=500.0, scale=0.3, cap=6.0, chunk=11, right=None, ls=0.7, rs=1.3):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "mask": {"size": chunk}}
    if dims:
        left["rot"] = {"dims": dims, "base": base}
    return {"type": "parallel", "mixer": {"left": left, "left_scale": ls, "right": (right or lightning(2, 20, 28))["mixer"], "right_scale": rs}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def make_cfg(layers, width=96, vocab=131, eps=1e-5, loop=(0, 1, 1)):
    d = {"architecture": "Safisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": [dict({"mlp": None}, **L) for L in layers]}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


def shape_a():
    """All three mixers, a loop that starts and ends inside the stack and runs three times, layers with and without a feed-forward."""
    return make_cfg([dict(lightning(), mlp=dense(40)), mamba(), dict(parallel(), mlp=dense()), dict(mamba(4, 1, 16, 16, 4, 1), mlp=dense(24)), lightning(5, 8, 12)],
                    loop=(1, 3, 3))


def shape_b():
    """One head, one key head, no rotation in one layer, one tap, sizes that are no multiples of four, a loop over the last layers, another eps."""
    return make_cfg([dict(parallel(1, 1, 10, 7, 0, chunk=5, right=lightning(1, 9, 5, [0.9]), ls=1.0, rs=0.25), mlp=dense(30)), mamba(3, 3, 7, 5, 1, 1),
                     dict(parallel(5, 1, 14, 9, 6, 50.0, 0.5, 2.0, 33, lightning(3, 6, 11), 0.4, 0.9), mlp=None), mamba(2, 1, 33, 9, 5, 2)],
                    width=62, vocab=77, eps=1e-4, loop=(2, 4, 2))


def shape_c():
    """Head sizes the matrix-core kernels take in bfloat16 (attention and the recurrence in pieces); a loop over everything."""
    return make_cfg([dict(parallel(8, 2, 64, 64, 24, 1e5, 0.15, 30.0, 40, lightning(3, 32, 64)), mlp=dense(64)), mamba(8, 2, 64, 32, 4, 4), lightning(2, 128, 128)],
                    width=128, vocab=50, loop=(0, 3, 2))


def shape_d():
    """No loop at all."""
    return make_cfg([mamba(2, 2, 8, 40, 2, 1), dict(lightning(2, 40, 16), mlp=dense(20))], width=40, vocab=33, loop=None)


SHAPES = {"a": shape_a, "b": shape_b, "c": shape_c, "d": shape_d}


def tensors_for(cfg_dict, seed):
    return SF.random_tensors(SF.SafisunConfig.from_dict(cfg_dict), seed)


def mixer_tensors(t, i, dtype=torch.float64):
    p = f"l{i}.mix."
    return {k[len(p):]: v.to(dtype) for k, v in t.items() if k.startswith(p)}


def rel_err(got, want):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    return float(np.sqrt(((got - want) ** 2).mean()) / max(np.sqrt((want ** 2).mean()), 1e-30))


F32_TOL, BF16_TOL = 2e-4, 6e-2


def close(got, want, dtype) -> bool:
    """float32: within F32_TOL.  bfloat16: half the positions within BF16_TOL and at most one in eight (or one) beyond 0.15 — a norm on a
    sublayer's output divides by its size, so a position whose sublayer nearly cancels carries that rounding on, and later layers and
    passes enlarge it (rounding nothing but the mixers' inputs and outputs in the oracle moves such positions as far)."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    if dtype == torch.float32:
        return rel_err(got, want) < F32_TOL
    err = np.sqrt(((got - want) ** 2).mean(-1)) / np.maximum(np.sqrt((want ** 2).mean(-1)), 1e-30)
    return float(np.median(err)) < BF16_TOL and int((err > 0.15).sum()) <= max(1, len(err) // 8)


def toks(n, vocab, seed):
    return [random.Random(seed * 7919 + i).randrange(vocab) for i in range(n)]


# =====================================================================================================================================
# CPU: oracle pieces, config reader, weights, cache layout
# =====================================================================================================================================
def test_registry_reads_the_architecture_key(tmp_path):
    assert MODEL_REGISTRY["Safisun"][2] == "ragged"
    (tmp_path / "config.json").write_text(json.dumps(shape_a()))
    cfg = read_model_config(tmp_path)
    assert isinstance(cfg, SF.SafisunConfig) and cfg.family == "ragged" and cfg.num_hidden_layers == 5 and cfg.norm_eps == 1e-5
    assert cfg.runs() == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None), (4, None)]
    assert SF.SafisunConfig.from_dict(shape_c()).runs() == [(0, 0), (1, None), (2, None), (0, 1), (1, None), (2, None)]
    assert SF.SafisunConfig.from_dict(shape_d()).runs() == [(0, None), (1, None)]
    one = make_cfg([lightning(), lightning()], loop=(1, 2, 1))
    assert SF.SafisunConfig.from_dict(one).runs() == [(0, None), (1, 0)]                        # a single pass has its product in front of it too
    for c in (shape_a(), shape_b(), shape_c(), shape_d(), one):
        assert SF.SafisunConfig.from_dict(c).runs() == O.execution(c)


def test_config_rejects_what_the_design_does_not_have():
    for change in (lambda c: c["layers"][0].update(type="retention"), lambda c: c["layers"][0]["mlp"].update(kind="moe"),
                   lambda c: c["layers"][0]["mixer"].update(decay=[0.5]), lambda c: c["layers"][0]["mixer"].update(dim=300),
                   lambda c: c["layers"][1]["mixer"].update(groups=4), lambda c: c["layers"][1]["mixer"].update(norm_groups=7),
                   lambda c: c["layers"][1]["mixer"].update(conv=9), lambda c: c["layers"][2]["mixer"]["left"].update(kv_heads=4),
                   lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(dims=26), lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(dims=7),
                   lambda c: c["layers"][2]["mixer"]["right"].update(heads=3), lambda c: c["loop"].update(stop=6), lambda c: c["loop"].update(times=0),
                   lambda c: c["loop"].update(start=3)):
        bad = shape_a()
        change(bad)
        with pytest.raises(ValueError):
            SF.SafisunConfig.from_dict(bad)


def test_cache_layout_and_stacked_weights():
    cfg = SF.SafisunConfig.from_dict(shape_a())
    t = tensors_for(shape_a(), 1)
    w = SF.SafisunWeights(cfg, t, "cpu", torch.float32)
    specs = SF.SafisunModel(cfg, w, max_positions=16).cache_specs()
    assert [s.kind for s in specs] == ["state", "state", "kv+state", "state", "kv+state", "state", "kv+state", "state", "state"]      # every pass its own
    assert specs[0].state_shape == (3, 16, 24) and specs[1].state_shape == (6, 20, 12) and specs[1].tails == {"conv": (2, 72 + 80)}
    assert (specs[2].k_width, specs[2].v_width, specs[2].state_shape) == (48, 40, (2, 20, 28))
    l0, l1, l2 = w.layers[:3]
    assert tuple(l0["w_in"].shape) == (2 * 48 + 2 * 72, 96) and l0["cols"] == (0, 48, 96, 168)
    assert tuple(l1["w_in"].shape) == (72 + 152 + 6 + 2, 96) and float(l1["w_in"][-2:].abs().max()) == 0 and torch.equal(l1["w_in"][:230], t["l1.mix.in"])
    rows = 144 + 48 + 40
    assert l2["cols"] == (rows, rows + 40, rows + 80, rows + 136) and l2["a_cols"] == (0, 144, 192, rows + 192)
    assert torch.equal(l2["w_in"][l2["a_cols"][3]:l2["a_cols"][3] + 6], t["l2.mix.left.g"]) and torch.equal(l2["b_in"][144:192], t["l2.mix.left.k.b"])
    assert float(l2["b_in"][rows:].abs().max()) == 0 and torch.equal(l2["w_o"], torch.cat([t["l2.mix.left.o"], t["l2.mix.right.o"]], 1))
    bad = dict(t)
    bad["l1.mix.conv.b"] = bad["l1.mix.conv.b"][:-1]
    with pytest.raises(ValueError):
        SF.SafisunWeights(cfg, bad, "cpu", torch.float32)
    from jacobiforcing_amd.engine.state_cache import PagedStateCache, RunSpec
    cache = PagedStateCache(specs, 4, 8, 3, "cpu", torch.float32)
    assert tuple(cache.k[2].shape) == (32, 48) and tuple(cache.state[2].shape) == (3, 2, 20, 28) and cache.k[0] is None and cache.state[1] is not None
    assert tuple(cache.tails[1]["conv"].shape) == (3, 2, 152) and cache.bytes() > 0
    with pytest.raises(ValueError):
        PagedStateCache([RunSpec("pages")], 4, 8, 3, "cpu", torch.float32)


def test_oracle_pieces():
    g = torch.Generator().manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    z = torch.tensor([-3.0, 0.0, 0.5, 2.0], dtype=torch.float64)
    assert torch.allclose(O.silu(z), torch.nn.functional.silu(z)) and torch.allclose(O.softplus(z), torch.nn.functional.softplus(z))
    assert float(O.softplus(torch.tensor(50.0, dtype=torch.float64))) == 50.0
    assert torch.allclose(O.soft_cap(z * 100, 3.0), 3 * torch.tanh(z * 100 / 3)) and torch.allclose(O.soft_cap(z * 1e-4, 3.0), z * 1e-4)
    # one more in the denominator: the weights sum to less than one, and equal scores of zero share with it
    vis = O.chunk_mask(7, 3)
    assert vis[5].tolist() == [False, False, False, True, True, True, False] and vis[6].tolist() == [False] * 6 + [True]
    w = O.softmax_one_more(torch.zeros(2, 7, 7, dtype=torch.float64), vis)
    assert torch.allclose(w[0, 5], vis[5].double() / 4) and torch.allclose(w.sum(-1)[0, 6], torch.tensor(0.5, dtype=torch.float64))
    s = rn(1, 7, 7) * 3
    assert torch.allclose(O.softmax_one_more(s, vis), (torch.exp(s) * vis) / (1 + (torch.exp(s) * vis).sum(-1, keepdim=True)))
    # the rotation keeps lengths, leaves the rest alone, does nothing at position 0
    x, a = rn(4, 3, 10), O.angles(4, 6, 50.0)
    r = O.rotate_neighbours(x, a)
    assert torch.allclose((r * r).sum(-1), (x * x).sum(-1)) and torch.equal(r[..., 6:], x[..., 6:]) and torch.allclose(r[0], x[0])
    assert abs(float(r[2, 1, 3]) - float(x[2, 1, 3] * a[2, 1].cos() + x[2, 1, 2] * a[2, 1].sin())) < 1e-12
    # the convolution's last column is the current token's
    xs, cw, cb = rn(6, 3), rn(3, 4), rn(3)
    y = O.short_conv(xs, cw, cb)
    assert torch.allclose(y[0], cb + xs[0] * cw[:, 3]) and torch.allclose(y[4], cb + xs[4] * cw[:, 3] + xs[3] * cw[:, 2] + xs[2] * cw[:, 1] + xs[1] * cw[:, 0])
    # the recurrence unrolled: o_i = sum_j (q_i . k_j) (product of the decays behind j) v_j
    q, k, v, d = rn(5, 4), rn(5, 4), rn(5, 3), torch.rand(5, generator=g, dtype=torch.float64)
    want = sum((q[4] @ k[j]) * d[j + 1:5].prod() * v[j] for j in range(5))
    assert torch.allclose(O.decayed_sum(q, k, v, d)[4], want)


# =====================================================================================================================================
# GPU: the package against the oracle
# =====================================================================================================================================
class Rig:
    """A model on the GPU with a pool of shuffled pages; runs steps of (request, tokens) and keeps the bookkeeping a test needs."""

    def __init__(self, cfg_dict, seed=0, dtype=torch.float32, page=8, pages=64, slots=4, tensors=None, max_positions=1024):
        from jacobiforcing_amd import layer_ops as LO
        self.LO = LO
        self.cfg_dict = cfg_dict
        self.cfg = SF.SafisunConfig.from_dict(cfg_dict)
        self.tensors = tensors or tensors_for(cfg_dict, seed)
        self.model = SF.SafisunModel(self.cfg, SF.SafisunWeights(self.cfg, self.tensors, "cuda", dtype), max_positions=max_positions)
        self.page = page
        self.cache = self.model.new_cache(pages, page, slots)
        self.free_pages = list(range(pages))
        random.Random(seed).shuffle(self.free_pages)
        self.free_slots = list(range(slots))[::-1]
        self.req = {}

    def poison(self):
        """Fill pools, states and tails with large values: whatever a kernel reads without having written it shows."""
        for t in self.cache.k + self.cache.v + self.cache.state + [x for d in self.cache.tails for x in d.values()]:
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

    def portions(self, key, tokens, cuts):
        got, at = [], 0
        for n in cuts:
            got.append(self.step([(key, tokens[at:at + n])]))
            at += n
        assert at == len(tokens)
        return torch.cat(got)

    def end(self, key):
        r = self.req.pop(key)
        self.free_pages += r["pages"][::-1]
        self.free_slots.append(r["slot"])

    def oracle(self, tokens, trace=None):
        return O.forward(self.cfg_dict, self.tensors, list(tokens), torch.float64, trace)


# ---- each new launch alone ----------------------------------------------------------------------------------------------------------------
@gpu
@pytest.mark.parametrize("W", [50, 96, 324, 1000, 2052, 4096, 5000, 8200])
def test_norms_around_a_residual_update(W):
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(W)
    rn = lambda *s: torch.randn(*s, generator=g)
    n = 5
    x, y, wp, wn, row = rn(n, W), rn(n, W) * 3, rn(W), rn(W), rn(W)
    for ydt in (torch.float32, torch.bfloat16):
        yd = y.to(ydt)
        upd = x.double() + O.rms_norm(yd.double(), wp.double(), 1e-5)
        for odt, tol in ((torch.float32, 1e-6), (torch.bfloat16, 6e-3)):
            xi = x.cuda()
            out = LO.sandwich_norm(xi, yd.cuda(), wp.cuda(), 1e-5, wn.cuda(), odt)
            assert rel_err(xi.cpu(), upd) < 1e-6 and out.dtype == odt and rel_err(out.float().cpu(), O.rms_norm(upd, wn.double(), 1e-5)) < tol
            xi = x.cuda()
            out = LO.sandwich_norm(xi, yd.cuda(), wp.cuda(), 1e-5, wn.cuda(), odt, add_row=row.cuda())
            assert rel_err(xi.cpu(), upd + row) < 1e-6 and rel_err(out.float().cpu(), O.rms_norm(upd + row, wn.double(), 1e-5)) < tol
    # the stream itself into a column range of wider rows; the update alone; a row alone; the norm alone (nothing stored)
    wide = torch.full((n, 2 * W), 7.0, device="cuda")
    xi = x.cuda()
    LO.sandwich_norm(xi, y.cuda(), wp.cuda(), 1e-5, out=wide[:, :W], plain=True)
    assert torch.equal(wide[:, :W], xi) and float(wide[:, W:].min()) == 7.0 == float(wide[:, W:].max())
    xi = x.cuda()
    assert LO.sandwich_norm(xi, y.cuda(), wp.cuda(), 1e-5) is None and rel_err(xi.cpu(), x.double() + O.rms_norm(y.double(), wp.double(), 1e-5)) < 1e-6
    xi = x.cuda()
    out = LO.sandwich_norm(xi, None, None, 1e-5, wn.cuda(), torch.float32, add_row=row.cuda())
    assert rel_err(xi.cpu(), x + row) < 1e-6 and rel_err(out.cpu(), O.rms_norm((x + row).double(), wn.double(), 1e-5)) < 1e-6
    tiny = torch.full((1, W), 1e-4).cuda()                                                      # eps inside the root, both norms
    keep = tiny.clone()
    assert rel_err(LO.sandwich_norm(tiny, None, None, 1e-5, wn.cuda(), torch.float32).cpu(), O.rms_norm(keep.cpu().double(), wn.double(), 1e-5)) < 1e-6 and torch.equal(tiny, keep)
    z = torch.zeros(1, W).cuda()
    LO.sandwich_norm(z, keep, wp.cuda(), 1e-5)
    assert rel_err(z.cpu(), O.rms_norm(keep.cpu().double(), wp.double(), 1e-5)) < 1e-6
    with pytest.raises(ValueError):
        LO.sandwich_norm(x.cuda(), None, None, 1e-5, None, torch.float32)


@gpu
@pytest.mark.parametrize("C_,parts", [(24, 1), (24, 3), (35, 5), (48, 2), (1024, 1), (2304, 3), (4100, 1), (6000, 1), (8400, 1)])
def test_norm_with_its_gate(C_, parts):
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(C_)
    rn = lambda *s: torch.randn(*s, generator=g)
    n = 4
    raw, wide, w = rn(n, C_) * 2, rn(n, C_ + 12) * 2, rn(C_)
    norm = lambda v: O.rms_norm(v.view(n, parts, C_ // parts), None, 1e-5).reshape(n, C_)
    for dt, tol in ((torch.float32, 1e-6), (torch.bfloat16, 6e-3)):
        gate = wide.to(dt).cuda()[:, 8:8 + C_]
        gd = gate.cpu().double()
        first = LO.gated_norm(raw.cuda(), gate, w.cuda(), 1e-5, LO.ACT_SILU, True, parts=parts)
        assert first.dtype == dt and rel_err(first.float().cpu(), norm(raw.double() * O.silu(gd)) * w.double()) < tol
        buf = torch.full((n, C_ + 16), 3.0, dtype=dt, device="cuda")
        LO.gated_norm(raw.cuda(), gate, w.cuda(), 1e-5, LO.ACT_SIGMOID, False, parts=parts, scale=0.37, out=buf[:, 8:8 + C_])
        assert rel_err(buf[:, 8:8 + C_].float().cpu(), 0.37 * norm(raw.double()) * w.double() * torch.sigmoid(gd)) < tol
        assert float(buf[:, :8].float().sum()) == 24.0 * n and float(buf[:, 8 + C_:].float().sum()) == 24.0 * n
    with pytest.raises(ValueError):
        LO.gated_norm(raw.cuda(), wide.cuda()[:, :C_], w.cuda(), 1e-5, LO.ACT_SILU, True, parts=C_ - 1)


@gpu
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("C_,col,ld", [(70, 3, 80), (72, 4, 84)])
def test_short_convolution_with_a_bias_across_portions(taps, C_, col, ld):
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(taps)
    xa, xb = torch.randn(23, ld, generator=g), torch.randn(12, ld, generator=g)
    w, bias = torch.randn(C_, taps, generator=g), torch.randn(C_, generator=g)
    for dt, odt, tol in ((torch.float32, torch.float32, 1e-6), (torch.bfloat16, torch.float32, 1e-6), (torch.bfloat16, torch.bfloat16, 6e-3)):
        xs, wd, bd = [x.cuda().to(dt) for x in (xa, xb)], w.cuda().to(dt), bias.cuda().to(dt)
        want = [O.silu(O.short_conv(x.cpu().double()[:, col:col + C_], wd.cpu().double(), bd.cpu().double())) for x in xs]
        tail = torch.full((3, taps - 1, C_), 1e4, device="cuda") if taps > 1 else None
        got = [[], []]
        for a0, a1, b0, b1 in [(0, 9, 0, 1), (9, 10, 1, 3), (10, 19, 3, 4), (19, 23, 4, 12)]:    # portions beside single rows, shorter and longer than the taps
            b = LO.RaggedBatch.build([a1 - a0, b1 - b0], [a0, b0], [2, 0], [[0, 1, 2], [3, 4]], 8, "cuda")
            y = LO.short_conv(torch.cat([xs[0][a0:a1], xs[1][b0:b1]]), col, C_, wd, b, tail, LO.ACT_SILU, bias=bd, out_dtype=odt)
            assert y.dtype == odt
            got[0].append(y[:a1 - a0].float().cpu()); got[1].append(y[a1 - a0:].float().cpu())
        assert rel_err(torch.cat(got[0]), want[0]) < tol and rel_err(torch.cat(got[1]), want[1]) < tol, (dt, odt)


@gpu
@pytest.mark.parametrize("H,G,D,Dv,dims,pairing", [(6, 2, 24, 20, 16, 1), (3, 1, 10, 7, 6, 1), (3, 1, 10, 7, 6, 0), (5, 5, 8, 8, 0, 1), (10, 1, 64, 64, 24, 1), (16, 4, 128, 128, 128, 1),
                                                   (40, 40, 64, 32, 4, 1), (4, 2, 12, 12, 10, 1), (70, 2, 128, 64, 8, 1)])
def test_norm_over_the_whole_projection_with_rotation(H, G, D, Dv, dims, pairing):
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(H)
    rn = lambda *s: torch.randn(*s, generator=g)
    T, ld = 21, H * D + G * D + G * Dv + (-(H * D + G * D + G * Dv)) % 8
    proj, wq, wk = rn(T, ld) * 2, rn(H * D), rn(G * D)
    cols = (0, H * D, H * D + G * D)
    a = O.angles(64, dims, 90.0) if dims else None
    cos, sin = (a.cos().float().cuda().contiguous(), a.sin().float().cuda().contiguous()) if dims else (None, None)
    b = LO.RaggedBatch.build([T], [30], [0], [[5, 1, 0, 2, 6, 3, 4]], 8, "cuda")
    for dt, tol in ((torch.float32, 2e-6), (torch.bfloat16, 6e-3)):
        p, kq, kk = proj.cuda().to(dt), wq.cuda().to(dt), wk.cuda().to(dt)
        kc, vc = torch.full((64, G * D), 9.0, dtype=dt, device="cuda"), torch.full((64, G * Dv), 9.0, dtype=dt, device="cuda")
        q = LO.qk_norm_append(p, cols, H, G, D, Dv, kq, kk, 1e-5, kc, vc, b.kv_slot, rot_dims=dims, pairing=pairing, batch=b, cos=cos, sin=sin)
        pd = p.cpu().double()
        wantq = O.rms_norm(pd[:, :H * D], kq.cpu().double(), 1e-5).view(T, H, D)
        wantk = O.rms_norm(pd[:, H * D:H * D + G * D], kk.cpu().double(), 1e-5).view(T, G, D)
        if dims:
            def turn(x):
                if pairing == LO.ROT_NEIGHBOURS:
                    return O.rotate_neighbours(x, a[30:30 + T])
                half = dims // 2                                                                 # halves: the same turn on reordered dimensions
                order = [i // 2 + (i % 2) * half for i in range(dims)]
                y = x.clone()
                y[..., order] = O.rotate_neighbours(x[..., order], a[30:30 + T])
                return y
            wantq, wantk = turn(wantq), turn(wantk)
        at = b.kv_slot.cpu()
        assert rel_err(q.float().cpu(), wantq.reshape(T, -1)) < tol and rel_err(kc.float().cpu()[at], wantk.reshape(T, -1)) < tol, dt
        assert torch.equal(vc[b.kv_slot], p[:, cols[2]:cols[2] + G * Dv]) and int((kc == 9.0).all(1).sum()) == 64 - T


SCAN_SIZES = [(3, 3, 16, 24), (6, 2, 20, 12), (4, 1, 33, 9), (2, 2, 128, 128), (8, 2, 64, 32), (2, 1, 100, 68), (5, 5, 8, 130), (1, 1, 200, 40), (2, 2, 32, 4)]


def scan_reference(q, k, v, H, G, decay, dt, a_log, dt_bias, skip):
    T = q.shape[0]
    out = []
    for h in range(H):
        c = h // (H // G)
        if decay is not None:
            u, a = torch.ones(T, dtype=torch.float64), torch.full((T,), float(decay[h]), dtype=torch.float64)
        else:
            u = O.softplus(dt[:, h] + dt_bias[h])
            a = torch.exp(-torch.exp(a_log[h]) * u)
        o = O.decayed_sum(q[:, c], k[:, c], u.view(-1, 1) * v[:, h], a)
        out.append(o + (skip[h] * v[:, h] if skip is not None else 0))
    return torch.stack(out, 1).reshape(T, -1)


@gpu
@pytest.mark.parametrize("H,G,D,Dv", SCAN_SIZES)
@pytest.mark.parametrize("fixed", [True, False])
def test_linear_recurrence_alone(H, G, D, Dv, fixed):
    """Both forms (token by token; pieces on the matrix cores) through portions, single tokens and a long portion, on a poisoned slot, beside
    another request; the final states too."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(H * 1000 + D)
    rn = lambda *s: torch.randn(*s, generator=g)
    cuts = [19, 1, 40, 2, 1, 200, 33, 64, 3]
    T, To = sum(cuts), 90
    w = 2 * G * D + H * Dv
    ld = w + (-w) % 4
    src, dts = rn(T + To, ld), rn(T + To, H + 2) * 2
    decay = torch.tensor(decays(H)) if fixed else None
    a_log, dt_bias, skip = (None, None, None) if fixed else (rn(H), rn(H), rn(H))
    vcol = 0                                                                                    # v | k | q
    cols = (H * Dv + G * D, H * Dv, vcol)
    for dt_, tol in ((torch.float32, 3e-6), (torch.bfloat16, 4e-5 if not fixed else 4e-3)):
        s = src.cuda().to(dt_)
        dd = dts.cuda().to(dt_)[:, 1:1 + H]
        sd, ddd = s.cpu().double(), dd.cpu().double()
        act = O.silu if fixed else (lambda z: z)
        def ref(sl):
            x = act(sd[sl])
            return scan_reference(x[:, cols[0]:cols[0] + G * D].view(-1, G, D), x[:, cols[1]:cols[1] + G * D].view(-1, G, D), x[:, :H * Dv].view(-1, H, Dv), H, G,
                                  decay.double() if fixed else None, ddd[sl], None if fixed else a_log.double(), None if fixed else dt_bias.double(),
                                  None if fixed else skip.double())
        want, other = ref(slice(0, T)), ref(slice(T, T + To))
        state = torch.full((3, H, D, Dv), 1e4, device="cuda")
        kw = dict(act=LO.ACT_SILU, decay=decay.cuda()) if fixed else dict(a_log=a_log.cuda(), dt_bias=dt_bias.cuda(), skip=skip.cuda())
        run = lambda rows, b: LO.linear_scan(s[rows].contiguous(), cols, b, H, G, D, Dv, state, **kw, **({} if fixed else {"dt": dd[rows]})).cpu()
        got, got_o, at, ato = [], [], 0, 0
        for i, n in enumerate(cuts):
            no = (1, 36, 1, 1, 50, 1)[i] if i < 6 else 0                                        # the other request: single tokens beside portions and the reverse
            rows = list(range(at, at + n)) + list(range(T + ato, T + ato + no))
            b = LO.RaggedBatch.build([n] + ([no] if no else []), [at] + ([ato] if no else []), [2] + ([0] if no else []), [list(range(64))] + ([list(range(64, 80))] if no else []), 8, "cuda")
            y = run(torch.tensor(rows, device="cuda"), b)
            got.append(y[:n]); got_o.append(y[n:])
            at += n; ato += no
        assert ato == To
        assert rel_err(torch.cat(got), want) < tol and rel_err(torch.cat(got_o), other) < tol, dt_
        state2 = state.clone()                                                                  # one step over everything, from a used slot: the same final state
        b = LO.RaggedBatch.build([T, To], [0, 0], [2, 0], [list(range(64)), list(range(64, 80))], 8, "cuda")
        y = run(torch.arange(T + To, device="cuda"), b)
        assert rel_err(y, torch.cat([want, other])) < tol and rel_err(state[[0, 2]].cpu(), state2[[0, 2]].cpu()) < max(tol, 1e-4)


@gpu
def test_linear_recurrence_with_extreme_decays():
    """Decays of one, next to nothing and zero (a log decay without a bound); large step sizes."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(5)
    H, D, Dv, T = 4, 16, 16, 150
    x = torch.randn(T, H * (2 * D + Dv), generator=g).bfloat16()
    cols = (0, H * D, 2 * H * D)
    b = LO.RaggedBatch.build([T], [0], [0], [list(range(32))], 8, "cuda")
    q, k, v = (x.double()[:, c:c + H * D].view(T, H, D) for c in cols)
    decay = torch.tensor([1.0, 1e-30, 0.0, 0.9999])
    for dt in (torch.float32, torch.bfloat16):
        state = torch.zeros(1, H, D, Dv, device="cuda")
        y = LO.linear_scan(x.cuda().to(dt), cols, b, H, H, D, Dv, state, decay=decay.cuda())
        assert rel_err(y.cpu(), scan_reference(q, k, v, H, H, decay, None, None, None, None)) < 1e-4
        dts = torch.randn(T, H, generator=torch.Generator().manual_seed(6)).bfloat16() * 20
        a_log, bias = torch.tensor([3.0, -9.0, 1.0, 0.0]), torch.tensor([1.0, 0.0, 30.0, -30.0])
        y = LO.linear_scan(x.cuda().to(dt), cols, b, H, H, D, Dv, state, dt=dts.cuda().to(dt), a_log=a_log.cuda(), dt_bias=bias.cuda())
        assert rel_err(y.cpu(), scan_reference(q, k, v, H, H, None, dts.double(), a_log.double(), bias.double(), None)) < 1e-4


@gpu
@pytest.mark.parametrize("H,G,D,Dv", [(6, 2, 24, 20), (10, 1, 64, 64), (8, 8, 32, 32), (2, 1, 128, 128), (12, 4, 16, 16), (40, 1, 16, 32), (1, 1, 20, 10), (16, 2, 64, 96), (24, 2, 72, 32)])
@pytest.mark.parametrize("chunk", [1, 7, 32, 48, 90])
def test_chunked_attention_with_capped_scores(H, G, D, Dv, chunk):
    """Every attention launch (float; both matrix-core kernels; the 128-row form) over chunks smaller than, equal to and larger than their
    tiles: portions cut anywhere, single tokens, one in the denominator, a gate per head, a scaled output inside wider rows."""
    from jacobiforcing_amd import layer_ops as LO
    g = torch.Generator().manual_seed(H * 100 + chunk)
    rn = lambda *s: torch.randn(*s, generator=g)
    T, R = 211, 5 if chunk == 48 else 2
    cap, scale, out_scale = 4.0, 0.8 * D ** -0.5, 0.6
    counts_list = [[100, 1], [1, 7], [110, 203]]
    if R == 5:
        counts_list = [[T] * R]                                                                 # many rows: the launch's form for long portions
    q, k, v, gate = (rn(R, T, w_) * f for w_, f in ((H * D, 3.0), (G * D, 1.0), (G * Dv, 1.0), (H, 2.0)))
    per = -(-T // 16)
    tables = [list(range(r * per, (r + 1) * per))[::-1] for r in range(R)]
    vis = O.chunk_mask(T, chunk)
    sink = torch.zeros(H, device="cuda")
    for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2e-2)):
        kc, vc = torch.full((R * per * 16, G * D), 50.0, dtype=dt, device="cuda"), torch.full((R * per * 16, G * Dv), 50.0, dtype=dt, device="cuda")
        qd, kd, vd, gd = (x.cuda().to(dt) for x in (q, k, v, gate))
        want = []
        for r in range(R):
            kk = kd[r].cpu().double().view(T, G, D).repeat_interleave(H // G, 1)
            vv = vd[r].cpu().double().view(T, G, Dv).repeat_interleave(H // G, 1)
            s = O.soft_cap(torch.einsum("ihd,jhd->hij", qd[r].cpu().double().view(T, H, D), kk) * scale, cap)
            o = torch.einsum("hij,jhd->ihd", O.softmax_one_more(s, vis), vv) * torch.sigmoid(gd[r].cpu().double()).unsqueeze(-1) * out_scale
            want.append(o.reshape(T, H * Dv))
        at = [0] * R
        for counts in counts_list:
            starts = list(at)
            b = LO.RaggedBatch.build(counts, starts, list(range(R)), tables, 16, "cuda")
            pick = lambda x: torch.cat([x[r, starts[r]:starts[r] + counts[r]] for r in range(R)]).contiguous()
            kc[b.kv_slot], vc[b.kv_slot] = pick(kd), pick(vd)
            n = sum(counts)
            sweep = LO.attn_sweep_tile_rows(dt, H, G, D, Dv, kc, vc) > 0
            for kernel in ([LO.attn_sweep] if sweep else []) + [LO.attn_window]:
                buf = torch.full((n, H * Dv + 24), 5.0, dtype=dt, device="cuda")
                kw = dict(sink=sink, gate_per_head=True, chunk=chunk, softcap=cap, out_scale=out_scale, out=buf[:, 8:8 + H * Dv])
                if kernel is LO.attn_sweep:
                    kernel(pick(qd), kc, vc, b, H, G, D, Dv, scale, 0, gate=pick(gd), **kw)
                else:
                    kernel(pick(qd), pick(gd), kc, vc, b, H, G, D, Dv, scale, 0, 0, None, None, None, **kw)
                w_ = torch.cat([want[r][starts[r]:starts[r] + counts[r]] for r in range(R)])
                assert rel_err(buf[:, 8:8 + H * Dv].float().cpu(), w_) < tol, (dt, kernel.__name__, counts)
                assert float(buf[:, :8].float().sum()) == 40.0 * n and float(buf[:, 8 + H * Dv:].float().sum()) == 80.0 * n
            at = [a + c for a, c in zip(at, counts)]
    with pytest.raises(ValueError):
        LO.attn_window(pick(qd), None, kc, vc, b, H, G, D, Dv, scale, 4, 0, None, None, None, chunk=8)


# ---- each mixer alone ---------------------------------------------------------------------------------------------------------------------
MIXER_SIZES = [lightning(), lightning(1, 9, 5), lightning(3, 64, 64), lightning(2, 128, 128), lightning(5, 200, 24), lightning(3, 32, 160),
               mamba(), mamba(3, 3, 7, 5, 1, 1), mamba(8, 2, 64, 32, 4, 4), mamba(4, 1, 128, 64, 4, 1), mamba(2, 1, 33, 9, 5, 2), mamba(1, 1, 16, 48, 8, 6), mamba(6, 6, 24, 8, 2, 2),
               parallel(), parallel(1, 1, 10, 7, 0, chunk=5, right=lightning(1, 9, 5)), parallel(10, 1, 64, 64, 16, 1e5, 0.15, 20.0, 24, lightning(3, 32, 64)),
               parallel(8, 8, 32, 32, 32, 1e4, 0.2, 1.5, 64, lightning(2, 64, 16)), parallel(5, 1, 14, 9, 6, 50.0, 0.5, 2.0, 33, lightning(3, 6, 11), 0.0, 1.0),
               parallel(12, 3, 40, 32, 8, 1e4, 0.2, 20.0, 1000, lightning(3, 16, 20))]


@gpu
@pytest.mark.parametrize("layer", MIXER_SIZES, ids=lambda L: L["type"][0] + "-".join(str(v) for v in L["mixer"].get("left", L["mixer"]).values() if not isinstance(v, (dict, float, list))))
def test_each_mixer_alone_in_portions_and_single_tokens(layer):
    """One mixer on the oracle's own inputs, float32 and bfloat16: a prompt's first part in one step, a second part that starts inside a page
    and inside a chunk, two tokens, then single tokens, then a long portion, on shuffled pages and a poisoned slot."""
    W, cuts = 64, (19, 14, 2, 1, 1, 1, 5, 81)
    T = sum(cuts)
    cfg = make_cfg([layer], width=W, vocab=40, loop=None)
    t = tensors_for(cfg, 5)
    P = mixer_tensors(t, 0)
    h = torch.randn(T, W, generator=torch.Generator().manual_seed(7))
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        rig = Rig(cfg, tensors=t, dtype=dtype, pages=24)
        rig.poison()
        hd = h.cuda().to(dtype)
        want = O.MIXERS[layer["type"]](hd.cpu().double(), P, layer["mixer"], 1e-5)
        run = {"lightning": rig.model._lightning, "mamba2": rig.model._mamba2, "parallel": rig.model._parallel}[layer["type"]]
        got, at = [], 0
        for n in cuts:
            b, _ = rig.batch([("r", [0] * n)])
            got.append(run(0, 0, hd[at:at + n].contiguous(), b, rig.cache).float().cpu())
            at += n
        assert rel_err(torch.cat(got), want) < tol, dtype


# ---- whole models -------------------------------------------------------------------------------------------------------------------------
@gpu
@pytest.mark.parametrize("name", ["a", "b", "c", "d"])
def test_whole_prompt_and_every_layer_run(name):
    rig = Rig(SHAPES[name](), seed=3)
    t = toks(45, rig.cfg.vocab_size, 1)
    tr_o, tr_g = [], []
    want = rig.oracle(t, tr_o)
    got = rig.step([("r", t)], tr_g)
    assert len(tr_g) == len(tr_o) == len(rig.cfg.runs())
    for li, (g_, o_) in enumerate(zip(tr_g, tr_o)):
        assert rel_err(g_.cpu(), o_) < F32_TOL, li
    assert rel_err(got, want) < F32_TOL
    rig.end("r")
    assert rel_err(rig.step([("again", t)]), want) < F32_TOL                                    # without the trace: the updates folded into the norms' launches
    half = Rig(SHAPES[name](), seed=3, dtype=torch.bfloat16)
    assert close(half.step([("r", t)]), want, torch.bfloat16)


@gpu
@pytest.mark.parametrize("name", ["a", "b", "c", "d"])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_prefill_equals_token_by_token_decoding(name, dtype):
    rig = Rig(SHAPES[name](), seed=5, dtype=dtype)
    rig.poison()
    t = toks(49, rig.cfg.vocab_size, 2)
    want = rig.oracle(t)
    got = torch.cat([rig.step([("r", [x])]) for x in t])
    whole = rig.step([("p", t)])
    assert close(got, want, dtype) and close(whole, want, dtype)
    assert dtype == torch.float32 or close(whole, got, dtype)


@gpu
@pytest.mark.parametrize("cuts", [[2] * 24, [1, 2, 3, 5, 8, 13, 7, 9], [7, 9, 8, 24], [47, 1], [3, 45], [8] * 6, [15, 17, 1, 15], [11, 11, 11, 15], [10, 2, 10, 26], [5, 6, 22, 15]])
def test_portions_of_any_size(cuts):
    """Portions down to two tokens, at and beside the edges of pages (8), of the attention's chunks (11, 33 and 5) and of the recurrence's
    groups."""
    for name in ("a", "b"):
        rig = Rig(SHAPES[name](), seed=7)
        rig.poison()
        t = toks(sum(cuts), rig.cfg.vocab_size, 3)
        assert rel_err(rig.portions("r", t, cuts), rig.oracle(t)) < F32_TOL, name


@gpu
def test_long_portions_in_pieces_equal_the_whole():
    """bfloat16 sizes that run in pieces: prompts cut inside and at the groups of 64, pieces joined across steps; float32 beside them."""
    cfg = shape_c()
    t = tensors_for(cfg, 13)
    tk = toks(300, cfg["vocab"], 4)
    want = O.forward(cfg, t, tk, torch.float64)
    for dtype in (torch.float32, torch.bfloat16):
        for cuts in ([300], [64, 236], [63, 65, 172], [100, 1, 199], [32, 31, 237], [299, 1]):
            rig = Rig(cfg, tensors=t, dtype=dtype, pages=48)
            rig.poison()
            assert close(rig.portions("r", tk, cuts), want, dtype), (dtype, cuts)


@gpu
def test_unequal_requests_in_one_batch_equal_each_alone():
    for name in ("a", "b", "c"):
        for dtype in (torch.float32, torch.bfloat16):
            rig = Rig(SHAPES[name](), seed=3, pages=96, dtype=dtype)
            V = rig.cfg.vocab_size
            seqs = {"x": toks(41, V, 4), "y": toks(3, V, 5), "z": toks(18, V, 6), "w": toks(120, V, 7)}
            plan = [[("x", 17), ("y", 1), ("w", 33)], [("x", 1), ("y", 2), ("z", 18), ("w", 1)], [("x", 23), ("w", 86)]]
            at, got = {k: 0 for k in seqs}, {k: [] for k in seqs}
            for step in plan:
                out = rig.step([(k, seqs[k][at[k]:at[k] + n]) for k, n in step])
                r0 = 0
                for k, n in step:
                    got[k].append(out[r0:r0 + n]); r0 += n; at[k] += n
            for k, s in seqs.items():
                assert at[k] == len(s) and close(torch.cat(got[k]), rig.oracle(s), dtype), (name, k, dtype)


@gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_freed_pages_and_slots_are_used_again(dtype):
    """Two slots, a pool that holds two requests: requests end, their pages and slots go to new ones; old keys, states and convolution
    inputs must not leak."""
    rig = Rig(shape_a(), seed=17, pages=12, slots=2, dtype=dtype)
    V = rig.cfg.vocab_size
    rig.poison()
    for rnd in range(4):
        a, b = toks(40 + rnd, V, 20 + rnd), toks(17 + 3 * rnd, V, 30 + rnd)
        ga = rig.step([("a", a[:25]), ("b", b[:1])])                                           # b starts with a single token in a used slot
        gb = rig.step([("a", a[25:]), ("b", b[1:])])
        got_a = torch.cat([ga[:25], gb[:len(a) - 25]])
        got_b = torch.cat([ga[25:], gb[len(a) - 25:]])
        assert close(got_a, rig.oracle(a), dtype) and close(got_b, rig.oracle(b), dtype), rnd
        used = set(rig.req["a"]["pages"]) | set(rig.req["b"]["pages"])
        rig.end("b"); rig.end("a")
        assert len(rig.free_pages) == 12 and len(used) >= 8


def peaked_model(chunk, cap=60.0, scale=3.0):
    """One parallel layer whose right side is switched off, a sharp softmax, a rotation over a small part of the head.  Returns (cfg, tensors,
    hot query token, hot key token, scores): the pair of tokens whose unrotated score is the largest."""
    V, H, D = 40, 2, 16
    cfg = make_cfg([parallel(H, 1, D, 16, 4, 10000.0, scale, cap, chunk, lightning(1, 8, 8), 1.0, 0.0)], width=32, vocab=V, loop=None)
    t = tensors_for(cfg, 23)
    h = O.rms_norm(t["embed"].double(), t["l0.norm1"].double(), 1e-5)
    P = {k[len("l0.mix.left."):]: v.double() for k, v in t.items() if k.startswith("l0.mix.left.")}
    q = O.rms_norm(h @ P["q"].T + P["q.b"], P["q.norm"], 1e-5).view(V, H, D)[:, 0]
    k = O.rms_norm(h @ P["k"].T + P["k.b"], P["k.norm"], 1e-5)
    s = q[:, 4:] @ k[:, 4:].T
    qi, kj = divmod(int(s.argmax()), V)
    return cfg, t, qi, kj, s


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
@pytest.mark.parametrize("chunk,place", [(400, 16), (400, 23), (400, 24), (400, 0), (150, 150), (150, 149), (144, 144), (144, 143), (147, 152)])
def test_a_far_key_among_hundreds(dtype, tol, chunk, place):
    """The hot key sits up to 300 tokens back — at a page's first or last place, at position 0, at the first place of the reader's chunk and at the
    last place of the chunk before (which must not be seen) — and is read by a prompt's portion and by a single decoded token."""
    cfg, t, qi, kj, s = peaked_model(chunk)
    dull = [x for x in np.argsort(s[qi].numpy())[:12].tolist() if x != kj]
    T = min(300, 2 * chunk)
    seq = [dull[i % len(dull)] for i in range(T)]
    seq[place], seq[T - 1], seq[T - 9] = kj, qi, qi
    rig = Rig(cfg, tensors=t, pages=64, dtype=dtype)
    got = rig.portions("r", seq, [121, T - 2 - 121, 1, 1])
    want = rig.oracle(seq)
    assert rel_err(got[-1], want[-1]) < tol and rel_err(got[T - 9], want[T - 9]) < tol and rel_err(got, want) < tol
    seq2 = list(seq)
    seq2[place] = dull[0]
    other = rig.oracle(seq2)
    seen = place // chunk == (T - 1) // chunk
    for at in (T - 1, T - 9):                                                                   # the test would see the key missing, or seen where it must not be
        assert (rel_err(other[at], want[at]) > 0.05) == seen
    if not seen:
        wide = dict(cfg, layers=[json.loads(json.dumps(cfg["layers"][0]))])
        wide["layers"][0]["mixer"]["left"]["mask"]["size"] = chunk * 4
        assert rel_err(O.forward(wide, t, seq, torch.float64)[-1], want[-1]) > 0.05


@gpu
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
def test_chunk_borders_in_decoding(dtype, tol):
    """Single decoded tokens and pairs over several chunk borders; the first token of a chunk sees itself alone, beside the one in the denominator."""
    cfg, t, qi, kj, _ = peaked_model(9, cap=6.0)
    seq = [kj if i % 9 == 8 else qi for i in range(60)]                                         # a hot key at every chunk's last place, a hot query right behind it
    want = O.forward(cfg, t, seq, torch.float64)
    for cuts in ([1] * 60, [2] * 30, [8, 1, 1, 1, 7, 1, 1, 40], [9, 9, 9, 9, 9, 9, 6], [26, 1, 1, 32]):
        rig = Rig(cfg, tensors=t, dtype=dtype)
        rig.poison()
        assert rel_err(rig.portions("r", seq, cuts), want) < tol, cuts
    # without the one in the denominator, without the cap, with a window instead of chunks: each would show
    P = {k[len("l0.mix.left."):]: v.double() for k, v in t.items() if k.startswith("l0.mix.left.")}
    h = O.rms_norm(t["embed"].double()[torch.tensor(seq)], t["l0.norm1"].double(), 1e-5)
    m = cfg["layers"][0]["mixer"]["left"]
    base = O.attention(h, P, m, 1e-5)
    keep = O.softmax_one_more
    try:
        O.softmax_one_more = lambda s, vis: torch.softmax(s.masked_fill(~vis, float("-inf")), -1)
        assert rel_err(O.attention(h, P, m, 1e-5), base) > 1e-3
    finally:
        O.softmax_one_more = keep
    assert rel_err(O.attention(h, P, dict(m, softcap=1e9), 1e-5), base) > 1e-3
    keep = O.chunk_mask
    try:
        O.chunk_mask = lambda T, size: torch.ones(T, T, dtype=torch.bool).tril() & ~torch.ones(T, T, dtype=torch.bool).tril(-size)
        assert rel_err(O.attention(h, P, m, 1e-5), base) > 0.05
    finally:
        O.chunk_mask = keep


@gpu
@pytest.mark.parametrize("kind", ["lightning", "mamba2"])
@pytest.mark.parametrize("dtype,tol", [(torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)])
def test_an_old_write_stays_in_the_recurrent_state(kind, dtype, tol):
    """A layer that hardly decays: what token 3 wrote is still read 250 tokens later, through portions, a used slot and decoding."""
    layer = lightning(2, 16, 16, [0.9999, 0.9998]) if kind == "lightning" else mamba(2, 1, 16, 16, 2, 1)
    cfg = make_cfg([layer], width=32, vocab=40, loop=None)
    t = tensors_for(cfg, 41)
    if kind == "mamba2":
        t["l0.mix.A_log"] = torch.full((2,), -9.0)
        t["l0.mix.D"] = torch.zeros(2)
    T = 256
    seq = [x % 4 for x in toks(T, 40, 9)]
    seq[3] = 39
    t["embed"][39] *= 4
    if kind == "lightning":                                                                     # the write stands out among 250 others
        t["l0.norm1"] = t["l0.norm1"] * 3
    rig = Rig(cfg, tensors=t, pages=48, dtype=dtype)
    rig.step([("old", toks(20, 40, 1))])
    rig.end("old")
    got = rig.portions("r", seq, [5, 125, T - 133, 1, 1, 1])
    want = rig.oracle(seq)
    assert rel_err(got, want) < tol and rel_err(got[-1], want[-1]) < tol
    seq2 = list(seq)
    seq2[3] = 0
    assert rel_err(rig.oracle(seq2)[-1], want[-1]) > 3 * F32_TOL
    if kind == "mamba2":
        t2 = dict(t)
        t2["l0.mix.A_log"] = torch.full((2,), 3.0)                                              # with a fast decay the old write is gone: the test rests on the state
        assert rel_err(O.forward(cfg, t2, seq2, torch.float64)[-1], O.forward(cfg, t2, seq, torch.float64)[-1]) < 1e-6


@gpu
def test_every_pass_of_the_loop_has_its_own_state_and_step():
    """A looped model differs from the same layers with one state for all passes, and from one whose passes share a step vector."""
    cfg = shape_a()
    t = tensors_for(cfg, 47)
    tk = toks(30, cfg["vocab"], 5)
    rig = Rig(cfg, tensors=t)
    want = rig.oracle(tk)
    assert rel_err(rig.portions("r", tk, [13, 1, 1, 15]), want) < F32_TOL
    for change in (lambda d: d["loop.step"].__setitem__(2, d["loop.step"][1]), lambda d: d["loop.in"].__setitem__((slice(None), slice(96, 192)), 0.0)):
        t2 = {k: v.clone() for k, v in t.items()}
        change(t2)
        assert rel_err(O.forward(cfg, t2, tk, torch.float64), want) > 0.05
    assert len({x.data_ptr() for x in rig.cache.state if x is not None}) == len(rig.cfg.runs())


@gpu
def test_the_first_tokens_of_a_sequence():
    """One, two and three tokens in a slot and on pages that hold another request's keys, state and convolution inputs."""
    for name in ("a", "b"):
        rig = Rig(SHAPES[name](), seed=19, slots=1, pages=16)
        V = rig.cfg.vocab_size
        rig.step([("old", toks(30, V, 1))])
        rig.end("old")
        for n in (1, 2, 3):
            t = toks(n + 1, V, 50 + n)
            got = torch.cat([rig.step([("new", t[:n])]), rig.step([("new", t[n:])])])
            assert rel_err(got, rig.oracle(t)) < F32_TOL, (name, n)
            rig.end("new")


@gpu
@pytest.mark.parametrize("name,dtype", [("b", torch.float32), ("c", torch.bfloat16)])
def test_long_decoding(name, dtype):
    rig = Rig(SHAPES[name](), seed=29, pages=64, dtype=dtype)
    t = toks(200, rig.cfg.vocab_size, 8)
    want = rig.oracle(t)
    got = rig.portions("r", t, [40] + [1] * 160)
    assert close(got, want, dtype) and close(got[-20:], want[-20:], dtype)


def random_cfg(r):
    def light():
        H = r.choice([1, 2, 3, 5, 8])
        return lightning(H, r.choice([4, 8, 16, 24, 40, 64]), r.choice([6, 8, 16, 32, 70]), [r.choice([0.5, 0.9, 0.99, 0.999, r.random()]) for _ in range(H)])
    layers = []
    for _ in range(r.choice([1, 2, 3, 4])):
        kind = r.choice(["lightning", "mamba2", "parallel"])
        if kind == "lightning":
            L = light()
        elif kind == "mamba2":
            G = r.choice([1, 2, 3])
            H, Dv = G * r.choice([1, 2, 4]), r.choice([8, 12, 32])
            L = mamba(H, G, r.choice([8, 16, 24, 64]), Dv, r.choice([1, 2, 3, 4, 5]), r.choice([1, G, H]))
        else:
            kv, D = r.choice([1, 2, 3]), r.choice([8, 16, 24, 32, 64])
            dims = r.choice([d for d in (0, 2, 4, 6, 8, 12, 16, 32) if d <= D])
            L = parallel(kv * r.choice([1, 2, 4]), kv, D, r.choice([D, 16, 32, 40]), dims, r.choice([50.0, 1e4, 1e6]), r.choice([D ** -0.5, 0.2]), r.choice([1.0, 5.0, 50.0]),
                         r.choice([1, 3, 8, 16, 21, 64]), light(), r.choice([0.5, 1.0, 1.7]), r.choice([0.3, 1.0]))
        L["mlp"] = None if r.random() < 0.4 else dense(r.choice([24, 56, 100]))
        layers.append(L)
    a = r.randrange(len(layers))
    loop = None if r.random() < 0.15 else (a, r.randint(a + 1, len(layers)), r.choice([1, 2, 3]))
    return make_cfg(layers, width=r.choice([32, 48, 62, 100]), vocab=r.choice([30, 77, 131]), eps=r.choice([1e-5, 1e-6, 1e-3]), loop=loop)


@gpu
@pytest.mark.parametrize("seed", range(14))
def test_random_configurations_in_a_mixed_schedule(seed):
    """Random layer orders, loops, head counts, sizes, taps and constants; two requests of unequal length in a random schedule of portions and
    single tokens, float32 and bfloat16."""
    r = random.Random(2000 + seed)
    cfg = random_cfg(r)
    t = tensors_for(cfg, seed)
    V = cfg["vocab"]
    seqs = {"x": toks(r.choice([9, 31, 60, 110]), V, seed), "y": toks(r.choice([2, 17, 45]), V, seed + 100)}
    plan, at = [], {k: 0 for k in seqs}
    while any(at[k] < len(s) for k, s in seqs.items()):
        step = []
        for k, s in seqs.items():
            if at[k] < len(s) and r.random() < 0.8:
                n = min(len(s) - at[k], r.choice([1, 1, 2, 3, 7, 8, 9, 20, 40, 70]))
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
            assert close(torch.cat(got[k]), want[k], dtype), (cfg, k, dtype)


# ---- the engine ---------------------------------------------------------------------------------------------------------------------------
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
    """LLM.generate on a checkpoint directory: registry -> loader -> scheduler (prompts cut to the token budget, admissions limited by
    two slots, pages reused) -> ragged step -> argmax.  float32 so that the greedy choice is the oracle's."""
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
def test_a_preempted_request_starts_again_from_an_empty_state(tmp_path):
    """Three pages for two requests that need five: the newer one is preempted while it decodes, gives pages and slot back and is
    prefilled again later — its states and convolution inputs start from nothing, the results are the oracle's."""
    from jacobiforcing_amd import LLM, SamplingParams
    cfg_dict = shape_a()
    tensors = tensors_for(cfg_dict, 43)
    path = _write_model(tmp_path, cfg_dict, tensors)
    V = cfg_dict["vocab"]
    prompts = [toks(110, V, 61), toks(60, V, 62)]
    llm = LLM(path, tokenizer_path="none", dtype="float32", kvcache_block_size=64, num_kvcache_blocks=3, max_num_seqs=2, max_model_len=192,
              max_num_batched_tokens=192, device="cuda")
    preempted = []
    keep = llm.scheduler.preempt
    llm.scheduler.preempt = lambda seq: (preempted.append(seq.seq_id), keep(seq))[1]
    out = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True), use_tqdm=False)
    assert preempted, "the pool was meant to run out"
    for p, o in zip(prompts, out):
        assert o["token_ids"] == _oracle_greedy(cfg_dict, tensors, p, 20)
    assert len(llm.scheduler.block_manager.free_block_ids) == 3 and len(llm.model_runner.free_rows) == 2


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
