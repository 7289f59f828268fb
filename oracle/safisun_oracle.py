"""Plain, slow restatement of the Safisun decoder in torch on the CPU, one function per mechanism.  Test infrastructure only:
nothing under ``jacobiforcing_amd/`` imports it and it shares no code with the package.  Every function works on ONE whole
sequence (tokens 0 .. T-1) in the dtype of its inputs (float32 or float64) and has no cache: attention is a masked score
matrix, the recurrent mixers are loops over the tokens from a zero state.

Notation: ``h`` [T, width] a sublayer's input, ``P`` a dict of a mixer's (or feed-forward's) tensors keyed by the name behind its
prefix (``q``, ``left.q.norm`` ...), ``m`` the layer's ``mixer`` entry and ``f`` its ``mlp`` entry of config.json."""
from __future__ import annotations

import torch


def rms_norm(x, w=None, eps=1e-5):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def angles(T, dims, base, dtype=torch.float64):
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=dtype)
    return torch.arange(T, dtype=dtype).view(T, 1) * f.view(1, -1)                         # [T, dims/2]


def rotate_neighbours(x, a):
    """x [T, heads, >= dims]: dimension 2i pairs with 2i + 1; a [T, dims/2]."""
    half = a.shape[1]
    c, s = a.cos().unsqueeze(1), a.sin().unsqueeze(1)
    u, v, rest = x[..., 0:2 * half:2], x[..., 1:2 * half:2], x[..., 2 * half:]
    out = torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)
    return torch.cat([out, rest], -1)


def chunk_mask(T, size):
    """visible[i, j]: j <= i and both in the same run of ``size`` positions counted from the sequence's start."""
    i = torch.arange(T)
    return (i.view(T, 1) >= i.view(1, T)) & (i.view(T, 1) // size == i.view(1, T) // size)


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def softmax_one_more(s, visible):
    """exp(s_j) / (1 + sum of exp(s_j)) over the visible keys; s [heads, T, T]."""
    s = s.masked_fill(~visible, float("-inf"))
    top = torch.clamp(s.amax(-1, keepdim=True), min=0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention(h, P, m, eps):
    """The left half of a parallel mixer."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ P["q"].T + P["q.b"], P["q.norm"], eps).view(T, H, D)
    k = rms_norm(h @ P["k"].T + P["k.b"], P["k.norm"], eps).view(T, G, D)
    v = (h @ P["v"].T + P["v.b"]).view(T, G, Dv)
    rot = m.get("rot") or {}
    if rot.get("dims", 0):
        a = angles(T, rot["dims"], rot["base"], h.dtype)
        q, k = rotate_neighbours(q, a), rotate_neighbours(k, a)
    k, v = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    s = soft_cap(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], m["softcap"])
    w = softmax_one_more(s, chunk_mask(T, m["mask"]["size"]))
    o = torch.einsum("hij,jhd->ihd", w, v) * torch.sigmoid(h @ P["g"].T).unsqueeze(-1)
    return o.reshape(T, H * Dv) @ P["o"].T


def decayed_sum(q, k, v, decay):
    """S_t = decay_t S_(t-1) + k_t v_t^T, o_t = S_t^T q_t for one head: q, k [T, D], v [T, Dv], decay [T]."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = []
    for t in range(q.shape[0]):
        S = decay[t] * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out)


def lightning_mixer(h, P, m, eps):
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ P["q"].T).view(T, H, D), silu(h @ P["k"].T).view(T, H, D)
    v = silu(h @ P["v"].T).view(T, H, Dv)
    o = torch.stack([decayed_sum(q[:, x], k[:, x], v[:, x], torch.full((T,), m["decay"][x], dtype=h.dtype)) for x in range(H)], 1)
    o = rms_norm(o.reshape(T, H * Dv), P["norm"], eps) * torch.sigmoid(h @ P["g"].T)
    return o @ P["o"].T


def short_conv(x, w, b):
    """x [T, C], w [C, taps], b [C]: y_t = b + sum_j w[:, j] * x_(t - taps + 1 + j), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    xp = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x], 0)
    y = b.expand(T, -1).clone()
    for j in range(taps):
        y = y + xp[j:j + T] * w[:, j]
    return y


def mamba2_mixer(h, P, m, eps):
    T, H, Dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * Dv
    z, xbc, dt = torch.split(h @ P["in"].T, [inner, inner + 2 * G * N, H], -1)
    x, B, C = torch.split(silu(short_conv(xbc, P["conv"], P["conv.b"])), [inner, G * N, G * N], -1)
    x, B, C = x.view(T, H, Dv), B.view(T, G, N), C.view(T, G, N)
    dt = softplus(dt + P["dt_bias"])
    y = torch.zeros(T, H, Dv, dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        a = torch.exp(-torch.exp(P["A_log"][hh]) * dt[:, hh])
        y[:, hh] = decayed_sum(C[:, g], B[:, g], dt[:, hh:hh + 1] * x[:, hh], a) + P["D"][hh] * x[:, hh]
    y = y.reshape(T, inner) * silu(z)
    ng = m["norm_groups"]
    y = rms_norm(y.view(T, ng, inner // ng), None, eps).reshape(T, inner) * P["norm"]
    return y @ P["o"].T


def sub(P, prefix):
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


def parallel_mixer(h, P, m, eps):
    return m["left_scale"] * attention(h, sub(P, "left."), m["left"], eps) + m["right_scale"] * lightning_mixer(h, sub(P, "right."), m["right"], eps)


def feed_forward(h, P):
    return (silu(h @ P["gate"].T) * (h @ P["up"].T)) @ P["down"].T


MIXERS = {"lightning": lightning_mixer, "mamba2": mamba2_mixer, "parallel": parallel_mixer}


def execution(cfg):
    """(layer, number of the pass that starts in front of it or None) in the order the layers run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    span = range(lp["start"], lp["stop"])
    return ([(i, None) for i in range(lp["start"])] + [(i, t if i == lp["start"] else None) for t in range(lp["times"]) for i in span] +
            [(i, None) for i in range(lp["stop"], n)])


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, trace=None):
    """Logits [T, vocab] of one whole sequence.  ``trace``, when a list, receives the residual stream after every layer run."""
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x0 = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = x0
    for i, p in execution(cfg):
        L, P = cfg["layers"][i], sub(t, f"l{i}.")
        if p is not None:
            x = torch.cat([x, x0], -1) @ t["loop.in"].T + t["loop.step"][p]
        x = x + rms_norm(MIXERS[L["type"]](rms_norm(x, P["norm1"], eps), sub(P, "mix."), L["mixer"], eps), P["norm1b"], eps)
        if L.get("mlp") is not None:
            x = x + rms_norm(feed_forward(rms_norm(x, P["norm2"], eps), sub(P, "mlp.")), P["norm2b"], eps)
        if trace is not None:
            trace.append(x.clone())
    return rms_norm(x, t["final.norm"], eps) @ t["head"].T
