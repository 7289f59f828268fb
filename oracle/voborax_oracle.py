"""Plain, slow restatement of the Voborax decoder in torch on the CPU, one function per mechanism.  Test infrastructure only:
nothing under ``jacobiforcing_amd/`` imports it and it shares no code with the package.  Every function works on ONE whole
sequence (tokens 0 .. T-1) in the dtype of its inputs (float32 or float64) and has no cache: attention is a masked score matrix
over keys and values built from every token's latent, a layer that borrows another layer's latents is handed them.

Notation: ``h`` [T, width] a sublayer's input, ``P`` a dict of a layer's tensors keyed by the name behind ``l<i>.`` (``mix.uq``,
``mlp.e3.up`` ...), ``m`` the layer's ``mixer`` entry and ``f`` its ``mlp`` entry of config.json."""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def rotate(x, base):
    """x [T, heads, dims], row t at position t: dimensions 2i and 2i + 1 turn together by t * base^(-2i/dims)."""
    T, _, dims = x.shape
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    a = torch.arange(T, dtype=x.dtype).view(T, 1, 1) * f
    u, v = x[..., 0::2], x[..., 1::2]
    out = torch.empty_like(x)
    out[..., 0::2], out[..., 1::2] = u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()
    return out


def visible(T, window=None):
    """[T, T] bool: query i sees key j."""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    see = j <= i
    return see if window is None else see & (i - j < window)


def masked_softmax(s, see, sink=None):
    """s [heads, T, T] -> weights; with ``sink`` [heads] the denominator holds exp(sink_h) as well."""
    s = s.masked_fill(~see, float("-inf"))
    if sink is None:
        return torch.softmax(s, -1)
    full = torch.cat([s, sink.view(-1, 1, 1).expand(-1, s.shape[1], 1)], -1)
    return torch.softmax(full, -1)[..., :-1]


def latent_queries(h, P, heads, eps):
    return (rms_norm(h @ P["mix.dq"].T, P["mix.dq.norm"], eps) @ P["mix.uq"].T).view(h.shape[0], heads, -1)


def latents(h, P, m, eps):
    """What a layer's cache holds: the normed latent [T, kv_rank] and the rotated shared key [T, rot_dim] (None without rotation)."""
    d, R = h @ P["mix.dkv"].T, m["kv_rank"]
    turned = rotate(d[:, R:].unsqueeze(1), m["rot"]["base"])[:, 0] if m.get("rot_dim") else None
    return rms_norm(d[:, :R], P["mix.dkv.norm"], eps), turned


def windowed_latent_attention(h, P, m, eps, held):
    """``held``: this layer's latents, or those of the layer it borrows from."""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    c, kr = held
    q = latent_queries(h, P, H, eps)
    k, v = (c @ P["mix.uk"].T).view(T, H, D), (c @ P["mix.uv"].T).view(T, H, m["vdim"])
    s = torch.einsum("ihd,jhd->hij", q[..., :D], k) + torch.einsum("ihd,jd->hij", rotate(q[..., D:], m["rot"]["base"]), kr)
    w = masked_softmax(s * m["scale"], visible(T, m["mask"]["size"]))
    o = torch.einsum("hij,jhd->ihd", w, v) * torch.sigmoid(h @ P["mix.g"].T).unsqueeze(-1)
    return o.reshape(T, -1) @ P["mix.o"].T


def causal_latent_attention(h, P, m, eps):
    T, H = h.shape[0], m["heads"]
    c, _ = latents(h, P, m, eps)
    q = latent_queries(h, P, H, eps)
    k, v = (c @ P["mix.uk"].T).view(T, H, m["dim"]), (c @ P["mix.uv"].T).view(T, H, m["vdim"])
    w = masked_softmax(torch.einsum("ihd,jhd->hij", q, k) * m["scale"], visible(T), P["mix.sink"])
    return torch.einsum("hij,jhd->ihd", w, v).reshape(T, -1) @ P["mix.o"].T


def route(z, correction, top):
    """z [T, E] -> (chosen [T, top], weights [T, top]): softmax over all, the correction only in the choice."""
    s = torch.softmax(z, -1)
    idx = torch.sort(s + correction, dim=-1, descending=True, stable=True)[1][:, :top]
    w = s.gather(1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20)


def expert(h, P, name):
    return (silu(h @ P[name + "gate"].T) * (h @ P[name + "up"].T)) @ P[name + "down"].T


def dense_feed_forward(h, P):
    return gelu_tanh(h @ P["mlp.up"].T + P["mlp.up.b"]) @ P["mlp.down"].T + P["mlp.down.b"]


def routed_feed_forward(h, P, f):
    E = f["router"]["experts"]
    idx, wt = route(h @ P["mlp.router"].T, P["mlp.correction"], f["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(idx[t].tolist(), wt[t]):
            out[t] = out[t] + w * (expert(h[t], P, f"mlp.e{e}.") if e < E else h[t])
    return out + expert(h, P, "mlp.shared.") if f.get("shared") is not None else out


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, trace=None):
    """Logits [T, vocab] of one whole sequence.  ``trace``, when a list, receives the stream after every layer."""
    t = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    held = {}
    for i, L in enumerate(cfg["layers"]):
        P = {k[len(f"l{i}."):]: v for k, v in t.items() if k.startswith(f"l{i}.")}
        m, f = L["mixer"], L.get("mlp")
        if L["type"] == "latent_attention":
            j = m.get("kv_from")
            held[i] = latents(x, P, m, eps) if j is None else held[j]
            y = windowed_latent_attention(x, P, m, eps, held[i])
        else:
            y = causal_latent_attention(x, P, m, eps)
        x = x + mult * layer_norm(y, P["norm1"], eps)
        if f is not None:
            y = dense_feed_forward(x, P) if f["kind"] == "dense" else routed_feed_forward(x, P, f)
            x = x + mult * layer_norm(y, P["norm2"], eps)
        if trace is not None:
            trace.append(x.clone())
    return layer_norm(x, t["final.norm"], eps) @ t["head"].T
