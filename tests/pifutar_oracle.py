"""A plain, slow model of the Pifutar design in float64, one function per mechanism, written from the design's equations.
It shares no code with the package: it parses the config dictionary itself, takes the checkpoint's tensors by name, and
runs ONE whole sequence at a time (no cache, no batching), so everything the engine does with caches, slots and steps
can be held against it.

A layer:  x <- x + mixer(g1), x <- x + ff(g2), where g = h + causal_conv(h) and h is the layer's norm of x; the result
X_(i+1) is then replaced by a weighted sum of the embedding and of all layers' results so far.
"""
import math

import torch

F64 = torch.float64


def rms(x, eps, w=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def silu(z):
    return z * torch.sigmoid(z)


def input_conv(h, w):
    """h [T, width], w [width, taps] (the last column meets the current token): h plus its causal convolution, zeros in
    front of the sequence."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


def depth_average(c, results):
    """results: [embedding output, result of layer 0, ..., result of layer i]; c: as many numbers."""
    assert c.numel() == len(results)
    return sum(c[j] * r for j, r in enumerate(results))


def linear_attention(q, k, v, log_decay):
    """q, k [T, H, d], v [T, H, dv], log_decay [T, H, d]: S <- diag(exp(log_decay)) S + k v^T, o = S^T q, from zero."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = torch.exp(log_decay[t]).unsqueeze(2) * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(2)).sum(1)
    return out


def channel_log_decay(h, P, H, d, tau):
    """log of sigmoid(z)^(1 / tau), z a projection of low rank plus a bias, one number per key channel."""
    z = (h @ P["a1"].T) @ P["a2"].T + P["a2.b"]
    return (torch.nn.functional.logsigmoid(z) / tau).view(-1, H, d)


def gla(h, P, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ P["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ P["k"].T).view(T, H, d)
    v = (h @ P["v"].T).view(T, H, dv)
    o = linear_attention(q, k, v, channel_log_decay(h, P, H, d, float(m["tau"])))
    o = rms(o, eps, P["norm"]).reshape(T, H * dv)
    return (o * silu(h @ P["g"].T)) @ P["o"].T


def retention(h, P, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ P["q"].T).view(T, H, d)
    k = (h @ P["k"].T).view(T, H, d) * d ** -0.5
    v = (h @ P["v"].T).view(T, H, dv)
    ld = torch.log(torch.tensor(m["decay"], dtype=F64)).view(1, H, 1).expand(T, H, d)
    o = rms(linear_attention(q, k, v, ld), eps).reshape(T, H * dv)
    return (o * silu(h @ P["g"].T)) @ P["o"].T


def rotate_pairs(x, pos, dims, base):
    """x [T, ..., D]: entries (2i, 2i + 1) of the first `dims` turn by pos * base^(-2i / dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = (pos.to(F64) * base ** (-2.0 * i / dims)).view(-1, *([1] * (x.dim() - 2)))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


def window_mask(T, size):
    p = torch.arange(T)
    dist = p.view(-1, 1) - p.view(1, -1)
    return (dist >= 0) & (dist < size) if size else dist >= 0


def latents(h, P, m, eps):
    """The normed latent c [T, kv_rank] and the rotated key part [T, rot_dim] that a layer keeps."""
    R = m["kv_rank"]
    z = h @ P["dkv"].T
    rot = m.get("rot") or {}
    return rms(z[:, :R], eps, P["dkv.norm"]), rotate_pairs(z[:, R:], torch.arange(h.shape[0]), int(rot.get("dims", 0)), float(rot.get("base", 1.0)))


def latent_attention(h, P, m, kept):
    """`kept`: the latents, this layer's own or those of the layer it reads from."""
    T, H, d, dr, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = kept
    rot = m.get("rot") or {}
    q = (h @ P["q"].T).view(T, H, d + dr)
    qu, qr = q[..., :d], rotate_pairs(q[..., d:], torch.arange(T), int(rot.get("dims", 0)), float(rot.get("base", 1.0)))
    ku, v = (c @ P["uk"].T).view(T, H, d), (c @ P["uv"].T).view(T, H, dv)
    s = torch.einsum("ihd,jhd->hij", qu, ku) + torch.einsum("ihd,jd->hij", qr, kr)
    s = (s * float(m["scale"])).masked_fill(~window_mask(T, int((m.get("mask") or {}).get("size") or 0)), float("-inf"))
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, -1), v).reshape(T, H * dv) @ P["o"].T


def poly_norm(z, eps, c):
    return c[0] * rms(z, eps) + c[1] * rms(z ** 2, eps) + c[2] * rms(z ** 3, eps) + c[3]


def dense_ff(h, P, eps):
    return poly_norm(h @ P["up"].T, eps, P["act"]) @ P["down"].T


def expert(h, P, pre, limit):
    g = torch.clamp(h @ P[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ P[pre + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ P[pre + "down"].T


def moe_ff(h, P, mlp, tokens):
    """Experts by the token's id: row `id` of the table names them, each weighs 1 / top; the shared expert joins through a
    gate of its own."""
    table, top, limit = P["table"].long(), int(mlp["router"]["top"]), float(mlp["expert"]["limit"])
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in table[tok].tolist():
            out[t] += expert(h[t:t + 1], P, "e%d." % e, limit)[0] / top
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ P["shared.sg"].T) * expert(h, P, "shared.", float(mlp["shared"]["limit"]))
    return out


def sub(tensors, prefix):
    return {k[len(prefix):]: (v.to(F64) if v.is_floating_point() else v) for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens):
    """-> (logits [T, vocab], [what goes on from every layer])."""
    eps = float(cfg["norm"]["eps"])
    get = lambda n: tensors[n].to(F64)
    x = get("embed")[torch.as_tensor(tokens, dtype=torch.long)]
    results, after, kept = [x], [], {}
    for i, layer in enumerate(cfg["layers"]):
        pre, m = "l%d." % i, layer["mixer"]
        P = sub(tensors, pre + "mix.")
        g = input_conv(rms(x, eps, 1.0 + get(pre + "norm1")), get(pre + "canon1"))
        if layer["type"] == "gla":
            y = gla(g, P, m, eps)
        elif layer["type"] == "retention":
            y = retention(g, P, m, eps)
        else:
            if m.get("kv_from") is None:
                kept[i] = latents(g, P, m, eps)
            y = latent_attention(g, P, m, kept[i if m.get("kv_from") is None else int(m["kv_from"])])
        x = x + y
        mlp = layer.get("mlp")
        if mlp is not None:
            P = sub(tensors, pre + "mlp.")
            g = input_conv(rms(x, eps, 1.0 + get(pre + "norm2")), get(pre + "canon2"))
            x = x + (dense_ff(g, P, eps) if mlp.get("kind", "dense") == "dense" else moe_ff(g, P, mlp, list(tokens)))
        results.append(x)
        x = depth_average(get(pre + "dwa"), results)
        after.append(x)
    return rms(x, eps, 1.0 + get("final.norm")) @ get("embed").T, after
