"""A plain, slow model of the Migenex design in float64, one function per mechanism, written from the design's equations.
It shares no code with the package: it parses the config dictionary itself, takes the checkpoint's tensors by name, and
runs ONE whole sequence at a time (no cache, no batching), so everything the engine does with caches, slots and steps
can be held against it.

A layer:  x <- x + m N1b(mixer(N1(x))), x <- x + m N2b(ff(N2(x))), every N an RMS norm with a plain weight; a stretch of
layers runs several times, and each of its passes starts from a linear map of the stream beside the embedding output.
"""
import torch

F64 = torch.float64


def rms(x, eps, w=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def bigram_rows(tokens, mul_prev, mul_cur, buckets):
    """The row of the bigram table for every token: a hash of (previous token, token), and a row of its own for the first."""
    return [buckets if t == 0 else (tokens[t - 1] * mul_prev + tokens[t] * mul_cur) % buckets for t in range(len(tokens))]


def embedding(cfg, tensors, tokens):
    e = cfg["embedding"]
    x = tensors["embed"].to(F64)[torch.as_tensor(tokens, dtype=torch.long)] * float(e["scale"])
    if e.get("bigram"):
        b = e["bigram"]
        x = x + tensors["bigram"].to(F64)[torch.as_tensor(bigram_rows(list(tokens), b["mul_prev"], b["mul_cur"], b["buckets"]), dtype=torch.long)]
    return x


def rotate_halves(x, pos, dims, base):
    """x [T, heads, D]: entries (i, i + dims / 2) of the first `dims` turn by pos * base^(-2i / dims)."""
    out, h = x.clone(), dims // 2
    for i in range(h):
        a = (pos.to(F64) * base ** (-2.0 * i / dims)).view(-1, 1)
        u, v = x[..., i], x[..., i + h]
        out[..., i], out[..., i + h] = u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)
    return out


def rotate_pairs(x, pos, dims, base):
    """The same with neighbours: entries (2i, 2i + 1)."""
    out = x.clone()
    for i in range(dims // 2):
        a = (pos.to(F64) * base ** (-2.0 * i / dims)).view(-1, 1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)
    return out


def visible(T, size=0):
    """[T, T]: query i sees key j when 0 <= i - j (< size)."""
    p = torch.arange(T)
    dist = p.view(-1, 1) - p.view(1, -1)
    return (dist >= 0) & (dist < size) if size else dist >= 0


def softmax_attention(q, k, v, scale, mask, cap=0.0):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H dv]."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        out.append(torch.softmax(s.masked_fill(~mask, float("-inf")), -1) @ v[:, h // per])
    return torch.stack(out, 1).reshape(T, -1)


def full_attention(h, P, m, eps):
    """Queries and keys normed per head with a weight, then rotated in halves; capped scores over the whole context."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    rot, pos = m.get("rot") or {}, torch.arange(h.shape[0])
    q, k = rms((h @ P["q"].T).view(T, H, d), eps, P["q.norm"]), rms((h @ P["k"].T).view(T, G, d), eps, P["k.norm"])
    q, k = (rotate_halves(x, pos, int(rot.get("dims", 0)), float(rot.get("base", 1.0))) for x in (q, k))
    v = (h @ P["v"].T).view(T, G, m["vdim"])
    return softmax_attention(q, k, v, float(m["scale"]), visible(T), float(m.get("softcap") or 0.0)) @ P["o"].T


def keyed_attention(h, P, m, eps):
    """Values are the projected keys; queries and keys rotated in pairs, then divided by their root mean square; a window;
    the heads gated entry by entry."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    rot, pos = m.get("rot") or {}, torch.arange(h.shape[0])
    q, v = (h @ P["q"].T).view(T, H, d), (h @ P["k"].T).view(T, G, d)
    q, k = (rms(rotate_pairs(x, pos, int(rot.get("dims", 0)), float(rot.get("base", 1.0))), eps) for x in (q, v))
    o = softmax_attention(q, k, v, float(m["scale"]), visible(T, int((m.get("mask") or {}).get("size") or 0)))
    return (o * torch.sigmoid(h @ P["g"].T)) @ P["o"].T


def dense_ff(h, P):
    return (torch.relu(h @ P["gate"].T) * (h @ P["up"].T)) @ P["down"].T


def expert(h, P, pre):
    return (torch.relu(h @ P[pre + "up"].T) ** 2) @ P[pre + "down"].T


def routed_ff(h, P, mlp):
    """Sigmoid scores, the best `top` experts, each run on the token's input times its own score; the shared expert on the
    input itself."""
    s = torch.sigmoid(h @ P["router"].T)
    best = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :int(mlp["router"]["top"])]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in best[t].tolist():
            out[t] += expert(s[t, e] * h[t:t + 1], P, "e%d." % e)[0]
    if mlp.get("shared"):
        out = out + expert(h, P, "shared.")
    return out


def enter_pass(x, x0, w):
    return torch.cat([x, x0], -1) @ w.T


def run_order(cfg):
    """[(layer, starts a pass)]."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, False) for i in range(a)] + [(i, i == a) for _ in range(loop["times"]) for i in range(a, b)] + [(i, False) for i in range(b, n)]


def sub(tensors, prefix):
    return {k[len(prefix):]: v.to(F64) for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens):
    """-> (logits [T, vocab], [the stream after every layer run])."""
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    get = lambda n: tensors[n].to(F64)
    x0 = embedding(cfg, tensors, tokens)
    x, after = x0, []
    for i, opens in run_order(cfg):
        layer, pre = cfg["layers"][i], "l%d." % i
        if opens:
            x = enter_pass(x, x0, get("loop.in"))
        mixer = {"attention": full_attention, "attention_2": keyed_attention}[layer["type"]]
        y = mixer(rms(x, eps, get(pre + "norm1")), sub(tensors, pre + "mix."), layer["mixer"], eps)
        x = x + m * rms(y, eps, get(pre + "norm1b"))
        mlp = layer.get("mlp")
        if mlp is not None:
            h, P = rms(x, eps, get(pre + "norm2")), sub(tensors, pre + "mlp.")
            y = dense_ff(h, P) if mlp.get("kind", "dense") == "dense" else routed_ff(h, P, mlp)
            x = x + m * rms(y, eps, get(pre + "norm2b"))
        after.append(x)
    return rms(x, eps, get("final.norm")) @ get("head").T, after
