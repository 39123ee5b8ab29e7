"""Plain, slow Fedinex forward pass: one function per mechanism, written from
the design's equations with nothing shared with the framework's model code.

Everything runs on whole sequences (loops over tokens, heads and experts), in
one floating dtype, without any cache: a test feeds a prompt and compares the
framework's cached / batched / chunked results against it.

``cfg`` is the checkpoint's config.json as a dict; ``sd`` maps tensor names
to tensors.
"""
from __future__ import annotations

import torch


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms_unit(x, eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def log_sigmoid(x):
    return torch.minimum(x, torch.zeros_like(x)) \
        - torch.log1p(torch.exp(-x.abs()))


def short_conv(u, w):
    """Causal convolution over time per channel: u [T, C], w [C, taps], the
    last tap on the token itself, zeros before the first token."""
    T, taps = u.shape[0], w.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * u[s]
    return out


def turn(x, rot, layout):
    """x [T, heads, d], row t at position t: the first rot.dims entries of a
    head turn in pairs, entry 2i with 2i+1 ("pairs") or i with i + dims/2
    ("halves"); the rest pass through."""
    out = x.clone()
    if not rot:
        return out
    n = int(rot["dims"]) // 2
    pos = torch.arange(x.shape[0], dtype=torch.float64)
    for i in range(n):
        a = pos * float(rot["base"]) ** (-2.0 * i / (2 * n))
        c, s = (f(a).to(x.dtype).view(-1, 1) for f in (torch.cos, torch.sin))
        iu, iv = (2 * i, 2 * i + 1) if layout == "pairs" else (i, i + n)
        u, v = x[..., iu], x[..., iv]
        out[..., iu] = u * c - v * s
        out[..., iv] = v * c + u * s
    return out


def sees(i, j, mask):
    """Is key j visible to the query at position i?"""
    if j > i:
        return False
    if not mask:
        return True
    return i - j < int(mask["size"]) or j < int(mask.get("keep_first") or 0)


def visible(T, mask):
    return torch.tensor([[sees(i, j, mask) for j in range(T)]
                         for i in range(T)])


def attend(q, k, v, scale, mask):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]: softmax over the
    visible keys, query head h on key/value head h // (H / G)."""
    T, H = q.shape[0], q.shape[1]
    per = H // k.shape[1]
    vis = visible(T, mask)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        s = torch.where(vis, s, torch.full_like(s, float("-inf")))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, h // per]
    return out


def biased_attention(h, p, m, v_first=None):
    """Windowed attention with kept first tokens, biased projections, turning
    halves. ``v_first``: values of the stack's first value-mixing layer, or
    None when this layer mixes nothing. Returns (output, own values before
    mixing)."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = turn((h @ p["q"].T + p["q.b"]).view(T, H, d), m.get("rot"), "halves")
    k = turn((h @ p["k"].T + p["k.b"]).view(T, G, d), m.get("rot"), "halves")
    v = (h @ p["v"].T + p["v.b"]).view(T, G, dv)
    own = v
    if v_first is not None:
        lam = p["vmix"]
        v = (1.0 - lam) * v + lam * v_first
    o = attend(q, k, v, float(m["scale"]), m.get("mask"))
    return o.reshape(T, H * dv) @ p["o"].T + p["o.b"], own


def conv_attention(h, p, m):
    """Full causal attention whose q, k, v run through a short convolution,
    turning pairs, one output gate per head."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ p[n].T, p[n + ".conv"]) for n in "qkv")
    q = turn(q.view(T, H, d), m.get("rot"), "pairs")
    k = turn(k.view(T, G, d), m.get("rot"), "pairs")
    o = attend(q, k, v.view(T, G, dv), float(m["scale"]), None)
    o = o * sigmoid(h @ p["g"].T).unsqueeze(-1)
    return o.reshape(T, H * dv) @ p["o"].T


def matrix_memory(q, k, v, i, f):
    """Stabilized matrix memory: q, k [T, H, d], v [T, H, dv], log gates i, f
    [T, H] -> [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    n = torch.zeros(H, d, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = []
    for t in range(T):
        mn = torch.maximum(f[t] + m, i[t])
        keep, put = torch.exp(f[t] + m - mn), torch.exp(i[t] - mn)
        S = keep.view(H, 1, 1) * S + put.view(H, 1, 1) \
            * k[t].unsqueeze(2) * v[t].unsqueeze(1)
        n = keep.view(H, 1) * n + put.view(H, 1) * k[t]
        m = mn
        num = (S * q[t].unsqueeze(2)).sum(1)
        den = torch.maximum((n * q[t]).sum(1).abs(), torch.exp(-m)) + 1e-6
        out.append(num / den.view(H, 1))
    return torch.stack(out)


def mlstm(h, p, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    cap = float(m["gate_cap"])
    q = (h @ p["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ p["k"].T).view(T, H, d)
    v = (h @ p["v"].T).view(T, H, dv)
    i = cap * torch.tanh((h @ p["i"].T + p["i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ p["f"].T + p["f.b"]) / cap))
    o = rms_unit(matrix_memory(q, k, v, i, f), eps).reshape(T, H * dv)
    return (o * p["norm"] * sigmoid(h @ p["g"].T)) @ p["o"].T


def parallel(h, p, m, eps):
    return float(m["left_scale"]) * conv_attention(h, sub(p, "left."),
                                                   m["left"]) \
        + float(m["right_scale"]) * mlstm(h, sub(p, "right."), m["right"],
                                          eps)


def decayed_memory(q, k, v, alpha):
    """S <- diag(alpha) S + k v^T, o = S^T q: q, k, alpha [T, H, d], v
    [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        S = alpha[t].unsqueeze(2) * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(2)).sum(1))
    return torch.stack(out)


def gla(h, p, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ p["k"].T).view(T, H, d)
    v = (h @ p["v"].T).view(T, H, dv)
    z = (h @ p["a1"].T) @ p["a2"].T + p["a2.b"]
    alpha = torch.exp(log_sigmoid(z) / float(m["tau"])).view(T, H, d)
    o = norm(decayed_memory(q, k, v, alpha), p["norm"], eps)
    return (o.reshape(T, H * dv) * silu(h @ p["g"].T)) @ p["o"].T


def clamped_ff(x, p, pre, limit):
    g = torch.clamp(x @ p[pre + "gate"].T, max=limit)
    u = torch.clamp(x @ p[pre + "up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ p[pre + "down"].T


def choose(s, correction, router):
    """Indices of the chosen experts for one token's scores s [E]."""
    E, top = len(s), router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    c = [float(a) for a in s + correction]
    size = E // groups["count"]
    rank = sorted(range(groups["count"]), key=lambda g: -sum(
        sorted(c[g * size:(g + 1) * size])[-2:]))[:groups["keep"]]
    pool = [e for g in rank for e in range(g * size, (g + 1) * size)]
    return sorted(pool, key=lambda e: -c[e])[:top]


def moe(h, p, ff):
    s = sigmoid(h @ p["router"].T)
    limit = float(ff["expert"]["limit"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in choose(s[t], p["correction"], ff["router"]):
            out[t] = out[t] + s[t, e] * float(ff["router"]["scale"]) \
                * clamped_ff(h[t], p, f"e{e}.", limit)
    return out


def feed_forward(h, p, ff):
    if ff["kind"] == "dense":
        return clamped_ff(h, p, "", float(ff["limit"]))
    return moe(h, p, ff)


def sub(sd, prefix):
    n = len(prefix)
    return {k[n:]: v for k, v in sd.items() if k.startswith(prefix)}


def forward(tokens, sd, cfg, dtype=torch.float32, layers_out=None):
    """Logits [T, vocab] of one whole sequence. ``layers_out`` (a list)
    receives the residual after every layer."""
    sd = {k: (v.to(dtype) if v.is_floating_point() else v)
          for k, v in sd.items()}
    eps = float(cfg["norm"]["eps"])
    x = sd["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    v_first = None
    for i, spec in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", spec["mixer"]
        p = sub(sd, pre + "mix.")
        h = norm(x, sd[pre + "norm1"], eps)
        if spec["type"] == "parallel":
            y = parallel(h, p, m, eps)
        elif spec["type"] == "gla":
            y = gla(h, p, m, eps)
        else:
            mixes = bool(m.get("v_mix"))
            y, own = biased_attention(h, p, m, v_first if mixes else None)
            if mixes and v_first is None:
                v_first = own
        x = x + y
        if spec.get("mlp") is not None:
            x = x + feed_forward(norm(x, sd[pre + "norm2"], eps),
                                 sub(sd, pre + "mlp."), spec["mlp"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, sd["final.norm"], eps) @ sd["head"].T


def make_checkpoint(cfg, seed=0, dtype=torch.bfloat16, out_gain=1.0):
    """Random tensors for a config.json dict, under the checkpoint's names;
    values are rounded to ``dtype`` (so a bfloat16 and a float32 run read the
    same numbers). ``out_gain`` scales what the sublayers add to the
    residual."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(dtype)

    def lin(out, inp, gain=1.0):
        return rn(out, inp, std=gain * inp ** -0.5)

    def out(o, inp):
        return lin(o, inp, out_gain)

    sd = {"embed": rn(V, W), "final.norm": rn(W, std=0.2, mean=1.0),
          "head": lin(V, W)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        a = p + "mix."
        sd[p + "norm1"] = rn(W, std=0.2, mean=1.0)
        if spec["type"] == "parallel":
            lf, rt = m["left"], m["right"]
            H, G, d, dv = lf["heads"], lf["kv_heads"], lf["dim"], lf["vdim"]
            for n, c in (("q", H * d), ("k", G * d), ("v", G * dv)):
                sd[a + "left." + n] = lin(c, W, 1.5)
                cw = rn(c, lf["conv"], std=0.4)
                cw[:, -1] += 1.0
                sd[a + f"left.{n}.conv"] = cw
            sd[a + "left.g"] = lin(H, W)
            sd[a + "left.o"] = out(W, H * dv)
            H, d, dv = rt["heads"], rt["dim"], rt["vdim"]
            sd.update({a + "right.q": lin(H * d, W), a + "right.k":
                       lin(H * d, W), a + "right.v": lin(H * dv, W),
                       a + "right.g": lin(H * dv, W),
                       a + "right.o": out(W, H * dv),
                       a + "right.norm": rn(H * dv, std=0.2, mean=1.0),
                       a + "right.i": lin(H, W), a + "right.i.b": rn(H),
                       a + "right.f": lin(H, W),
                       a + "right.f.b": rn(H, mean=2.5)})
        elif spec["type"] == "gla":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            r = max(3, W // 8)
            sd.update({a + "q": lin(H * d, W), a + "k": lin(H * d, W),
                       a + "v": lin(H * dv, W), a + "g": lin(H * dv, W),
                       a + "o": out(W, H * dv),
                       a + "norm": rn(dv, std=0.2, mean=1.0),
                       a + "a1": lin(r, W), a + "a2": lin(H * d, r),
                       a + "a2.b": rn(H * d)})
        else:
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, c in (("q", H * d), ("k", G * d), ("v", G * dv)):
                sd[a + n] = lin(c, W, 1.5)
                sd[a + n + ".b"] = rn(c, std=0.5)
            sd[a + "o"] = out(W, H * dv)
            sd[a + "o.b"] = rn(W, std=0.3 * out_gain)
            if m.get("v_mix"):
                sd[a + "vmix"] = torch.tensor(0.2 + 0.1 * (i % 5)).to(dtype)
        ff = spec.get("mlp")
        if ff is None:
            continue
        sd[p + "norm2"] = rn(W, std=0.2, mean=1.0)
        if ff["kind"] == "dense":
            parts = [("", ff["ff"])]
        else:
            E = ff["router"]["experts"]
            parts = [(f"e{e}.", ff["expert"]["ff"]) for e in range(E)]
            sd[p + "mlp.router"] = lin(E, W)
            sd[p + "mlp.correction"] = rn(E, std=0.3, mean=-0.4)
        for n, I in parts:
            sd.update({p + f"mlp.{n}gate": lin(I, W, 1.5),
                       p + f"mlp.{n}up": lin(I, W, 1.5),
                       p + f"mlp.{n}down": out(W, I)})
    return sd
