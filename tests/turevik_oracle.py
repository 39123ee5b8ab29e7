"""Plain, slow Turevik forward pass: one function per mechanism, written from
the design's equations with nothing shared with the framework's model code.

Everything runs on whole sequences (loops over tokens, heads and experts), in
one floating dtype, without any cache: a test feeds a prompt and compares the
framework's cached / batched / chunked results against it.

``cfg`` is the checkpoint's config.json as a dict; ``sd`` maps tensor names
to tensors.
"""
from __future__ import annotations

import math

import torch


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    """RMS norm whose stored weight is the difference from one."""
    return rms_unit(x, eps) * (1.0 + w)


def norm_plain(x, w, eps):
    return rms_unit(x, eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (x + 0.044715 * x * x * x)))


def token_shift(h, mu):
    """h [T, W] moved towards the previous token's h, element by element;
    the token before the first one counts as zero."""
    out = h.clone()
    for t in range(h.shape[0]):
        before = h[t - 1] if t else torch.zeros_like(h[0])
        out[t] = h[t] + (before - h[t]) * mu
    return out


def turn_pairs(x, pos, base, dims):
    """x [..., d] at integer position pos: entries (2i, 2i+1), i < dims/2,
    turn by pos * base^(-2i/dims); the rest pass through."""
    out = x.clone()
    for i in range(dims // 2):
        a = pos * (base ** (-2.0 * i / dims))
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_rows(h, p, m, eps):
    """What a layer with its own down-projection shares: the normed latent
    [T, R] and the rotated key part [T, rd]."""
    R, rd = m["kv_rank"], m["rot_dim"]
    z = h @ p["dkv"].T
    c = norm_plain(z[:, :R], p["dkv.norm"], eps)
    kr = torch.stack([turn_pairs(z[t, R:R + rd], t, float(m["rot"]["base"]),
                                 int(m["rot"]["dims"]))
                      for t in range(h.shape[0])])
    return c, kr


def sink_softmax(s, sink):
    """Softmax weights of the scores s [n] with exp(sink) in the
    denominator."""
    top = torch.maximum(s.max(), sink)
    e = torch.exp(s - top)
    return e / (e.sum() + torch.exp(sink - top))


def latent_attention(h, p, m, eps, shared=None):
    """h [T, W]; ``shared`` = (latent, rotated key part) of another layer, or
    None when the layer computes its own."""
    T = h.shape[0]
    H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = latent_rows(h, p, m, eps) if shared is None else shared
    q = (h @ p["q"].T).view(T, H, d + rd)
    k = (c @ p["uk"].T).view(T, H, d)
    v = (c @ p["uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        qr = turn_pairs(q[i, :, d:], i, float(m["rot"]["base"]),
                        int(m["rot"]["dims"]))
        for hh in range(H):
            s = (k[:i + 1, hh] @ q[i, hh, :d] + kr[:i + 1] @ qr[hh]) \
                * float(m["scale"])
            out[i, hh] = sink_softmax(s, p["sink"][hh]) @ v[:i + 1, hh]
    return out.reshape(T, H * dv) @ p["o"].T


def mingru(h, p, m, eps):
    """S_t = (1 - z_t) S_(t-1) + z_t c_t per channel; no state feedback into
    z and c."""
    z = sigmoid(h @ p["z"].T + p["z.b"])
    u = h @ p["x"].T + p["x.b"]
    cand = torch.where(u >= 0, u + 0.5, sigmoid(u))
    S = torch.zeros(m["width"], dtype=h.dtype)
    states = []
    for t in range(h.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        states.append(S)
    return (torch.stack(states) * silu(h @ p["g"].T)) @ p["o"].T


def gated_ff(x, p, pre, act):
    return (act(x @ p[pre + "gate"].T) * (x @ p[pre + "up"].T)) \
        @ p[pre + "down"].T


def moe(h, p, ff):
    """Sigmoid scores, the largest ``top`` kept as they are, each chosen
    expert reading its score times the input; a gated shared expert."""
    E, top = ff["router"]["experts"], ff["router"]["top"]
    s = sigmoid(h @ p["router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        order = sorted(range(E), key=lambda e: -float(s[t, e]))[:top]
        for e in order:
            out[t] = out[t] + gated_ff(h[t] * s[t, e], p, f"e{e}.", silu)
    if ff.get("shared"):
        out = out + sigmoid(h @ p["shared.sg"].T) * gated_ff(h, p, "shared.",
                                                            silu)
    return out


def feed_forward(h, p, ff):
    if ff["kind"] == "dense":
        return gated_ff(h, p, "", gelu_tanh)
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
    rows = {}                     # layer -> its (latent, rotated key part)
    for i, spec in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", spec["mixer"]
        p = sub(sd, pre + "mix.")
        h = token_shift(norm_around_one(x, sd[pre + "norm1"], eps),
                        sd[pre + "shift"])
        if spec["type"] == "mingru":
            y = mingru(h, p, m, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                rows[i] = latent_rows(h, p, m, eps)
                src = i
            y = latent_attention(h, p, m, eps, rows[src])
        x = x + norm_around_one(y, sd[pre + "norm1b"], eps)
        if spec.get("mlp") is not None:
            y = feed_forward(norm_around_one(x, sd[pre + "norm2"], eps),
                             sub(sd, pre + "mlp."), spec["mlp"])
            x = x + norm_around_one(y, sd[pre + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_around_one(x, sd["final.norm"], eps) @ sd["embed"].T


def make_checkpoint(cfg, seed=0, dtype=torch.bfloat16, out_gain=1.0):
    """Random tensors for a config.json dict, under the checkpoint's names;
    values are rounded to ``dtype`` (so a bfloat16 and a float32 run read the
    same numbers). ``out_gain`` scales what the sublayers add to the
    residual."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rn(*shape, std=1.0):
        return (torch.randn(*shape, generator=g) * std).to(dtype)

    def lin(out, inp, gain=1.0):
        return rn(out, inp, std=gain * inp ** -0.5)

    sd = {"embed": rn(V, W), "final.norm": rn(W, std=0.2)}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        for n in ("norm1", "norm2"):
            sd[p + n] = rn(W, std=0.2)
        for n in ("norm1b", "norm2b"):
            sd[p + n] = ((1.0 + rn(W, std=0.2).float()) * out_gain
                         - 1.0).to(dtype)
        sd[p + "shift"] = torch.rand(W, generator=g).to(dtype)
        if spec["type"] == "mingru":
            D = m["width"]
            sd.update({p + "mix.z": lin(D, W), p + "mix.z.b": rn(D) - 1.0,
                       p + "mix.x": lin(D, W), p + "mix.x.b": rn(D, std=0.5),
                       p + "mix.g": lin(D, W), p + "mix.o": lin(W, D)})
            sd[p + "mix.z.b"] = sd[p + "mix.z.b"].to(dtype)
        else:
            H, d, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            R = m["kv_rank"]
            sd[p + "mix.q"] = lin(H * (d + rd), W, 1.5)
            if m.get("kv_from") is None:
                sd[p + "mix.dkv"] = lin(R + rd, W)
                sd[p + "mix.dkv.norm"] = (1 + rn(R, std=0.2).float()).to(dtype)
            sd.update({p + "mix.uk": lin(H * d, R, 1.5),
                       p + "mix.uv": lin(H * dv, R),
                       p + "mix.sink": rn(H), p + "mix.o": lin(W, H * dv)})
        ff = spec.get("mlp")
        if ff is None:
            del sd[p + "norm2"], sd[p + "norm2b"]
        elif ff["kind"] == "dense":
            sd.update({p + "mlp.gate": lin(ff["ff"], W),
                       p + "mlp.up": lin(ff["ff"], W),
                       p + "mlp.down": lin(W, ff["ff"])})
        else:
            parts = [(f"e{e}", ff["expert"]["ff"])
                     for e in range(ff["router"]["experts"])]
            sd[p + "mlp.router"] = lin(ff["router"]["experts"], W, 2.0)
            if ff.get("shared"):
                parts.append(("shared", ff["shared"]["ff"]))
                sd[p + "mlp.shared.sg"] = lin(1, W)
            for n, I in parts:
                sd.update({p + f"mlp.{n}.gate": lin(I, W, 1.5),
                           p + f"mlp.{n}.up": lin(I, W),
                           p + f"mlp.{n}.down": lin(W, I)})
    return sd
