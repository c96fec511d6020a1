"""Plain float64 implementation of the Fuvuvik design, written from its
equations: whole sequences, no cache, no state pool, no batching. One
function per mechanism; the engine is compared with these in
tests/test_fuvuvik.py and tests/test_fuvuvik_gpu.py. Nothing here imports
the product path.

`cfg` is the dict of a checkpoint's config.json, `w` maps checkpoint tensor
names to tensors (any float dtype; converted to float64 on use).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def f64(t):
    return t.to(F64)


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * f64(w)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


# ---- the residual: streams, gate, token shift -----------------------------------

def stream_in(xs, a):
    """xs [S, T, W], a [S]: the sublayer reads sum_s a_s x_s."""
    return sum(f64(a)[s] * xs[s] for s in range(xs.shape[0]))


def stream_out(xs, mix, b, y):
    """New streams, all from the old ones: x_t = sum_s mix[s, t] x_s + b_t y."""
    S = xs.shape[0]
    mix, b = f64(mix), f64(b)
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(S)) + b[t] * y
                        for t in range(S)])


def token_shift(h, mu):
    """h [T, W]: every row moves the share mu towards the row before it
    (zeros before the first)."""
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)
    return h + (prev - h) * f64(mu)


def residual_gate(h, w, b):
    return torch.sigmoid(h @ f64(w).t() + f64(b))


# ---- attention ------------------------------------------------------------------

def causal_conv(x, w):
    """x [T, C], w [C, taps] (last column = the current token's): zeros
    before the sequence starts; no bias, no activation."""
    T, C = x.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=F64), x], 0)
    acc = torch.zeros(T, C, dtype=F64)
    for k in range(taps):
        acc = acc + pad[k:k + T] * f64(w)[:, k][None, :]
    return acc


def rotate(x, base, dims):
    """x [..., T, D]: of the first `dims` channels, i pairs with i + dims/2
    and the pair turns by t * base^(-2i/dims); angles in 32-bit as the
    design computes them."""
    T, half = x.shape[-2], dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)],
                     dtype=F64).to(torch.float32)
    ang = torch.arange(T, dtype=torch.float32)[:, None] * f[None, :]
    c, s = f64(torch.cos(ang)), f64(torch.sin(ang))
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def sees(i, j, chunk):
    return j <= i and (chunk <= 0 or i // chunk == j // chunk)


def attend(q, k, v, scale, chunk=0, one_in_denominator=False, misplaced=0):
    """One head: q, k [T, D], v [T, VD]. chunk > 0: keys of the query's own
    chunk of positions only. one_in_denominator: exp(0) joins the sum.
    misplaced: a planted mistake, chunk borders that many positions off."""
    T = q.shape[0]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    mask = j <= i
    if chunk > 0:
        mask = mask & ((i + misplaced) // chunk == (j + misplaced) // chunk)
    if T <= 8 and not misplaced:      # the table above is `sees`, element by element
        assert all(bool(mask[a, b]) == sees(a, b, chunk)
                   for a in range(T) for b in range(T))
    s = ((q @ k.t()) * scale).masked_fill(~mask, -float("inf"))
    mx = s.max(-1, keepdim=True)[0]
    if one_in_denominator:
        mx = torch.clamp(mx, min=0.0)
    e = torch.exp(s - mx)
    den = e.sum(-1, keepdim=True)
    if one_in_denominator:
        den = den + torch.exp(-mx)
    return (e / den) @ v


def attention_mixer(h, m, w, p, eps, kind):
    """kind "attention": convolved q, k, v, rotation, then unit RMS per q
    and k head, plain causal softmax. kind "attention_2": rotation, keys of
    the own chunk, one more in the denominator. Both gate every head."""
    T = h.shape[0]
    H, G = int(m["heads"]), int(m["kv_heads"])
    D, VD = int(m["dim"]), int(m["vdim"])
    W = lambda n: f64(w[p + n])
    q, k, v = (h @ W(n).t() for n in "qkv")
    if kind == "attention":
        q, k, v = (causal_conv(x, w[p + n + ".conv"])
                   for x, n in ((q, "q"), (k, "k"), (v, "v")))
    q = q.view(T, H, D).transpose(0, 1)
    k = k.view(T, G, D).transpose(0, 1)
    v = v.view(T, G, VD).transpose(0, 1)
    rot = m["rot"]
    q = rotate(q, float(rot["base"]), int(rot["dims"]))
    k = rotate(k, float(rot["base"]), int(rot["dims"]))
    chunk, one, off = 0, False, 0
    if kind == "attention":
        q, k = rms_unit(q, eps), rms_unit(k, eps)
    else:
        chunk, one = int(m["mask"]["size"]), not m["mask"].get("no_one")
        off = int(m["mask"].get("misplaced", 0))
    gate = torch.sigmoid(h @ W("g").t())                         # [T, H]
    rep = H // G
    outs = [attend(q[a], k[a // rep], v[a // rep], float(m["scale"]), chunk,
                   one, off) * gate[:, a:a + 1] for a in range(H)]
    return torch.cat(outs, -1) @ W("o").t()


# ---- minGRU ---------------------------------------------------------------------

def mingru_recurrence(z, c):
    """z, c [T, N]: S_t = (1 - z_t) S_(t-1) + z_t c_t from zero."""
    S = torch.zeros(z.shape[1], dtype=F64)
    out = torch.zeros_like(z)
    for t in range(z.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * c[t]
        out[t] = S
    return out


def mingru_candidate(u):
    return torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def mingru_mixer(h, w, p):
    W = lambda n: f64(w[p + n])
    z = torch.sigmoid(h @ W("z").t() + W("z.b"))
    u = h @ W("x").t() + W("x.b")
    s = mingru_recurrence(z, mingru_candidate(u))
    return (s * silu(h @ W("g").t())) @ W("o").t()


def dense_ff(h, w, p):
    return (gelu_tanh(h @ f64(w[p + "gate"]).t())
            * (h @ f64(w[p + "up"]).t())) @ f64(w[p + "down"]).t()


# ---- the model ------------------------------------------------------------------

def mix(h, ent, w, p, eps):
    if ent["type"] == "mingru":
        return mingru_mixer(h, w, p + "mix.")
    if ent["type"] in ("attention", "attention_2"):
        return attention_mixer(h, ent["mixer"], w, p + "mix.", eps, ent["type"])
    raise ValueError(ent["type"])


def forward(cfg, w, tokens, return_layers=False):
    """Logits [T, vocab] of one sequence (and the sum of the streams after
    every layer)."""
    eps = float(cfg["norm"]["eps"])
    e = f64(w["embed"])[torch.as_tensor(tokens)] \
        * float(cfg["embedding"]["scale"])
    xs = torch.stack([e] * int(cfg["streams"]))
    sums = []
    for i, ent in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(stream_in(xs, w[p + "hc1.in"]), w[p + "norm1"], eps)
        y = mix(token_shift(h, w[p + "shift"]), ent, w, p, eps)
        y = y * residual_gate(h, w[p + "rg1"], w[p + "rg1.b"])
        xs = stream_out(xs, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        if ent.get("mlp"):
            h = rms_norm(stream_in(xs, w[p + "hc2.in"]), w[p + "norm2"], eps)
            y = dense_ff(h, w, p + "mlp.")
            y = y * residual_gate(h, w[p + "rg2"], w[p + "rg2.b"])
            xs = stream_out(xs, w[p + "hc2.mix"], w[p + "hc2.out"], y)
        sums.append(xs.sum(0))
    logits = rms_norm(xs.sum(0), w["final.norm"], eps) @ f64(w["head"]).t()
    if return_layers:
        return logits, torch.stack(sums)
    return logits


def greedy(cfg, w, prompt, n):
    """n greedy tokens after `prompt`, recomputing the whole sequence."""
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, w, toks)[-1].argmax())
        out.append(nxt)
        toks.append(nxt)
    return out


# ---- small configurations and random checkpoints for the tests ------------------

def attention_layer(heads=4, kv_heads=2, dim=8, vdim=6, conv=4, scale=0.4,
                    rot_dims=6, base=100.0, ff=20):
    return {"type": "attention",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv, "scale": scale,
                      "rot": {"dims": rot_dims, "base": base}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def chunk_layer(heads=3, kv_heads=1, dim=6, vdim=5, size=9, scale=0.5,
                rot_dims=4, base=300.0, ff=14):
    return {"type": "attention_2",
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale, "mask": {"size": size},
                      "rot": {"dims": rot_dims, "base": base}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def mingru_layer(width=18, ff=0):
    return {"type": "mingru", "mixer": {"width": width},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def make_config(width=22, vocab=50, streams=3, layers=None, eps=1e-5,
                embed_scale=0.7):
    if layers is None:
        layers = [chunk_layer(), attention_layer(), mingru_layer(),
                  mingru_layer(width=26, ff=16), chunk_layer(size=5, ff=0)]
    return {"architecture": "Fuvuvik", "vocab": vocab, "width": width,
            "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "layers": layers}


def make_weights(cfg, seed=0):
    """Random bf16 checkpoint of a configuration (norm weights, shifts,
    gates and mixing matrices spread enough to matter)."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg["width"], cfg["streams"]
    w = {}

    def lin(name, out, inp, gain=1.0):
        w[name] = (torch.randn(out, inp, generator=g) * gain * inp ** -0.5
                   ).to(torch.bfloat16)

    def vec(name, n, base=1.0, std=0.2):
        w[name] = (base + std * torch.randn(n, generator=g)).to(torch.bfloat16)

    def hyper(p):
        vec(p + "in", S, 1.0 / S, 0.4)
        vec(p + "out", S, 0.8, 0.4)
        w[p + "mix"] = (torch.eye(S) * 0.7 + 0.3 / S
                        + 0.25 * torch.randn(S, S, generator=g)
                        ).to(torch.bfloat16)

    w["embed"] = torch.randn(cfg["vocab"], W, generator=g).to(torch.bfloat16)
    vec("final.norm", W)
    lin("head", cfg["vocab"], W)
    for i, ent in enumerate(cfg["layers"]):
        p, m = f"l{i}.", ent["mixer"]
        vec(p + "norm1", W)
        vec(p + "shift", W, 0.4, 0.4)
        hyper(p + "hc1.")
        lin(p + "rg1", W, W, 1.5)
        vec(p + "rg1.b", W, 0.3, 0.5)
        if ent["type"] == "mingru":
            n = m["width"]
            for nm in "zx":
                lin(p + "mix." + nm, n, W, 1.5)
                vec(p + f"mix.{nm}.b", n, -0.5, 0.8)
            lin(p + "mix.g", n, W, 1.5)
            lin(p + "mix.o", W, n)
        else:
            H, G, D, VD = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for nm, rows in (("q", H * D), ("k", G * D), ("v", G * VD)):
                lin(p + "mix." + nm, rows, W, 1.5)
                if ent["type"] == "attention":
                    w[p + f"mix.{nm}.conv"] = (
                        torch.randn(rows, m["conv"], generator=g) * 0.6
                    ).to(torch.bfloat16)
            lin(p + "mix.g", H, W, 2.0)
            lin(p + "mix.o", W, H * VD)
        if ent.get("mlp"):
            vec(p + "norm2", W)
            hyper(p + "hc2.")
            lin(p + "rg2", W, W, 1.5)
            vec(p + "rg2.b", W, 0.3, 0.5)
            lin(p + "mlp.gate", ent["mlp"]["ff"], W, 1.5)
            lin(p + "mlp.up", ent["mlp"]["ff"], W)
            lin(p + "mlp.down", W, ent["mlp"]["ff"])
    return w


def save_model(path, cfg, weights):
    import json
    from pathlib import Path

    from safetensors.torch import save_file

    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in weights.items()},
              str(path / "model.safetensors"))
    return str(path)
