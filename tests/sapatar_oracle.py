"""Plain float64 implementation of the Sapatar design, written from its
equations: whole sequences, no cache, no state pool, no batching. One
function per mechanism; the engine is compared with these in
tests/test_sapatar.py and tests/test_sapatar_gpu.py. Nothing here imports
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


def log_sigmoid(z):
    return -(torch.clamp(-z, min=0) + torch.log1p(torch.exp(-z.abs())))


# ---- the residual streams -------------------------------------------------------

def stream_in(xs, a):
    """xs [S, T, W], a [S]: the sublayer reads sum_s a_s x_s."""
    return sum(f64(a)[s] * xs[s] for s in range(xs.shape[0]))


def stream_out(xs, mix, b, y):
    """New streams, all from the old ones: x_t = sum_s mix[s, t] x_s + b_t y."""
    S = xs.shape[0]
    mix, b = f64(mix), f64(b)
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(S)) + b[t] * y
                        for t in range(S)])


# ---- positions ------------------------------------------------------------------

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


def heads_of(x, n):
    """[T, n * d] -> [n, T, d]."""
    return x.view(x.shape[0], n, -1).transpose(0, 1)


# ---- wkv: per-channel decay, bonus for the current token --------------------------

def previous_rows(h):
    """The row before each row (zeros before the first)."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)


def shifted(h, mu):
    return h + (previous_rows(h) - h) * f64(mu)


def wkv_recurrence(r, k, v, decay, u):
    """One head: r, k, decay [T, D], v [T, P], u [D]. A token sees the state
    its predecessors left plus its own k v^T weighted by u."""
    T, D = k.shape
    S = torch.zeros(D, v.shape[1], dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        kv = k[t][:, None] * v[t][None, :]
        out[t] = (S + f64(u)[:, None] * kv).t() @ r[t]
        S = decay[t][:, None] * S + kv
    return out


def wkv_decay(mix_w, w1, w2, w0):
    return torch.exp(-torch.exp(torch.tanh(mix_w @ f64(w1).t()) @ f64(w2).t()
                                + f64(w0)))


def wkv_mixer(h, m, w, p, eps):
    H = int(m["heads"])
    W = lambda n: f64(w[p + n])
    r, k, v, g = (shifted(h, w[p + "mu." + n]) @ W(n).t() for n in "rkvg")
    decay = wkv_decay(shifted(h, w[p + "mu.w"]), w[p + "w1"], w[p + "w2"],
                      w[p + "w0"])
    o = [rms_unit(wkv_recurrence(*t, W("u")[a]), eps) for a, t in enumerate(
        zip(*(heads_of(x, H) for x in (r, k, v, decay))))]
    return (torch.cat(o, -1) * W("norm") * silu(g)) @ W("o").t()


# ---- retention: one constant decay per head -----------------------------------------

def retention_recurrence(q, k, v, decay):
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64)
    out = torch.zeros(k.shape[0], v.shape[1], dtype=F64)
    for t in range(k.shape[0]):
        S = decay * S + k[t][:, None] * v[t][None, :]
        out[t] = S.t() @ q[t]
    return out


def retention_mixer(h, m, w, p, eps):
    H, D = int(m["heads"]), int(m["dim"])
    rot = (float(m["rot"]["base"]), int(m["rot"]["dims"]))
    q, k, v, g = (h @ f64(w[p + n]).t() for n in "qkvg")
    q = rotate(heads_of(q, H), *rot)
    k = rotate(heads_of(k, H), *rot) * D ** -0.5
    v = heads_of(v, H)
    o = [rms_unit(retention_recurrence(q[a], k[a], v[a], float(m["decay"][a])),
                  eps) for a in range(H)]
    return (torch.cat(o, -1) * silu(g)) @ f64(w[p + "o"]).t()


# ---- parallel, left: windowed softmax attention -----------------------------------

def sees(i, j, window):
    return 0 <= i - j < window


def attend(q, k, v, scale, window, misplaced=0):
    """One head: q, k [T, D], v [T, VD]. misplaced: a planted mistake, a
    window that many positions too long."""
    T = q.shape[0]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    mask = (j <= i) & (i - j < window + misplaced)
    if T <= 8 and not misplaced:      # the table above is `sees`, element by element
        assert all(bool(mask[a, b]) == sees(a, b, window)
                   for a in range(T) for b in range(T))
    s = ((q @ k.t()) * scale).masked_fill(~mask, -float("inf"))
    return torch.softmax(s, -1) @ v


def attention_half(h, m, w, p):
    H, G = int(m["heads"]), int(m["kv_heads"])
    q, k, v = (h @ f64(w[p + n]).t() + f64(w[p + n + ".b"]) for n in "qkv")
    rot = (float(m["rot"]["base"]), int(m["rot"]["dims"]))
    q, k = rotate(heads_of(q, H), *rot), rotate(heads_of(k, G), *rot)
    v, rep = heads_of(v, G), H // G
    o = [attend(q[a], k[a // rep], v[a // rep], float(m["scale"]),
                int(m["mask"]["size"]), int(m["mask"].get("misplaced", 0)))
         for a in range(H)]
    return torch.cat(o, -1) @ f64(w[p + "o"]).t()


# ---- parallel, right: matrix memory with exponential gates ------------------------

def capped(z, cap):
    return cap * torch.tanh(z / cap)


def mlstm_recurrence(q, k, v, i, f, floor=True):
    """One head: q, k [T, D], v [T, P]; i, f [T] log gates. The running
    maximum m starts at 0. floor False: a planted mistake, no lower bound
    under the denominator."""
    T, D = k.shape
    S = torch.zeros(D, v.shape[1], dtype=F64)
    n = torch.zeros(D, dtype=F64)
    m = torch.zeros((), dtype=F64)
    out = torch.zeros(T, v.shape[1], dtype=F64)
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        a, b = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = a * S + b * k[t][:, None] * v[t][None, :]
        n = a * n + b * k[t]
        m = new
        den = (n @ q[t]).abs()
        if floor:
            den = torch.maximum(den, torch.exp(-m))
        den = den + 1e-6
        out[t] = (S.t() @ q[t]) / den
    return out


def mlstm_half(h, m, w, p, eps):
    H, D, cap = int(m["heads"]), int(m["dim"]), float(m["gate_cap"])
    W = lambda n: f64(w[p + n])
    q, k, v, g = (h @ W(n).t() for n in "qkvg")
    i = capped(h @ W("i").t() + W("i.b"), cap)                   # [T, H]
    f = log_sigmoid(capped(h @ W("f").t() + W("f.b"), cap))
    q = heads_of(q * D ** -0.5, H)
    k, v = heads_of(k, H), heads_of(v, H)
    o = [rms_unit(mlstm_recurrence(q[a], k[a], v[a], i[:, a], f[:, a],
                                  not m.get("no_floor")), eps)
         for a in range(H)]
    return (torch.cat(o, -1) * W("norm") * torch.sigmoid(g)) @ W("o").t()


def parallel_mixer(h, m, w, p, eps):
    return (float(m["left_scale"]) * attention_half(h, m["left"], w, p + "left.")
            + float(m["right_scale"])
            * mlstm_half(h, m["right"], w, p + "right.", eps))


# ---- feed-forward -----------------------------------------------------------------

def gated_ff(h, w, p):
    return (silu(h @ f64(w[p + "gate"]).t())
            * (h @ f64(w[p + "up"]).t())) @ f64(w[p + "down"]).t()


def route(h, w, p, top):
    """Chosen experts [T, top] and their weights: softmax over the chosen
    logits only."""
    z = h @ f64(w[p + "router"]).t() + f64(w[p + "router.b"])
    val, idx = torch.topk(z, top, -1)
    return idx, torch.softmax(val, -1)


def moe_ff(h, f, w, p):
    idx, wt = route(h, w, p, int(f["router"]["top"]))
    y = torch.zeros_like(h)
    for e in range(int(f["router"]["experts"])):
        share = (wt * (idx == e)).sum(-1)
        rows = share.nonzero()[:, 0]
        if rows.numel():
            y[rows] += share[rows, None] * gated_ff(h[rows], w, p + f"e{e}.")
    gate = torch.sigmoid(h @ f64(w[p + "shared.sg"]).t())        # [T, 1]
    return y + gate * gated_ff(h, w, p + "shared.")


# ---- the model ------------------------------------------------------------------

def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = int(cfg["layers"][i]["weights_of"])
    return i


def mix(h, ent, w, p, eps):
    fn = {"wkv": wkv_mixer, "retention": retention_mixer,
          "parallel": parallel_mixer}[ent["type"]]
    return fn(h, ent["mixer"], w, p + "mix.", eps)


def forward(cfg, w, tokens, return_layers=False):
    """Logits [T, vocab] of one sequence (and the sum of the streams after
    every layer)."""
    eps = float(cfg["norm"]["eps"])
    e = f64(w["embed"])[torch.as_tensor(tokens)]
    xs = torch.stack([e] * int(cfg["streams"]))
    sums = []
    for i, ent in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."
        h = rms_norm(stream_in(xs, w[p + "hc1.in"]), w[p + "norm1"], eps)
        xs = stream_out(xs, w[p + "hc1.mix"], w[p + "hc1.out"],
                        mix(h, ent, w, p, eps))
        if ent.get("mlp"):
            h = rms_norm(stream_in(xs, w[p + "hc2.in"]), w[p + "norm2"], eps)
            xs = stream_out(xs, w[p + "hc2.mix"], w[p + "hc2.out"],
                            moe_ff(h, ent["mlp"], w, p + "mlp."))
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

def moe(experts=5, top=2, ff=10, shared=14):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top},
            "shared": {"ff": shared}}


def retention_layer(heads=3, dim=8, vdim=6, rot_dims=6, base=100.0,
                    decay=None, mlp="moe"):
    if decay is None:
        decay = [1.0 - 2.0 ** -(2 + 2 * a) for a in range(heads)]
    return {"type": "retention",
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "rot": {"dims": rot_dims, "base": base},
                      "decay": decay},
            "mlp": moe() if mlp == "moe" else mlp}


def parallel_layer(heads=4, kv_heads=2, dim=6, vdim=5, size=9, scale=0.45,
                   rot_dims=4, base=300.0, r_heads=2, r_dim=5, r_vdim=7,
                   cap=4.0, left_scale=0.8, right_scale=1.3, mlp="moe"):
    return {"type": "parallel",
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads,
                               "dim": dim, "vdim": vdim, "scale": scale,
                               "mask": {"size": size},
                               "rot": {"dims": rot_dims, "base": base}},
                      "left_scale": left_scale,
                      "right": {"heads": r_heads, "dim": r_dim,
                                "vdim": r_vdim, "gate_cap": cap},
                      "right_scale": right_scale},
            "mlp": moe() if mlp == "moe" else mlp}


def wkv_layer(heads=2, dim=7, mlp="moe"):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim},
            "mlp": moe() if mlp == "moe" else mlp}


def again(layers, j):
    """The entry of a layer that uses layer j's weights."""
    import copy

    ent = copy.deepcopy(layers[j])
    ent["weights_of"] = j
    return ent


def make_config(width=22, vocab=50, streams=3, layers=None, eps=1e-5):
    if layers is None:
        layers = [parallel_layer(), wkv_layer(mlp=moe(4, 1, 12, 6)),
                  retention_layer(), wkv_layer(heads=3, dim=4, mlp=None)]
        layers += [again(layers, 0), again(layers, 2), again(layers, 1)]
    return {"architecture": "Sapatar", "vocab": vocab, "width": width,
            "streams": streams, "norm": {"eps": eps}, "layers": layers}


def make_weights(cfg, seed=0, rank=3):
    """Random bf16 checkpoint of a configuration (norm weights, shifts,
    gates and mixing matrices spread enough to matter; streams that keep
    their size over many layers; router logits far apart)."""
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
                        + 0.2 * torch.randn(S, S, generator=g)
                        ).to(torch.bfloat16)

    def ff(p, n):
        lin(p + "gate", n, W, 1.5)
        lin(p + "up", n, W)
        lin(p + "down", W, n)

    w["embed"] = torch.randn(cfg["vocab"], W, generator=g).to(torch.bfloat16)
    vec("final.norm", W)
    lin("head", cfg["vocab"], W)
    for i, ent in enumerate(cfg["layers"]):
        if ent.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", ent["mixer"]
        vec(p + "norm1", W)
        hyper(p + "hc1.")
        p += "mix."
        if ent["type"] == "wkv":
            n = m["heads"] * m["dim"]
            for nm in "rkvgw":
                vec(p + "mu." + nm, W, 0.4, 0.5)
            for nm in "rkvg":
                lin(p + nm, n, W, 1.3)
            lin(p + "w1", rank, W, 1.5)
            lin(p + "w2", n, rank, 1.0)
            vec(p + "w0", n, -1.5, 1.0)
            vec(p + "u", n, 0.6, 0.6)
            w[p + "u"] = w[p + "u"].view(m["heads"], m["dim"])
            vec(p + "norm", n)
            lin(p + "o", W, n)
        elif ent["type"] == "retention":
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for nm, rows in (("q", nk), ("k", nk), ("v", nv), ("g", nv)):
                lin(p + nm, rows, W, 1.5)
            lin(p + "o", W, nv)
        else:
            L, R = m["left"], m["right"]
            H, G = L["heads"], L["kv_heads"]
            for nm, rows in (("q", H * L["dim"]), ("k", G * L["dim"]),
                             ("v", G * L["vdim"])):
                lin(p + "left." + nm, rows, W, 1.5)
                vec(p + f"left.{nm}.b", rows, 0.0, 0.4)
            lin(p + "left.o", W, H * L["vdim"])
            H = R["heads"]
            nk, nv = H * R["dim"], H * R["vdim"]
            for nm, rows in (("q", nk), ("k", nk), ("v", nv), ("g", nv)):
                lin(p + "right." + nm, rows, W, 1.5)
            for nm, base in (("i", 0.5), ("f", 2.0)):
                lin(p + "right." + nm, H, W, 2.5)
                vec(p + f"right.{nm}.b", H, base, 1.0)
            vec(p + "right.norm", nv)
            lin(p + "right.o", W, nv)
        f = ent.get("mlp")
        if f:
            p = f"l{i}."
            vec(p + "norm2", W)
            hyper(p + "hc2.")
            E = f["router"]["experts"]
            lin(p + "mlp.router", E, W, 3.0)
            vec(p + "mlp.router.b", E, 0.0, 0.5)
            for e in range(E):
                ff(p + f"mlp.e{e}.", f["expert"]["ff"])
            ff(p + "mlp.shared.", f["shared"]["ff"])
            lin(p + "mlp.shared.sg", 1, W, 1.5)
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
