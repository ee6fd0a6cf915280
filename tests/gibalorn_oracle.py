"""Plain, slow statement of the Gibalorn design in float64, one function per mechanism, sharing no code with gbx_lm_amd.  A whole
sequence at a time, token after token where the design recurs, query after query where it attends: no cache, no batching, no
chunked scan, no absorbed or fused products, no folded weights.

Notation.  Stream x [T, W]; ``unit(v) = v / sqrt(mean(v^2) + eps)``.  A layer: x += mixer(unit(x) * w1), then (unless it has no
feed-forward) x += ff(unit(x) * w2).  A span of layers may run several times; in front of every pass but the first the embedding rows
are added to x.  logits = head . (unit(x) * w_final).
Also here: config builders and a random checkpoint writer (config.json + model.safetensors in the design's tensor names), so that
tests go through the framework's own loader.
"""
import json
import math
import os

import torch

F64 = torch.float64


def unit(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


# ------------------------------------------------------------------------------------------------ rotations
def rotate(x, dims, base, interleaved):
    """x [T, heads, d], row t at position t: the first ``dims`` channels turn in pairs -- (2i, 2i + 1) or (i, i + dims / 2) -- by
    t * base^(-2i / dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = torch.arange(x.shape[0], dtype=F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        i0, i1 = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        u, v = x[:, :, i0], x[:, :, i1]
        out[:, :, i0], out[:, :, i1] = u * c - v * s, v * c + u * s
    return out


# ------------------------------------------------------------------------------------------------ softmax attention
def causal_attention(q, k, v, scale, sink):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; position i sees every j <= i; ``sink``: one more term exp(0) in the denominator."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for i in range(T):
        for h in range(H):
            s = (k[:i + 1, h // rep] @ q[i, h]) * scale
            top = torch.clamp(s.max(), min=0.0) if sink else s.max()
            e = torch.exp(s - top)
            out[i, h] = (e / (e.sum() + (torch.exp(-top) if sink else 0.0))) @ v[:i + 1, h // rep]
    return out


def latent_mixer(h, w, p, m, eps):
    """Queries, keys and values of all heads grow from two small normed rows per token; one rotated key part is shared by all heads."""
    T, H, d, r, dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).view(T, H, d + r)
    down = h @ w[p + "dkv"].T
    c = unit(down[:, :rank], eps) * w[p + "dkv.norm"]
    base = m["rot"]["base"]
    qr = rotate(q[:, :, d:], r, base, True)
    kr = rotate(down[:, rank:].view(T, 1, r), r, base, True)
    kn = (c @ w[p + "uk"].T).view(T, H, d)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    o = causal_attention(torch.cat([q[:, :, :d], qr], -1), torch.cat([kn, kr.expand(T, H, r)], -1), v, m["scale"], False)
    return (o.reshape(T, H * dv) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def attention_mixer(h, w, p, m, eps):
    """The values are the key projections before they are rotated."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    k = (h @ w[p + "k"].T).view(T, G, d)
    rot = m["rot"]
    q = rotate((h @ w[p + "q"].T).view(T, H, d), rot["dims"], rot["base"], False)
    o = causal_attention(q, rotate(k, rot["dims"], rot["base"], False), k, m["scale"], True)
    return o.reshape(T, H * d) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ state space mixer (mamba2)
def causal_conv(x, taps, bias):
    """x [T, C], taps [C, n] (the last one meets the current token), bias [C]."""
    n = taps.shape[1]
    out = bias[None, :].repeat(x.shape[0], 1)
    for t in range(x.shape[0]):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * x[s]
    return out


def state_space_recurrence(x, B, C, dt, A, D):
    """x [T, H, dv], B, C [T, G, N], dt [T, H] (after softplus), A, D [H] ->  S <- exp(-A dt) S + dt B x^T,  y = S^T C + D x."""
    T, H, dv = x.shape
    rep = H // B.shape[1]
    S = torch.zeros((H, B.shape[2], dv), dtype=F64)
    out = []
    for t in range(T):
        b, c = B[t].repeat_interleave(rep, 0), C[t].repeat_interleave(rep, 0)
        S = torch.exp(-A * dt[t])[:, None, None] * S + dt[t][:, None, None] * b[:, :, None] * x[t][:, None, :]
        out.append((S * c[:, :, None]).sum(1) + D[:, None] * x[t])
    return torch.stack(out)


def mamba2_mixer(h, w, p, m, eps):
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    y = h @ w[p + "in"].T
    z, xbc, dt = y[:, :inner], y[:, inner:2 * inner + 2 * G * N], y[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc[:, :inner].view(T, H, dv), xbc[:, inner:inner + G * N].view(T, G, N), xbc[:, inner + G * N:].view(T, G, N)
    o = state_space_recurrence(x, B, C, softplus(dt + w[p + "dt_bias"]), torch.exp(w[p + "A_log"]), w[p + "D"]).reshape(T, inner)
    y = o * silu(z)                                                      # the gate comes in front of the norm
    return (unit(y.view(T, m["norm_groups"], -1), eps).reshape(T, inner) * w[p + "norm"]) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def expert(h, up, down):
    return torch.clamp(h @ up.T, min=0.0).pow(2) @ down.T


def route(logits, top):
    """One token's logits [E] -> [(expert, weight)]: the ``top`` largest sigmoids (ties: the lower index), as they are."""
    s = sigmoid(logits)
    return [(e, s[e]) for e in sorted(range(logits.shape[0]), key=lambda e: (-float(s[e]), e))[:top]]


def moe_ff(h, w, p, spec):
    """An expert reads its token scaled by the token's weight for it; the outputs are added as they are."""
    logits = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in route(logits[t], spec["router"]["top"]):
            out[t] += expert(s * h[t:t + 1], w[p + f"e{e}.up"], w[p + f"e{e}.down"])[0]
    return out


# ------------------------------------------------------------------------------------------------ the model
MIXERS = {"latent_attention": latent_mixer, "attention": attention_mixer, "mamba2": mamba2_mixer}


def runs_of(cfg):
    """[(layer, the embedding is added in front of this run)] in running order."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(lp["start"])]
    for k in range(lp["times"]):
        out += [(i, k > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return out + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg, weights, tokens):
    """-> (logits [T, vocab], stream after every layer run [runs, T, W]), float64."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    e = w["embed"][list(tokens)]
    x = e.clone()
    after = []
    for i, again in runs_of(cfg):
        if again:
            x = x + e
        p, layer = f"l{i}.", cfg["layers"][i]
        x = x + MIXERS[layer["type"]](unit(x, eps) * w[p + "norm1"], w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + moe_ff(unit(x, eps) * w[p + "norm2"], w, p + "mlp.", layer["mlp"])
        after.append(x.clone())
    return (unit(x, eps) * w["final.norm"]) @ w["head"].T, torch.stack(after)


# ------------------------------------------------------------------------------------------------ configurations and checkpoints
def latent_layer(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=10000.0, scale=None, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                                                  "rot": {"base": base, "dims": rot_dim},
                                                  "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}, "mlp": mlp}


def attention_layer(heads, kv_heads, dim, rot_dims, base=10000.0, scale=None, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": rot_dims},
                                           "scale": scale if scale is not None else dim ** -0.5}, "mlp": mlp}


def mamba2_layer(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups},
            "mlp": mlp}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def make_config(layers, vocab=61, width=64, eps=1e-5, loop=None):
    return {"architecture": "Gibalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "loop": None if loop is None else {"start": loop[0], "stop": loop[1], "times": loop[2]}}


def make_weights(cfg, seed=0, steady=False):
    """``steady``: output projections are halved, so that a row's rounding is not amplified run after run."""
    gen = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    bf = torch.bfloat16

    def mat(o, i, scale=1.0):
        return (torch.randn((o, i), generator=gen) * scale / math.sqrt(i)).to(bf)

    def vec(n, lo, hi):
        return (torch.rand((n,), generator=gen) * (hi - lo) + lo).to(bf)

    w = {"embed": torch.randn((cfg["vocab"], W), generator=gen).to(bf), "final.norm": vec(W, 0.5, 1.5), "head": mat(cfg["vocab"], W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, kind = f"l{i}.", layer["mixer"], layer["type"]
        w[p + "norm1"] = vec(W, 0.5, 1.5)
        x = p + "mix."
        H, dv = m["heads"], m["vdim"]
        if kind == "latent_attention":
            d, r, rank, qr = m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
            w[x + "dq"], w[x + "dq.norm"], w[x + "uq"] = mat(qr, W), vec(qr, 0.5, 1.5), mat(H * (d + r), qr)
            w[x + "dkv"], w[x + "dkv.norm"] = mat(rank + r, W), vec(rank, 0.5, 1.5)
            w[x + "uk"], w[x + "uv"], w[x + "g"], w[x + "o"] = mat(H * d, rank), mat(H * dv, rank), mat(H * dv, W), mat(W, H * dv)
        elif kind == "mamba2":
            inner, gn = H * dv, m["groups"] * m["state"]
            w[x + "in"] = mat(2 * inner + 2 * gn + H, W)
            w[x + "conv"] = (torch.randn((inner + 2 * gn, m["conv"]), generator=gen) * 0.6 + 0.25).to(bf)
            w[x + "conv.b"] = vec(inner + 2 * gn, -0.2, 0.2)
            w[x + "dt_bias"], w[x + "A_log"], w[x + "D"] = vec(H, -4.0, 0.5), vec(H, -2.0, 1.5), vec(H, -1.0, 1.0)
            w[x + "norm"], w[x + "o"] = vec(inner, 0.5, 1.5), mat(W, inner)
        else:
            w[x + "q"], w[x + "k"], w[x + "o"] = mat(H * m["dim"], W), mat(m["kv_heads"] * m["dim"], W), mat(W, H * dv)
        if steady:
            w[x + "o"] = 0.5 * w[x + "o"]
        ff = layer.get("mlp")
        if ff is not None:
            w[p + "norm2"] = vec(W, 0.5, 1.5)
            f, n, E = p + "mlp.", ff["expert"]["ff"], ff["router"]["experts"]
            w[f + "router"] = mat(E, W, 1.5)
            for e in range(E):
                w[f + f"e{e}.up"], w[f + f"e{e}.down"] = mat(n, W, 1.5), mat(W, n, 0.5 if steady else 1.0)
    return w


def save_checkpoint(folder, cfg, weights):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def row_errors(got, want):
    """Root mean square of the difference over that of the reference, per row."""
    got, want = got.to(F64).cpu(), want.to(F64).cpu()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-12)


def rel_err(got, want):
    """The worst row's error."""
    return float(row_errors(got, want).max())


def rel_err_most(got, want, share=0.9):
    """The error that ``share`` of the rows stay under."""
    e = row_errors(got, want).flatten().sort().values
    return float(e[min(int(math.ceil(share * e.numel())) - 1, e.numel() - 1)])
