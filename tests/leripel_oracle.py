"""Plain, slow statement of the Leripel design in float64, one function per mechanism, sharing no code with gbx_lm_amd.  A whole
sequence at a time, token after token where the design recurs, query after query where it attends: no cache, no batching, no
chunked scan, no fused products.

Notation.  Stream x [T, W]; ``unit(v) = v / sqrt(mean(v^2) + eps)``.  A layer reads ONE norm of the stream, h = unit(x) * w, and adds
both of its sublayers: x += mixer(h) + ff(h).  A span of layers may run several times; before each of its passes
x <- W_in [x ; e], e being the embedding rows.  logits = head . (unit(x) * w_final).
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


# ------------------------------------------------------------------------------------------------ linear attention with a fixed decay
def retention_recurrence(q, k, v, decay):
    """q, k [T, H, dk], v [T, H, dv], decay [H] -> [T, H, dv]:  S <- decay S + k v^T,  o = S^T q."""
    S = torch.zeros((q.shape[1], q.shape[2], v.shape[2]), dtype=F64)
    out = []
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def retention_mixer(h, w, p, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d)
    k = (h @ w[p + "k"].T).view(T, H, d) / math.sqrt(d)
    v = (h @ w[p + "v"].T).view(T, H, dv)
    o = retention_recurrence(q, k, v, torch.tensor(m["decay"], dtype=F64))
    return (unit(o, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


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


def gate_then_group_norm(y, z, weight, groups, eps):
    """The gate comes first, then each of the equal parts is scaled by its own root mean square."""
    y = y * silu(z)
    return unit(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * weight


def mamba2_mixer(h, w, p, m, eps):
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    y = h @ w[p + "in"].T
    z, xbc, dt = y[:, :inner], y[:, inner:2 * inner + 2 * G * N], y[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc[:, :inner].view(T, H, dv), xbc[:, inner:inner + G * N].view(T, G, N), xbc[:, inner + G * N:].view(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    o = state_space_recurrence(x, B, C, dt, torch.exp(w[p + "A_log"]), w[p + "D"]).reshape(T, inner)
    return gate_then_group_norm(o, z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ chunked softmax attention
def rotate_pairs(x, dims, base):
    """x [T, heads, d]: channels (2i, 2i + 1) below ``dims`` turn by position * base^(-2i / dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = torch.arange(x.shape[0], dtype=F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i], out[:, :, 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def chunked_attention(q, k, v, scale, chunk):
    """q [T, H, d], k [T, G, d], v [T, G, dv], scale [H]; position i sees j <= i of its own chunk only (None: all j <= i)."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for i in range(T):
        seen = [j for j in range(i + 1) if chunk is None or j // chunk == i // chunk]
        for h in range(H):
            s = (k[seen, h // rep] @ q[i, h]) * scale[h]
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[seen, h // rep]
    return out


def attention_mixer(h, w, p, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"]
    rot = m["rot"]
    q = rotate_pairs((h @ w[p + "q"].T).view(T, H, d), rot["dims"], rot["base"])
    k = rotate_pairs((h @ w[p + "k"].T).view(T, G, d), rot["dims"], rot["base"])
    v = (h @ w[p + "v"].T).view(T, G, dv)
    o = chunked_attention(q, k, v, m["scale"] * w[p + "temp"], m["mask"]["size"])
    return (o * sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, H * dv) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def gated_ff(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(logits, router):
    """One token's logits [E] -> [(expert, weight)]: softmax over all experts, the best groups by their largest score, the best experts
    of those, weights as they are."""
    E = logits.shape[0]
    e = torch.exp(logits - logits.max())
    s = e / e.sum()
    allowed = list(range(E))
    g = router.get("groups")
    if g:
        size = E // g["count"]
        best = sorted(range(g["count"]), key=lambda n: (-float(s[n * size:(n + 1) * size].max()), n))[:g["keep"]]
        allowed = [x for x in allowed if x // size in best]
    return [(x, s[x]) for x in sorted(allowed, key=lambda x: (-float(s[x]), x))[:router["top"]]]


def moe_ff(h, w, p, spec):
    logits = h @ w[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in route(logits[t], spec["router"]):
            out[t] += s * gated_ff(h[t:t + 1], w, p + f"e{e}.")[0]
    if spec.get("shared"):
        out = out + sigmoid(h @ w[p + "shared.sg"].T) * gated_ff(h, w, p + "shared.")
    return out


# ------------------------------------------------------------------------------------------------ the model
MIXERS = {"retention": retention_mixer, "mamba2": mamba2_mixer, "attention": attention_mixer}


def runs_of(cfg):
    """[(layer, a pass of the loop starts here)] in running order."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        out += [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return out + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg, weights, tokens):
    """-> (logits [T, vocab], stream after every layer run [runs, T, W]), float64."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    e = w["embed"][list(tokens)]
    x = e.clone()
    after = []
    for i, enters in runs_of(cfg):
        if enters:
            x = torch.cat([x, e], dim=-1) @ w["loop.in"].T
        p, layer = f"l{i}.", cfg["layers"][i]
        h = unit(x, eps) * w[p + "norm1"]
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + moe_ff(h, w, p + "mlp.", layer["mlp"])
        x = x + y
        after.append(x.clone())
    return (unit(x, eps) * w["final.norm"]) @ w["head"].T, torch.stack(after)


# ------------------------------------------------------------------------------------------------ configurations and checkpoints
def retention_layer(heads, dim, vdim, decay, mlp=None):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp}


def mamba2_layer(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups},
            "mlp": mlp}


def attention_layer(heads, kv_heads, dim, vdim, chunk, rot_dims, base=10000.0, scale=None, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
                                           "rot": {"base": base, "dims": rot_dims}, "scale": scale if scale is not None else dim ** -0.5}, "mlp": mlp}


def moe(experts, top, ff, groups=None, shared=None):
    r = {"experts": experts, "top": top}
    if groups is not None:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r, "shared": None if shared is None else {"ff": shared}}


def make_config(layers, vocab=61, width=64, eps=1e-5, loop=None):
    return {"architecture": "Leripel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "loop": None if loop is None else {"start": loop[0], "stop": loop[1], "times": loop[2]}}


def make_weights(cfg, seed=0, steady=False):
    """``steady``: a retention head's keys lie near its queries.  A sequence's first read-out is <q, k> v / sqrt(dk) before its norm: with
    unrelated q and k the product is near zero now and then, and the norm turns its rounding into a change of sign.  Output projections
    are halved, so that a row's rounding is not amplified run after run."""
    gen = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    bf = torch.bfloat16

    def mat(o, i, scale=1.0):
        return (torch.randn((o, i), generator=gen) * scale / math.sqrt(i)).to(bf)

    def vec(n, lo, hi):
        return (torch.rand((n,), generator=gen) * (hi - lo) + lo).to(bf)

    w = {"embed": torch.randn((cfg["vocab"], W), generator=gen).to(bf), "final.norm": vec(W, 0.5, 1.5), "head": mat(cfg["vocab"], W)}
    if cfg.get("loop"):
        w["loop.in"] = mat(W, 2 * W)
    for i, layer in enumerate(cfg["layers"]):
        p, m, kind = f"l{i}.", layer["mixer"], layer["type"]
        w[p + "norm1"] = vec(W, 0.5, 1.5)
        x = p + "mix."
        H, dv = m["heads"], m["vdim"]
        if kind == "retention":
            d = m["dim"]
            w[x + "q"], w[x + "k"], w[x + "v"], w[x + "g"], w[x + "o"] = mat(H * d, W), mat(H * d, W), mat(H * dv, W), mat(H * dv, W), mat(W, H * dv)
            if steady:
                w[x + "k"] = (w[x + "q"].float() + 0.5 * w[x + "k"].float()).to(bf)
        elif kind == "mamba2":
            inner, gn = H * dv, m["groups"] * m["state"]
            w[x + "in"] = mat(2 * inner + 2 * gn + H, W)
            w[x + "conv"] = (torch.randn((inner + 2 * gn, m["conv"]), generator=gen) * 0.6 + 0.25).to(bf)
            w[x + "conv.b"] = vec(inner + 2 * gn, -0.2, 0.2)
            w[x + "dt_bias"], w[x + "A_log"], w[x + "D"] = vec(H, -4.0, 0.5), vec(H, -2.0, 1.5), vec(H, -1.0, 1.0)
            w[x + "norm"], w[x + "o"] = vec(inner, 0.5, 1.5), mat(W, inner)
        else:
            G, d = m["kv_heads"], m["dim"]
            w[x + "q"], w[x + "k"], w[x + "v"], w[x + "g"], w[x + "o"] = mat(H * d, W), mat(G * d, W), mat(G * dv, W), mat(H, W, 2.0), mat(W, H * dv)
            w[x + "temp"] = vec(H, 0.5, 2.0)
        if steady:
            w[x + "o"] = 0.5 * w[x + "o"]
        ff = layer.get("mlp")
        if ff is not None:
            f, n, E = p + "mlp.", ff["expert"]["ff"], ff["router"]["experts"]
            w[f + "router"] = mat(E, W, 1.5)
            for e in range(E):
                w[f + f"e{e}.gate"], w[f + f"e{e}.up"], w[f + f"e{e}.down"] = mat(n, W, 1.5), mat(n, W, 1.5), mat(W, n)
            if ff.get("shared"):
                s = ff["shared"]["ff"]
                w[f + "shared.gate"], w[f + "shared.up"], w[f + "shared.down"], w[f + "shared.sg"] = mat(s, W), mat(s, W), mat(W, s), mat(1, W, 2.0)
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
