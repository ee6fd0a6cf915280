"""Leripel through the framework (loader, slot scheduler, ragged batches, generate loops) against the plain float64 statement of the
design in tests/leripel_oracle.py.  Every scenario runs on the CPU (the modules' torch graph: cache, slot and batching logic) and,
marked gpu, on the HIP kernels of libgbx_mixers.so.  Configurations and weights are made here; sizes differ between layers of one model
and include the corners: head sizes off every grid, one head, grouped and ungrouped key heads, partial and full rotations, chunks of 1
to beyond the sequences, convolutions of 1 to 5 taps, one norm group and several, one expert group and several, top 1, no shared
expert, layers without a feed-forward, loops that start at the first layer, end at the last, run once or never."""
import json
import os
import subprocess
import sys

import pytest
import torch

import leripel_oracle as O
from gbx_lm_amd.batching import BatchScheduler, StepBatch
from gbx_lm_amd.models.cache import SequenceSlots, SlotStateCache
from gbx_lm_amd.models.feed_forward import glu_
from gbx_lm_amd.models.recurrent_mixers import (GATE_SILU, Retention, StateSpaceDual, gate_group_norm, head_norm_gate, head_state_scan, ssm_prepare)
from gbx_lm_amd.models.residual import StreamRMSNorm, layer_update_
from gbx_lm_amd.models.sink_attention import ChunkedAttention
from gbx_lm_amd.models.step_model import loop_runs
from gbx_lm_amd.models.switch_layers import DenseRoutedGLU
from gbx_lm_amd.utils import generate_step, load_model

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-4, torch.bfloat16: 0.15}      # whole models: the worst row's rms difference over the reference row's rms
SAME = {torch.float32: 2e-4, torch.bfloat16: 0.15}     # the same arithmetic through another schedule
ROW = {torch.float32: 5e-5, torch.bfloat16: 2e-2}      # one mechanism


def model_err(got, want, dtype):
    if dtype == torch.float32:
        return O.rel_err(got, want)
    return max(O.rel_err_most(got, want, 0.95), O.rel_err(got, want) / 5)


MIXED = O.make_config([
    O.attention_layer(4, 2, 24, 16, chunk=9, rot_dims=16, base=500.0, scale=0.3, mlp=O.moe(8, 3, 32, groups=(4, 2), shared=24)),   # attention first
    O.retention_layer(3, 20, 12, (0.5, 0.97, 1.0), mlp=O.moe(6, 1, 24)),                              # top 1, no groups, no shared expert, a head that never decays
    O.mamba2_layer(4, 8, 24, groups=2, conv=3, norm_groups=4, mlp=O.moe(6, 4, 16, groups=(3, 3), shared=40)),      # every group kept
    O.attention_layer(2, 2, 16, 24, chunk=300, rot_dims=16, mlp=None),                                # a chunk longer than any test
    O.mamba2_layer(3, 20, 10, groups=1, conv=1, norm_groups=1, mlp=None),                             # one tap, sizes off the 8-grid
], vocab=61, width=64, loop=(1, 3, 3))
PLAIN = O.make_config([
    O.mamba2_layer(2, 72, 136, groups=2, conv=5, norm_groups=3, mlp=O.moe(9, 2, 32, groups=(3, 2), shared=56)),     # 136 state channels, five taps
    O.retention_layer(1, 72, 136, (0.99,), mlp=O.moe(16, 6, 32, groups=(8, 5), shared=8)),
    O.attention_layer(6, 3, 32, 40, chunk=5, rot_dims=8, base=1e6, mlp=O.moe(4, 2, 32, groups=(1, 1))),             # one expert group
    O.retention_layer(4, 16, 32, (0.9, 0.99, 0.999, 0.0), mlp=None),                                  # a head that keeps nothing
    O.attention_layer(3, 1, 8, 8, chunk=2, rot_dims=4, mlp=None),                                     # chunks of two
], vocab=40, width=136, eps=1e-6)
LOOPED = O.make_config([O.attention_layer(2, 1, 16, 16, chunk=6, rot_dims=16, mlp=O.moe(4, 2, 16, groups=(2, 1), shared=16)),
                        O.retention_layer(2, 16, 16, (0.8, 0.99), mlp=None),
                        O.mamba2_layer(2, 16, 16, groups=1, conv=4, norm_groups=2, mlp=O.moe(4, 2, 16, shared=16))], vocab=33, width=32, loop=(0, 3, 2))


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
    out = {}
    for name, cfg, seed in (("mixed", MIXED, 3), ("plain", PLAIN, 5), ("looped", LOOPED, 8)):
        for steady in (False, True):
            # bf16 runs take models whose routers choose ALL experts: a discrete choice that the rounding of one layer flips would change
            # the recurrent state of every later token, which is a property of the design and not an error of a kernel.  The choice
            # itself is tested in fp32 and in the router's own test.
            c = json.loads(json.dumps(cfg))
            if steady:
                for layer in c["layers"]:
                    if layer.get("mlp"):
                        r = layer["mlp"]["router"]
                        r["top"] = r["experts"]
                        if r.get("groups"):
                            r["groups"]["keep"] = r["groups"]["count"]
            w = O.make_weights(c, seed, steady)
            out[name, steady] = (O.save_checkpoint(str(tmp_path_factory.mktemp(name)), c, w), c, w)
    return out


def ckpt(checkpoints, name, dtype):
    return checkpoints[name, dtype == torch.bfloat16]


_loaded, _memo = {}, {}


def model_for(checkpoints, name, device, dtype):
    key = (name, device, dtype)
    if key not in _loaded:
        _loaded[key] = load_model(ckpt(checkpoints, name, dtype)[0], device=device, dtype=dtype)[0]
    return _loaded[key]


def oracle(cfg, w, toks):
    key = (id(w), tuple(toks))
    if key not in _memo:
        _memo[key] = O.forward(cfg, w, toks)
    return _memo[key]


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def run_portions(fn, total, portions, device, slots, slot=0):
    """Calls fn(first row, rows, batch) portion by portion on one slot and concatenates what it returns."""
    out, pos = [], 0
    for n in portions:
        out.append(fn(pos, n, StepBatch.build([slot], [pos], [n], device)))
        pos += n
        slots.length[slot] = pos
    assert pos == total
    return torch.cat(out)


def fresh_slots(n=2):
    slots = SequenceSlots(n)
    for i in range(n):
        slots.length[i] = 0
    return slots


SCHEDULES = lambda T: ([T], [T - 9] + [1] * 9, [1] * T, [2] * (T // 2) + [T % 2] * (T % 2), [3, 1, 5, T - 9])


def mixer_of(layer, width, seed, device, dtype, eps=1e-5):
    """(the framework's mixer with its own projections, the oracle's weights) for one layer's random tensors."""
    cfg = O.make_config([layer], width=width, eps=eps)
    w = O.make_weights(cfg, seed)
    m, p, kind = layer["mixer"], "l0.mix.", layer["type"]
    if kind == "retention":
        mod = Retention(width, m["heads"], m["dim"], m["vdim"], m["decay"], eps)
        rows = torch.cat([w[p + n] for n in "qkvg"])
    elif kind == "mamba2":
        mod = StateSpaceDual(width, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], eps)
        rows = w[p + "in"]
        mod.conv = w[p + "conv"].t().contiguous().to(dtype)
        mod.conv_bias, mod.dt_bias, mod.skip, mod.out_norm = (w[p + n].float() for n in ("conv.b", "dt_bias", "D", "norm"))
        mod.rate = torch.exp(w[p + "A_log"].float())
    else:
        mod = ChunkedAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["rot"]["dims"], m["rot"]["base"], m["mask"]["size"], m["scale"])
        rows = torch.cat([w[p + n] for n in "qkvg"])
        mod.temp = w[p + "temp"].float()
    full = torch.zeros((mod.in_rows, width), dtype=rows.dtype)
    full[:rows.shape[0]] = rows
    mod.inp.weight.data, mod.o.weight.data = full.to(dtype), w[p + "o"].to(dtype)
    return mod.to(device), {k: v.to(O.F64) for k, v in w.items()}


# ------------------------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", [O.retention_layer(3, 20, 12, (0.5, 0.97, 1.0)), O.retention_layer(2, 64, 80, (0.999, 0.9)), O.retention_layer(1, 7, 5, (0.8,)),
                                   O.retention_layer(2, 136, 72, (0.0, 0.95)), O.mamba2_layer(4, 8, 24, 2, 3, 4), O.mamba2_layer(3, 20, 10, 1, 1, 1),
                                   O.mamba2_layer(2, 72, 136, 2, 5, 3), O.mamba2_layer(6, 16, 64, 3, 4, 2), O.mamba2_layer(5, 3, 6, 5, 2, 5),
                                   O.attention_layer(4, 2, 24, 16, 9, 16, 500.0, 0.3), O.attention_layer(3, 3, 10, 6, 7, 4), O.attention_layer(2, 1, 16, 32, 1, 16),
                                   O.attention_layer(4, 1, 64, 48, 64, 0)],
                         ids=lambda l: "-".join([l["type"]] + [str(l["mixer"][k]) for k in ("heads", "vdim") ]))
def test_mixers_alone(device, dtype, layer):
    """Each mixer with its own projections in every schedule (whole, decoded, portions of two, portions across every edge) on a slot whose
    buffers another sequence left dirty; a prompt of several scan chunks too."""
    mod, w = mixer_of(layer, 40, 7, device, dtype)
    for T in (33, 300):
        h = torch.randn((T, 40), generator=torch.Generator().manual_seed(11)).to(dtype)
        want = O.MIXERS[layer["type"]](h.to(O.F64), w, "l0.mix.", layer["mixer"], 1e-5)
        for portions in (SCHEDULES(T) if T < 100 else ([T], [T - 20] + [1] * 20, [129, 127, 44], [2, T - 2], [40] * 7 + [20])):
            slots = fresh_slots()
            cache = mod.make_cache(slots)
            if isinstance(cache, SlotStateCache):
                cache.reserve(dtype, device)
                cache.state.fill_(1.5)
                cache.tail.fill_(2.0)
            got = run_portions(lambda p, n, b: mod(h[p:p + n].to(device), b, cache), T, portions, device, slots, slot=1)
            assert model_err(got, want, dtype) < (1e-4 if dtype == torch.float32 else 4e-2), (T, portions[:4])      # (bf16: a small read-out's norm magnifies its rounding)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dk,dv,heads,groups", [(64, 64, 4, 2), (128, 128, 2, 2), (40, 72, 6, 1), (256, 24, 1, 1), (400, 16, 2, 1), (16, 8, 3, 3), (30, 9, 2, 1)])
def test_state_scan_is_32_bit(device, dtype, dk, dv, heads, groups):
    """The state, the decays and the sums are 32-bit in both dtypes and in every kernel form (q, k and v are the same bf16 numbers here):
    unequal sequences of one step with history, log decays per row from tiny to -40, write factors, skip.  Then one more step."""
    g = torch.Generator().manual_seed(5)
    lens = [(0, 270, 1), (3, 5, 0), (9, 130, 2), (0, 1, 3)]                  # (earlier tokens, new tokens, slot)
    T = sum(n for _, n, _ in lens)
    rows = torch.randn((T, 2 * groups * dk + heads * dv + 5), generator=g).to(torch.bfloat16)
    rows = rows[:, :rows.shape[1] // 8 * 8] if rows.shape[1] % 8 < 5 else rows[:, :rows.shape[1]]
    log_decay = -torch.exp(torch.rand((T, heads), generator=g) * 9 - 7)
    log_decay[torch.rand((T, heads), generator=g) < 0.02] = -40.0
    write = torch.rand((T, heads), generator=g) * 2
    skip = torch.randn((heads,), generator=g)
    state = torch.randn((4, heads, dv, dk), generator=g)
    cache = SlotStateCache(heads, dk, dv, 0, 0, fresh_slots(4))
    cache.reserve(dtype, device)
    cache.state.copy_(state)
    off_v = 2 * groups * dk
    batch = StepBatch.build([s for _, _, s in lens], [p for p, _, _ in lens], [n for _, n, _ in lens], device)
    dt = torch.stack([log_decay, write], dim=1).to(device)
    got = head_state_scan(rows.to(dtype).to(device), heads, groups, dk, dv, 0, groups * dk, off_v, cache, batch, 0.7, log_decay=dt[:, 0], write=dt[:, 1],
                          skip=skip.to(device)).cpu().double()
    r0 = 0
    for pos0, n, slot in lens:
        f = rows[r0:r0 + n].to(O.F64)
        q, k = (f[:, i * groups * dk:(i + 1) * groups * dk].view(n, groups, dk).repeat_interleave(heads // groups, 1) for i in (0, 1))
        v = f[:, off_v:off_v + heads * dv].view(n, heads, dv)
        S = state[slot].double().transpose(1, 2) if pos0 else torch.zeros((heads, dk, dv), dtype=O.F64)
        want = []
        for t in range(n):
            S = torch.exp(log_decay[r0 + t].double())[:, None, None] * S + (write[r0 + t].double()[:, None] * k[t])[:, :, None] * v[t][:, None, :]
            want.append(0.7 * (S * q[t][:, :, None]).sum(1) + skip.double()[:, None] * v[t])
        want = torch.stack(want).view(n, -1)
        assert (got[r0:r0 + n] - want).abs().max() < 2e-5 * want.abs().max(), (pos0, n)
        left = cache.state[slot].cpu().double().transpose(1, 2)
        assert (left - S).abs().max() < 1e-5 * S.abs().max(), (pos0, n)
        r0 += n


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_one_write_is_carried(device, dtype):
    """ONE WRITE STANDS OUT: a head that (almost) never decays gets one key-value pair; everything after it is orthogonal to the query, and
    400 tokens later the query reads exactly that value -- whole, across prompt / decode borders, with a portion border at the write."""
    T, far = 420, 7
    d = 16
    m = Retention(3 * d, 1, d, d, (1.0,), 1e-6)
    w = torch.zeros((m.in_rows, 3 * d))
    w[:3 * d] = torch.eye(3 * d)                              # q | k | v are the input's channels, the gate's rows stay zero
    m.inp.weight.data = w.to(dtype)
    m.o.weight.data = torch.eye(3 * d, d).to(dtype)
    m = m.to(device)
    g = torch.Generator().manual_seed(2)
    h = torch.zeros((T, 3 * d))
    h[:, d + 1:2 * d] = torch.randn((T, d - 1), generator=g)  # keys without a first channel
    h[:, 2 * d:] = torch.randn((T, d), generator=g)
    h[far, d] = 3.0                                           # the one write under the first channel
    h[T - 1, 0] = 2.0                                         # the one query
    hq = h.to(dtype)
    gate_w = w.clone()
    gate_w[3 * d:4 * d, 0] = 1.0                              # the gate opens where the query is: silu(2)
    m.inp.weight.data = gate_w.to(dtype).to(device)
    v = hq[far, 2 * d:].double()
    want = O.unit(v * 6.0 * d ** -0.5, 1e-6) * float(O.silu(torch.tensor(2.0, dtype=O.F64)))
    for portions in ([T], [T - 30] + [1] * 30, [far + 1, T - far - 1], [far, 2, T - far - 2], [1] * 20 + [T - 20]):
        slots = fresh_slots()
        cache = m.make_cache(slots)
        got = run_portions(lambda p, n, b: m(hq[p:p + n].to(device), b, cache), T, portions, device, slots)
        assert (got[-1, :d].cpu().double() - want).abs().max() < (1e-4 if dtype == torch.float32 else 2e-2), portions[:3]


def _copy_attention(device, dtype, chunk, d=16, heads=2, scale=3.0, temp=(1.0, 0.5)):
    """An attention mixer whose projections copy input channels: q heads, then k, then v; gates wide open; no rotation."""
    width = heads * d + 2 * d
    m = ChunkedAttention(width, heads, 1, d, d, 0, 10000.0, chunk, scale)
    w = torch.zeros((m.in_rows, width))
    w[:width] = torch.eye(width)
    m.inp.weight.data, m.o.weight.data = w.to(dtype), torch.eye(width, heads * d).to(dtype)
    m.temp = torch.tensor(temp)
    return m.to(device), width


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [70, 64, 3, 1, None])
def test_chunk_edges_stand_out(device, dtype, chunk):
    """ONE KEY STANDS OUT: a token's queries score one chosen position far above all others.  The chunk's first key must be found from the
    chunk's last token, the last key of the chunk before must not be seen from the chunk's first and second token; without chunks the
    very first token is found -- whole, prompt + decoding across the table, token by token, portion borders at the target and the edge."""
    d, T = 16, 213
    m, width = _copy_attention(device, dtype, chunk, d)
    base = torch.randn((T, width), generator=torch.Generator().manual_seed(9))
    c = chunk or T
    edge = (T - 2) // c * c                                   # a chunk's first token
    cases = [(min(edge + c, T) - 1, edge), (edge, edge), (T - 1, 0 if chunk is None else edge)]
    if edge:
        cases += [(edge, edge - 1), (min(edge + 1, T - 1), edge - 1), (edge, 0), (edge + min(c, 2) - 1, max(edge - c, 0))]
    for at, target in cases:
        h = base.clone()
        h[target, 2 * d:3 * d] *= 2.0
        h[at, :d] = h[target, 2 * d:3 * d] * 2.0              # head 0 looks for the target, head 1 stays random
        hq = h.to(dtype)
        f = hq.to(O.F64)
        q, k, v = f[:, :2 * d].view(T, 2, d), f[:, 2 * d:3 * d].view(T, 1, d), f[:, 3 * d:].view(T, 1, d)
        want = 0.5 * O.chunked_attention(q, k, v, 3.0 * torch.tensor([1.0, 0.5], dtype=O.F64), chunk).reshape(T, 2 * d)
        seen = chunk is None or at // chunk == target // chunk
        assert ((want[at, :d] - 0.5 * v[target, 0]).abs().max() < 1e-2) == seen, (at, target)
        for portions in ([T], [T - 75] + [1] * 75, [target + 1, T - target - 1], [at, T - at] if at else [T], [1] * T if target == edge else [T - 1, 1]):
            if 0 in portions:
                continue
            slots = fresh_slots()
            cache = m.make_cache(slots)
            cache.reserve(4, dtype, device)
            cache.keys.fill_(3.0)                             # another sequence's keys and values
            cache.values.fill_(50.0)
            got = run_portions(lambda p, n, b: m(hq[p:p + n].to(device), b, cache), T, portions, device, slots, slot=1)
            assert O.rel_err(got[:, :2 * d], want) < (2e-5 if dtype == torch.float32 else 6e-2), (at, target, portions[:3])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,d,dv,chunk", [(8, 8, 64, 64, 96), (4, 2, 128, 128, 40), (6, 2, 24, 40, 130), (2, 1, 12, 20, 33)])
def test_chunked_attention_in_batches(device, dtype, heads, groups, d, dv, chunk):
    """Unequal sequences with history in one step, query tiles that span several chunks, temperatures (one negative), output gates."""
    layer = O.attention_layer(heads, groups, d, dv, chunk, rot_dims=d // 4 * 2, base=900.0)
    mod, w = mixer_of(layer, 48, 3, device, dtype)
    temp = torch.linspace(-0.6, 1.9, heads)
    mod.temp, w["l0.mix.temp"] = temp.to(device), temp.double()
    seqs = [300, 7, 141, 64]
    hs = [torch.randn((n, 48), generator=torch.Generator().manual_seed(i)).to(dtype) for i, n in enumerate(seqs)]
    wants = [O.attention_mixer(h.to(O.F64), w, "l0.mix.", layer["mixer"], 1e-5) for h in hs]
    slots = fresh_slots(4)
    cache = mod.make_cache(slots)
    for cuts in ([200, 4, 1, 60], [99, 2, 139, 3], [1, 1, 1, 1]):
        rows = torch.cat([h[p:p + n] for h, p, n in zip(hs, slots.length, cuts)])
        batch = StepBatch.build([0, 1, 2, 3], list(slots.length), cuts, device)
        got = mod(rows.to(device), batch, cache)
        r = 0
        for i, n in enumerate(cuts):
            assert O.rel_err(got[r:r + n], wants[i][slots.length[i]:slots.length[i] + n]) < (1e-4 if dtype == torch.float32 else 4e-2), (cuts, i)
            slots.length[i] += n
            r += n


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps,channels,heads", [(4, 48, 5), (1, 20, 2), (5, 13, 3), (2, 640, 70)])
def test_state_space_rows(device, dtype, taps, channels, heads):
    """Convolution with bias, zeros in front, silu, softplus of large and small steps: portions shorter than the tail, two sequences at once."""
    g = torch.Generator().manual_seed(4)
    T, off_x, off_dt = 21, 8, 8 + channels
    y = torch.randn((T, off_dt + heads + 3), generator=g).to(dtype)
    y[:, off_dt:] *= 12.0
    conv, bias = torch.randn((channels, taps), generator=g).to(dtype), torch.randn((channels,), generator=g)
    dt_bias, rate = torch.randn((heads,), generator=g), torch.rand((heads,), generator=g) * 3
    f = y.to(O.F64)
    want = O.silu(O.causal_conv(f[:, off_x:off_x + channels], conv.to(O.F64), bias.to(O.F64)))
    w_want = O.softplus(f[:, off_dt:off_dt + heads] + dt_bias.to(O.F64))
    for portions in SCHEDULES(T):
        slots = fresh_slots(3)
        cache = SlotStateCache(heads, 4, 4, channels if taps > 1 else 0, taps, slots)
        cache.reserve(dtype, device)
        cache.tail.fill_(7.0)
        pos, got, dts = 0, [], []
        for n in portions:
            rows = torch.cat([y[pos:pos + n], y[:1]])         # beside it the first token of another sequence, over and over
            x, dt = ssm_prepare(rows.to(device), off_x, off_dt, conv.t().contiguous().to(device), bias.to(device), dt_bias.to(device), rate.to(device),
                                cache, StepBatch.build([2, 0], [pos, 0], [n, 1], device))
            assert O.rel_err(x[n:], want[:1]) < ROW[dtype]
            got.append(x[:n])
            dts.append(dt[:n])
            pos += n
        assert O.rel_err(torch.cat(got), want) < ROW[dtype], portions[:3]
        dt = torch.cat(dts).cpu().double()
        assert (dt[:, 1] - w_want).abs().max() < 1e-5 * w_want.abs().max() and (dt[:, 0] + rate.double() * w_want).abs().max() < 1e-5 * w_want.abs().max() * 3


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_norms_of_read_outs(device, dtype):
    """Head norm without a weight; gate first, then norm in 1 to 9 parts (parts longer than a thread's registers); rows with a stride."""
    g = torch.Generator().manual_seed(6)
    for n, parts in ((48, 4), (90, 9), (9000, 1), (1300, 2), (7, 1)):
        o, z, w = torch.randn((5, n), generator=g), torch.randn((5, n + 8), generator=g).to(dtype), torch.rand((n,), generator=g) + 0.5
        out = torch.zeros((5, n + 24), dtype=dtype, device=device)
        gate_group_norm(o.to(device), z.to(device)[:, :n], w.to(device), parts, 1e-5, out[:, 8:8 + n])
        assert O.rel_err(out[:, 8:8 + n], O.gate_then_group_norm(o.double(), z[:, :n].double(), w.double(), parts, 1e-5)) < ROW[dtype], (n, parts)
        head_norm_gate(o.to(device), z.to(device)[:, :n], None, parts, 1e-5, GATE_SILU, out[:, 16:16 + n])
        want = O.unit(o.double().view(5, parts, -1), 1e-5).reshape(5, n) * O.silu(z[:, :n].double())
        assert O.rel_err(out[:, 16:16 + n], want) < ROW[dtype], (n, parts)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("rows", [5, 70])
@pytest.mark.parametrize("experts,top,groups,gate", [(8, 3, (4, 2), True), (6, 1, None, True), (12, 12, (3, 3), False), (130, 8, (13, 4), True), (5, 2, (1, 1), False),
                                                     (300, 6, (10, 1), True), (64, 4, None, False)])
def test_router_with_groups_and_a_gate_row(device, rows, experts, top, groups, gate):
    """The choice and the weights of every row: groups by their largest score, probabilities over ALL experts as they are, equal logits by
    the lower index, the gate's sigmoid in the last column -- for steps of few rows and of many."""
    g = torch.Generator().manual_seed(7)
    width = 24
    m = DenseRoutedGLU(width, 8, experts, top, groups=groups, gate_row=gate)
    eighths = lambda *shape: torch.round(torch.randn(shape, generator=g) * 8) / 8          # products and sums of these are exact: equal stays equal
    m.router = eighths(*m.router.shape)
    if experts > 4:
        m.router[2] = m.router[0]                             # equal scores, in one group or in two
        m.router[experts - 1] = m.router[0]
    m = m.to(device)
    h = eighths(rows, width)
    idx, w = m.route(h.to(device))
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    logits = h.double() @ m.router.cpu().double().T
    for t in range(rows):
        want = O.route(logits[t, :experts], r)
        assert idx[t].cpu().tolist() == [e for e, _ in want], t
        assert (w[t, :top].cpu().double() - torch.stack([s for _, s in want])).abs().max() < 1e-5
        if gate:
            assert abs(float(w[t, top]) - float(O.sigmoid(logits[t, experts]))) < 1e-5
    assert w.shape == (rows, top + int(gate))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_layer_update(device, dtype):
    """Add or replace, candidates with fp32 weights (a further column unused), image rows with a stride, the next norm; widths on and off
    the vector grid and beyond a thread's registers."""
    g = torch.Generator().manual_seed(8)
    for width, top in ((64, 3), (37, 1), (5000, 2), (8200, 0)):
        x, a = torch.randn((4, width), generator=g), torch.randn((4, width), generator=g).to(dtype)
        cand = torch.randn((4, top, width), generator=g).to(dtype) if top else None
        mix = torch.rand((4, top + 1), generator=g) if top else None
        norm = StreamRMSNorm(width, 1e-5)
        norm.weight = torch.rand((width,), generator=g) + 0.5
        for replace in (False, True):
            want = a.double() + (0.0 if replace else x.double())
            if top:
                want = want + (cand.double() * mix[:, :top, None].double()).sum(1)
            s = x.clone().to(device)
            img = torch.zeros((4, 2 * width + 4), dtype=dtype, device=device)
            h = layer_update_(s, a.to(device), None if cand is None else cand.to(device), None if mix is None else mix.to(device), norm.to(device),
                              img[:, 4:4 + width], replace)
            assert O.rel_err(s, want) < 1e-6 and O.rel_err(img[:, 4:4 + width], want) < ROW[dtype] and h.dtype == dtype
            assert float(img[:, :4].abs().max()) == 0 and float(img[:, 4 + width:].abs().max()) == 0
            assert O.rel_err(h, O.unit(want, 1e-5) * norm.weight.cpu().double()) < ROW[dtype]
            assert layer_update_(s, a.to(device), None, None, None, None, True) is None and O.rel_err(s, a) == 0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_gated_rows_with_a_factor_per_row(device, dtype):
    g = torch.Generator().manual_seed(9)
    for f in (24, 7, 1500):
        gu, s = torch.randn((6, 2 * f + 8), generator=g).to(dtype), torch.rand((6, 3), generator=g)
        out = torch.zeros((6, f + 8), dtype=dtype, device=device)
        glu_(gu.to(device)[:, :2 * f], "silu", row_scale=s.to(device)[:, 2], out=out[:, 8:])
        want = O.silu(gu[:, :f].double()) * gu[:, f:2 * f].double() * s[:, 2:].double()
        assert O.rel_err(out[:, 8:], want) < ROW[dtype] and float(out[:, :8].abs().max()) == 0


def test_loop_runs():
    assert loop_runs(3, None) == [(0, False), (1, False), (2, False)]
    assert loop_runs(4, {"start": 1, "stop": 3, "times": 2}) == [(0, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert loop_runs(2, {"start": 0, "stop": 2, "times": 1}) == [(0, True), (1, False)]
    assert loop_runs(2, {"start": 1, "stop": 2, "times": 0}) == [(0, False)]
    with pytest.raises(ValueError):
        loop_runs(2, {"start": 1, "stop": 3, "times": 1})


# ------------------------------------------------------------------------------------------------ whole models
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "plain", "looped"])
def test_model_layers_against_oracle(checkpoints, device, dtype, name):
    """One prompt through the scheduler: the stream after every layer run and the logits of every position."""
    path, cfg, w = ckpt(checkpoints, name, dtype)
    model = model_for(checkpoints, name, device, dtype)
    toks = tokens_for(cfg, 45, 1)
    want, after = oracle(cfg, w, toks)
    model.trace_layers = []
    try:
        got = BatchScheduler(model).step([("a", toks)], [list(range(len(toks)))])
        layers = torch.stack([x.cpu() for x in model.trace_layers])
    finally:
        model.trace_layers = None
    assert layers.shape[0] == after.shape[0] == len(O.runs_of(cfg))
    if dtype == torch.float32:
        for i in range(layers.shape[0]):
            assert O.rel_err(layers[i], after[i]) < 1e-4, i
    assert model_err(got, want, dtype) < TOL[dtype]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("loop", [None, (1, 2, 1), (0, 1, 3), (1, 3, 2), (1, 3, 0), (2, 2, 4)])
def test_loop_spans(device, loop, tmp_path):
    """A span at the start, in the middle and at the end; one pass (its entry product counts too), none, an empty span, no loop."""
    layers = [O.retention_layer(2, 8, 8, (0.7, 0.98), mlp=None), O.attention_layer(2, 1, 8, 8, 5, 8, mlp=O.moe(4, 2, 8, groups=(2, 1), shared=8)),
              O.mamba2_layer(2, 8, 8, 1, 3, 1, mlp=None)]
    cfg = O.make_config(layers, vocab=29, width=24, loop=loop)
    w = O.make_weights(cfg, 13)
    model = load_model(O.save_checkpoint(str(tmp_path), cfg, w), device=device, dtype=torch.float32)[0]
    toks = tokens_for(cfg, 19, 2)
    want = O.forward(cfg, w, toks)[0]
    eng = BatchScheduler(model)
    got = torch.cat([eng.step([("a", toks[:11])], [list(range(11))])] + [eng.step([("a", [t])]) for t in toks[11:]])
    assert O.rel_err(got, want) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "plain"])
def test_prefill_against_decoding(checkpoints, device, dtype, name):
    """A prompt, then 70 single-token steps (on the GPU the later ones are graph replays): chunks begin and end among decoded tokens, tables
    wrap, states recur; against the oracle and against the whole sequence in one step."""
    path, cfg, w = ckpt(checkpoints, name, dtype)
    model = model_for(checkpoints, name, device, dtype)
    toks = tokens_for(cfg, 90, 2)
    want, _ = oracle(cfg, w, toks)
    whole = BatchScheduler(model).step([("a", toks)], [list(range(90))])
    eng = BatchScheduler(model)
    got = [eng.step([("a", toks[:20])], [list(range(20))])] + [eng.step([("a", [t])]) for t in toks[20:]]
    got = torch.cat(got)
    assert model_err(got, want, dtype) < TOL[dtype]
    assert model_err(got, whole, dtype) < SAME[dtype]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["mixed", "plain"])
@pytest.mark.parametrize("size", [2, 3, 16, 64])
def test_portions(checkpoints, device, name, size):
    path, cfg, w = ckpt(checkpoints, name, torch.float32)
    model = model_for(checkpoints, name, device, torch.float32)
    toks = tokens_for(cfg, 70, 3)
    want, _ = oracle(cfg, w, toks)
    eng = BatchScheduler(model)
    got = torch.cat([eng.step([("a", toks[i:i + size])], [list(range(len(toks[i:i + size])))]) for i in range(0, 70, size)])
    assert O.rel_err(got, want) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batch_and_slot_reuse(checkpoints, device, dtype):
    """Four unequal requests (1, 7, 33, 140 tokens) start in one step and decode together; the shortest ends first, a new request takes
    its slot while the others go on.  Every logit against the oracle and against the request alone."""
    path, cfg, w = ckpt(checkpoints, "mixed", dtype)
    model = model_for(checkpoints, "mixed", device, dtype)
    start = {"a": 1, "b": 7, "c": 33, "d": 140}
    full = {k: tokens_for(cfg, n + 12, 30 + i) for i, (k, n) in enumerate(start.items())}
    eng = BatchScheduler(model)
    got = {k: [] for k in full}
    out = eng.step([(k, full[k][:start[k]]) for k in "abcd"], [list(range(start[k])) for k in "abcd"])
    r = 0
    for k in "abcd":
        got[k].append(out[r:r + start[k]])
        r += start[k]
    done = dict(start)
    live = list("abcd")
    late = tokens_for(cfg, 9, 77)
    for step in range(12):
        if step == 4:
            eng.release("a")
            live.remove("a")
            freed = eng.step([("e", late)], [list(range(9))])                 # takes the slot that "a" left
            assert model_err(freed, oracle(cfg, w, late)[0], dtype) < TOL[dtype]
        out = eng.step([(k, [full[k][done[k]]]) for k in live])
        for i, k in enumerate(live):
            got[k].append(out[i:i + 1])
            done[k] += 1
    assert len(set(eng.slot_of.values())) == 4
    for k in full:
        seen = torch.cat(got[k])
        want = oracle(cfg, w, full[k][:seen.shape[0]])[0]
        assert model_err(seen, want, dtype) < TOL[dtype], k
        alone = BatchScheduler(model).step([("x", full[k][:seen.shape[0]])], [list(range(seen.shape[0]))])
        assert model_err(seen, alone, dtype) < SAME[dtype], k


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_steps_of_prompts_and_decoding(checkpoints, device):
    """Sequences that start, go on in portions and decode share steps; slot tables grow under running sequences."""
    path, cfg, w = ckpt(checkpoints, "looped", torch.float32)
    model = model_for(checkpoints, "looped", device, torch.float32)
    seqs = {k: tokens_for(cfg, 60, 40 + i) for i, k in enumerate("abcde")}
    plan = [{"a": 5}, {"a": 1, "b": 30}, {"a": 1, "b": 2, "c": 1}, {"a": 7, "b": 1, "c": 40, "d": 3}, {"a": 1, "b": 1, "c": 1, "d": 1, "e": 33},
            {"a": 1, "b": 1, "c": 1, "d": 1, "e": 1}, {"a": 1, "b": 1, "c": 1, "d": 1, "e": 1}, {"a": 1, "b": 1, "c": 1, "d": 1, "e": 1}, {"e": 2, "d": 20}]
    eng = BatchScheduler(model)
    got, done = {k: [] for k in seqs}, {k: 0 for k in seqs}
    for step in plan:
        out = eng.step([(k, seqs[k][done[k]:done[k] + n]) for k, n in step.items()], [list(range(n)) for n in step.values()])
        r = 0
        for k, n in step.items():
            got[k].append(out[r:r + n])
            done[k] += n
            r += n
    for k in seqs:
        assert O.rel_err(torch.cat(got[k]), oracle(cfg, w, seqs[k][:done[k]])[0]) < TOL[torch.float32], k


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_from_the_first_token(checkpoints, device):
    """320 single-token steps from the first token: chunks of 6, tables that start over dozens of times, states that recur 320 times."""
    path, cfg, w = ckpt(checkpoints, "looped", torch.float32)
    model = model_for(checkpoints, "looped", device, torch.float32)
    toks = tokens_for(cfg, 320, 4)
    want, _ = oracle(cfg, w, toks)
    eng = BatchScheduler(model)
    got = torch.cat([eng.step([("a", [t])]) for t in toks])
    assert O.rel_err(got, want) < 2e-4


# ------------------------------------------------------------------------------------------------ generation
@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_entry_points(checkpoints, device, tmp_path):
    """Greedy tokens through generate_step (one sequence), BatchScheduler.generate (a batch) and the command line agree with the
    oracle's own greedy loop."""
    path, cfg, w = ckpt(checkpoints, "looped", torch.float32)
    model = model_for(checkpoints, "looped", device, torch.float32)
    prompts = [tokens_for(cfg, 9, 20), tokens_for(cfg, 4, 21)]
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(8):
            seq.append(int(torch.argmax(O.forward(cfg, w, seq)[0][-1])))
        want.append(seq[len(p):])
    one = [t for t, _, _ in generate_step(torch.tensor(prompts[0]), model, max_tokens=8)]
    assert [int(t) for t in one] == want[0]
    assert BatchScheduler(model).generate(prompts, max_tokens=8) == want
    if device == "cpu":
        cmd = [sys.executable, "-m", "gbx_lm_amd.cli", "--model", path, "--dtype", "float32", "--max-tokens", "8"]
        for p in prompts:
            cmd += ["--prompt-ids", ",".join(map(str, p))]
        env = dict(os.environ, CUDA_VISIBLE_DEVICES="", HIP_VISIBLE_DEVICES="")
        out = subprocess.run(cmd, capture_output=True, text=True, check=True, env=env, cwd=os.path.dirname(os.path.dirname(__file__)))
        assert [json.loads(l)["tokens"] for l in out.stdout.strip().splitlines()] == want


@pytest.mark.parametrize("device", DEVICES)
def test_trace_replay_program(checkpoints, device, tmp_path):
    """bin/trace_run on a schedule with a ragged start, decoding, a request that ends and one that takes its slot."""
    path, cfg, w = ckpt(checkpoints, "looped", torch.float32)
    a, b, c = tokens_for(cfg, 12, 30), tokens_for(cfg, 5, 31), tokens_for(cfg, 6, 32)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[9:10], "want": [0]}, {"id": "b", "tokens": b[3:4], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:11], "want": []}, {"id": "b", "tokens": b[4:5], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [5]}], "end": ["c"]},
             {"step": 4, "entries": [{"id": "a", "tokens": a[11:12], "want": [0]}], "end": ["a"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    env = dict(os.environ)
    if device == "cpu":
        env.update(CUDA_VISIBLE_DEVICES="", HIP_VISIBLE_DEVICES="")
    out = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, env=env, cwd=root)
    assert out.returncode == 0, out.stderr[-2000:]
    assert [l for l in out.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    la, lb, lc = oracle(cfg, w, a)[0], oracle(cfg, w, b)[0], oracle(cfg, w, c)[0]
    import numpy as np
    read = lambda i: torch.from_numpy(np.fromfile(os.path.join(str(tmp_path), f"{i}.f32"), dtype="<f4").reshape(-1, cfg["vocab"]).copy())
    assert O.rel_err(read(0), torch.stack([la[0], la[8], lb[2]])) < 3e-5
    assert O.rel_err(read(1), la[9:10]) < 3e-5 and O.rel_err(read(2), lb[4:5]) < 3e-5
    assert O.rel_err(read(3), lc[5:6]) < 3e-5 and O.rel_err(read(4), la[11:12]) < 3e-5
