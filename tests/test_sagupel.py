"""The Sagupel model and its mechanisms through the serving engine against the plain float64 statement (tests/_sagupel_plain.py).

Every test runs with the unfused tensor-op backend on the CPU (host logic: pages, state rows, runs, the layers' composition) and,
marked `gpu`, with the HIP kernels.  Configurations and weights are made here: small, random, sizes unlike each other so that a mixed-up
dimension shows; where random weights would hide a fault (one key among hundreds, a window's edge, a sink that is left out, a state that
is lost, a head that listens to the wrong head) the weights or inputs are made so that it shows.
"""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

import _sagupel_plain as P
from qserve_amd.layers.moe import GatedFeedForward
from qserve_amd.layers.ops import make_ops
from qserve_amd.layers.recurrent import GatedDeltaRule, Retention
from qserve_amd.layers.rotary import RotaryTable
from qserve_amd.layers.softmax_attention import SinkWindowAttention, distance_slopes
from qserve_amd.models.sagupel import Sagupel
from qserve_amd.serving import Engine, SamplingParams
from qserve_amd.serving.cache import CacheFull, PagedCache, StateSpec
from qserve_amd.serving.engine import StepBatch

BACKENDS = [pytest.param("unfused", id="unfused-cpu"), pytest.param("hip", marks=pytest.mark.gpu, id="hip")]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
STORAGE = [pytest.param(torch.float32, 2e-5, id="float32"), pytest.param(torch.bfloat16, 3e-2, id="bfloat16")]


@pytest.fixture(params=BACKENDS)
def backend(request):
    if request.param == "hip" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    return request.param


def device_of(backend):
    return "cuda:0" if backend == "hip" else "cpu"


def att(heads=6, kv_heads=2, dim=12, size=24, scale=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": size},
         "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def ret(heads=3, dim=10, vdim=14, rot=6, base=300.0, decay=None, mlp=None):
    decay = decay or [1.0 - 2.0 ** -(2 + h) for h in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": rot}}, "mlp": mlp}


def par(heads=6, kv_heads=3, dim=8, rot=4, base=1000.0, factor=4.0, cap=5.0, scale=None, d_heads=4, d_kv=2, d_dim=6, d_vdim=10, conv=4, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "softcap": cap, "rot": {"base": base, "dims": rot},
            "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}
    if factor is not None:
        left["rot"]["scaling"] = {"factor": factor}
    right = {"heads": d_heads, "kv_heads": d_kv, "dim": d_dim, "vdim": d_vdim, "conv": conv}
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def dense(ff=28, limit=0.8):
    return {"kind": "dense", "ff": ff, "limit": limit}


def make_config(layers, width=40, vocab=53, eps=1e-5, alpha=1.7, taps=4):
    return {"architecture": "Sagupel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "postln_alpha": alpha, "canon": {"taps": taps},
            "layers": layers}


def standard_config():
    return make_config([par(mlp=dense()), ret(mlp=dense(19, 2.5)), att(mlp=dense(36, 1.2)), att(heads=2, kv_heads=1, dim=6, size=64, mlp=None),
                        par(heads=2, kv_heads=2, dim=6, rot=6, cap=50.0, factor=None, d_heads=3, d_kv=3, d_dim=4, d_vdim=4, conv=2, mlp=None),
                        ret(heads=5, dim=6, vdim=4, rot=6, base=1e4, mlp=dense(12))])


def t64(W):
    return {k: torch.from_numpy(np.asarray(v)) for k, v in W.items()}


def f32(W):
    return {k: v.float() for k, v in t64(W).items()}


def bf16(W):
    return {k: v.bfloat16() for k, v in t64(W).items()}


def build_engine(cfg, W, backend, dtype="float32", max_tokens=1024, max_seqs=4, **kw):
    return Engine(Sagupel, cfg, W, dtype=dtype, device=device_of(backend), max_tokens=max_tokens, max_seqs=max_seqs, backend=backend, **kw)


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def plain_logits(cfg, W, toks, taps=None):
    return torch.from_numpy(P.forward(cfg, W, toks, taps))


def run_schedule(eng, seqs, steps):
    """seqs: {name: tokens}; steps: [[(name, count), ...]] -> {name: logits [len, vocab]}; a sequence is closed after its last token."""
    at, slots, got = {k: 0 for k in seqs}, {}, {k: [] for k in seqs}
    for step in steps:
        items, want, n = [], [], 0
        for name, count in step:
            if name not in slots:
                slots[name] = eng.open_sequence()
            items.append((slots[name], seqs[name][at[name]:at[name] + count]))
            want += range(n, n + count)
            n += count
        logits = eng.execute(items, want).double().cpu()
        n = 0
        for name, count in step:
            got[name].append(logits[n:n + count])
            n += count
            at[name] += count
            if at[name] == len(seqs[name]):
                eng.close_sequence(slots.pop(name))
    return {k: torch.cat(v) for k, v in got.items() if v}


def assert_close(got, ref, tol, what=""):
    ref = torch.as_tensor(ref)
    err = (got - ref).abs().max().item()
    scale = max(1.0, ref.abs().max().item())
    assert err <= tol * scale, f"{what}: max error {err:.3e} (allowed {tol * scale:.3e})"


F32_TOL = 2e-4      # float32 runs of a whole model against float64 (a fault shows at 1e-2 and above)


def run_batch(lo, hi, dev, slot=0, rd=-1, wr=-1):
    """The step [lo, hi) of one sequence without cache rows."""
    n = hi - lo
    return StepBatch(tokens=None, seq=None, pos=torch.arange(lo, hi, dtype=torch.int32, device=dev), slot=None, block_table=None, max_pos=hi - 1,
                     n_tokens=n, items=[(slot, 0, n)], run_off=torch.arange(n, dtype=torch.int32, device=dev),
                     state_rd=torch.full((n,), rd, dtype=torch.int32, device=dev),
                     state_wr=torch.tensor([-1] * (n - 1) + [wr], dtype=torch.int32, device=dev))


def cache_batch(cache, slot, lo, hi, dev):
    rows = cache.extend(slot, hi - lo)
    b = run_batch(lo, hi, dev, slot)
    b.seq = torch.full((hi - lo,), slot, dtype=torch.int32, device=dev)
    b.slot, b.block_table = torch.tensor(rows, dtype=torch.int64, device=dev), cache.block_table()
    return b


# ---- mechanisms alone ---------------------------------------------------------------------------------------------------------

def test_embedding_norm_and_norm_after_the_sum(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(0)
    for D in (7, 40, 300, 1024 + 36):
        table, w = torch.randn(11, D, generator=g) + 0.5, torch.randn(D, generator=g)
        toks = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32)
        x = ops.embed_rms_norm(toks.to(dev), table.to(dev), w.to(dev), 1e-2)
        want = P.rms(table.double().numpy()[toks.numpy()], 1e-2) * w.double().numpy()
        assert_close(x.double().cpu(), want, 2e-6, f"normed embedding, width {D}")
        y = torch.randn(5, D, generator=g) * 2 + 1.0                          # a mean far from zero: RMS, not a variance
        for alpha in (1.0, 2.75):
            xd = x.clone()
            h = ops.scaled_add_rms_norm(xd, y.to(dev), alpha, w.to(dev), 1e-2)
            new = P.rms(alpha * want + y.double().numpy(), 1e-2) * w.double().numpy()
            assert_close(xd.double().cpu(), new, 3e-6, f"norm after the sum, width {D}")
            assert torch.equal(h, xd)
            xd = x.clone()
            assert ops.scaled_add_rms_norm(xd, y.to(dev), alpha, w.to(dev), 1e-2, want_h=False) is None
            assert_close(xd.double().cpu(), new, 3e-6, "the sum alone")


def test_mixer_input_convolution_carries_its_last_rows(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(2)
    for D, taps, cuts in ((10, 3, [1, 2, 3, 9]), (72, 4, [5]), (40, 3, [1, 3, 20]), (12, 2, []), (1040, 4, [16]), (6, 2, [1, 2, 3]), (300, 5, [2, 3, 4, 30]), (12, 1, [4, 5]), (8, 6, [1, 2, 3, 4, 5, 6, 7])):
        T = 33
        x = torch.randn(T, D, generator=g)
        w = torch.randn(D, taps, generator=g)
        ref = x.double().numpy() + P.causal_conv(x.double().numpy(), w.double().numpy())
        cache = PagedCache([], 2, 3, torch.float32, dev, states=[StateSpec((taps - 1, D), copies=2)] if taps > 1 else [])
        hist = cache.states[0] if taps > 1 else None
        if taps > 1:
            hist.fill_(7.0)
        wt, slot, outs, lo = w.t().contiguous().to(dev), 1, [], 0
        for hi in cuts + [T]:
            rd, wr = cache.step_rows(slot)
            b = run_batch(lo, hi, dev, slot, rd if lo else -1, wr)
            outs.append(ops.residual_conv(x[lo:hi].contiguous().to(dev), wt, hist, b).cpu())
            lo = hi
        assert_close(torch.cat(outs).double(), ref, 3e-6, f"{taps} taps cut at {cuts}")
        # the form that rides in the norm's launch: token by token
        n2, y = torch.rand(D, generator=g) + 0.5, torch.randn(T, D, generator=g)
        new = P.rms(1.5 * x.double().numpy() + y.double().numpy(), 1e-5) * n2.double().numpy()
        ref = new + P.causal_conv(new, w.double().numpy())
        outs = []
        for t in range(T):
            rd, wr = cache.step_rows(2)
            b = run_batch(t, t + 1, dev, 2, rd if t else -1, wr)
            xd = x[t:t + 1].clone().to(dev)
            outs.append(ops.scaled_add_rms_norm(xd, y[t:t + 1].contiguous().to(dev), 1.5, n2.to(dev), 1e-5, then_conv=(wt, hist), batch=b).cpu())
            assert_close(xd.double().cpu(), new[t:t + 1], 3e-6, "the normed sum itself")
        assert_close(torch.cat(outs).double(), ref, 5e-6, f"{taps} taps behind the norm")


def test_rotation_in_halves_and_linear_frequency_scaling(backend):
    """q and k heads turn (all of a head or its first dimensions), values pass; every frequency divided by the factor; positions far
    from zero."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(1)
    pos = torch.tensor([0, 1, 63, 64, 700, 2], dtype=torch.int32)
    for H, d, dv, rot, base, factor in ((3, 10, 6, 6, 50.0, None), (2, 8, 4, 8, 1e6, 3.0), (5, 4, 9, 2, 100.0, 8.0)):
        u = torch.randn(6, H * (2 * d + dv) + 5, generator=g)
        table = RotaryTable(rot, base, {"factor": factor} if factor else None, dev, positions=701)
        b = run_batch(0, 6, dev)
        b.pos, b.max_pos = pos.to(dev), 700
        out = ops.rotate_qk(u.to(dev), H, d, dv, table.table, rot, b).double().cpu()
        qk = u[:, :2 * H * d].double().numpy().reshape(6, 2 * H, d)
        assert_close(out[:, :2 * H * d], P.rotate_halves(qk, pos.numpy(), rot, base, factor or 1.0).reshape(6, -1), 1e-5, "queries and keys")
        assert torch.equal(out[:, 2 * H * d:].float(), u[:, 2 * H * d:H * (2 * d + dv)])


def test_query_key_preparation_with_biases_head_scales_and_tied_values(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(3)
    pos = torch.tensor([5, 0, 64, 129, 1], dtype=torch.int32)
    for H, G, d, rot, pad, per_head in ((4, 2, 12, 8, 0, True), (6, 3, 8, 8, 3, True), (3, 1, 6, 2, 0, False)):
        T = 5
        proj = torch.randn(T, (H + G) * d + 3, generator=g)
        qb, kb = torch.randn(H * d, generator=g), torch.randn(G * d, generator=g)
        qw, kw = torch.randn(d if per_head else H * d, generator=g), torch.randn(d if per_head else G * d, generator=g)
        temp = torch.rand(H, generator=g) + 0.5
        table = RotaryTable(rot, 77.0, {"factor": 2.5}, dev, positions=130)
        cache = PagedCache([(G, 2 * d)], 4, 1, torch.float32, dev)
        b = cache_batch(cache, cache.admit(), 0, T, dev)
        b.pos, b.max_pos = pos.to(dev), 129
        pd = proj.to(dev)
        k = pd[:, H * d:(H + G) * d]
        qf = ops.qk_norm_rope_prep(pd[:, :H * d], k, k, H, G, d, d, qw.to(dev), kw.to(dev), per_head, 1e-4, table.table, rot, 0.6,
                                   cache.pools[0], b, q_b=qb.to(dev), k_b=kb.to(dev), v_b=kb.to(dev), halves=True, head_scale=temp.to(dev), q_pad=pad)

        def plain(u, w, n):
            u = P.rms(u.reshape(T, n, d), 1e-4) * w if per_head else (P.rms(u, 1e-4) * w).reshape(T, n, d)
            return torch.from_numpy(P.rotate_halves(u, pos.numpy(), rot, 77.0, 2.5))

        q64, k64 = proj[:, :H * d].double() + qb.double(), proj[:, H * d:(H + G) * d].double() + kb.double()
        assert qf.shape == (T, H, pad + d) and (pad == 0 or float(qf[..., :pad].abs().max()) == 0.0)
        assert_close(qf[..., pad:].double().cpu(), plain(q64.numpy(), qw.double().numpy(), H) * 0.6 * temp.double()[:, None], 1e-5, "queries")
        rows = cache.pools[0][:, b.slot].transpose(0, 1).double().cpu()
        assert_close(rows[..., d:], plain(k64.numpy(), kw.double().numpy(), G), 1e-5, "cached keys")
        assert_close(rows[..., :d], k64.view(T, G, d), 1e-6, "cached values: the biased projection, neither normed nor turned")


def _mixer_alone(backend, layer, T, splits, seed=3, width=24, tol=3e-5, dtype="float32", tweak=None):
    """One mixer through its layer object, the engine's cache and state, the tokens cut at `splits`, against the plain statement."""
    cfg = make_config([layer], width=width)
    W = P.random_weights(cfg, seed=seed)
    if tweak:
        tweak(W)
    eng = build_engine(cfg, f32(W) if dtype == "float32" else bf16(W), backend, dtype=dtype, max_tokens=max(256, T + 64), max_seqs=3)
    dev, st = eng.device, torch.float32 if dtype == "float32" else torch.bfloat16
    mixer = eng.model.layers[0]["mixer"]
    p0, p1, s0, s1 = eng.model.slices[0]
    g = torch.Generator().manual_seed(seed + 100)
    h = torch.randn(T, width, generator=g).bfloat16().float()
    ref = P.mixer(layer["type"], h.double().numpy(), W, "l0.mix.", layer["mixer"], cfg["norm"]["eps"])
    eng.open_sequence()                                                    # (not slot 0)
    slot = eng.open_sequence()
    for s in eng.cache.states:
        s.fill_(5.0)                                                       # stale state: a new sequence must not read it
    outs, lo = [], 0
    for hi in list(splits) + [T]:
        b = eng.layout([(slot, [0] * (hi - lo))])
        outs.append(mixer(h[lo:hi].to(st).to(dev), b, eng.cache.pools[p0:p1], eng.cache.states[s0:s1]).double().cpu())
        lo = hi
    got, ref = torch.cat(outs), torch.from_numpy(ref)
    if dtype == "float32":
        return assert_close(got, ref, tol, f"{layer['type']} cut at {splits}")
    # bfloat16: by root mean squares (a read-out that happens to be small is blown up by its norm, rounding and all)
    d, size = (got - ref).pow(2), ref.pow(2).mean().sqrt()
    assert d.mean().sqrt() < 0.01 * size and d.mean(-1).sqrt().max() < 0.1 * size, f"{layer['type']} cut at {splits}: {d.mean().sqrt() / size:.4f} "\
        f"overall, {d.mean(-1).sqrt().max() / size:.4f} in token {int(d.mean(-1).argmax())}"


def test_sloped_window_attention_alone(backend):
    _mixer_alone(backend, att(), 70, [])
    _mixer_alone(backend, att(), 70, [1, 3, 5, 23, 24, 25, 47, 48, 69])                               # cuts around the window's edge
    _mixer_alone(backend, att(heads=5, kv_heads=1, dim=6, size=64), 200, [63, 64, 65, 128, 129])       # window = page
    _mixer_alone(backend, att(heads=2, kv_heads=2, dim=16, size=1), 20, [1, 2, 7])                     # the token itself
    _mixer_alone(backend, att(heads=3, kv_heads=3, dim=4, size=300), 130, [39, 40, 41, 100])           # wider than the sequence


def test_retention_alone(backend):
    _mixer_alone(backend, ret(), 70, [])
    _mixer_alone(backend, ret(), 70, [1, 3, 5, 16, 17, 63, 64, 69])
    _mixer_alone(backend, ret(heads=2, dim=16, vdim=12, rot=16, base=1e5, decay=[1.0, 0.5]), 90, [2, 30, 31])     # a state that never fades
    _mixer_alone(backend, ret(heads=1, dim=4, vdim=40, rot=2, decay=[0.999]), 130, [64, 128, 129])
    _mixer_alone(backend, ret(heads=4, dim=70, vdim=5, rot=10), 40, [7])


def test_talking_heads_beside_the_delta_rule_alone(backend):
    _mixer_alone(backend, par(), 70, [])
    _mixer_alone(backend, par(), 70, [1, 2, 3, 4, 5, 6, 31, 32, 33, 63, 64, 65, 69])
    _mixer_alone(backend, par(heads=4, kv_heads=4, dim=10, rot=10, cap=2.0, factor=None, d_heads=1, d_kv=1, d_dim=5, d_vdim=7, conv=1), 90, [3, 4, 80])
    _mixer_alone(backend, par(heads=5, kv_heads=1, dim=4, rot=2, cap=60.0, d_heads=6, d_kv=2, d_dim=12, d_vdim=4, conv=3), 140, [2, 64, 65, 66, 130])
    _mixer_alone(backend, par(heads=1, kv_heads=1, dim=2, rot=2, cap=None), 20, [9])


@pytest.mark.gpu
def test_mixers_on_the_matrix_cores():
    """bfloat16 storage with sizes the matrix-core kernels take: prompt tiles and single tokens, several row groups, head groups beyond 16,
    values cut over workgroups, key splits; soft caps below and above the one that bounds the scores without a running maximum."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    for layer, T, splits in ((att(heads=4, kv_heads=2, dim=16, size=88), 300, [87, 88, 89, 126, 170, 298, 299]),
                             (att(heads=3, kv_heads=1, dim=40, size=33), 420, [399, 400, 401, 419]),
                             (par(heads=8, kv_heads=4, dim=16, rot=8), 330, [43, 44, 53, 54, 126, 170, 328, 329]),
                             (par(heads=6, kv_heads=2, dim=24, rot=24, cap=55.0), 300, [200, 201, 203, 290] + list(range(292, 300))),
                             (par(heads=20, kv_heads=1, dim=8, rot=4, cap=None), 150, [100, 101, 102, 140]),
                             (par(heads=12, kv_heads=12, dim=40, rot=8), 140, [64, 65, 130] + list(range(132, 140))),
                             (par(heads=4, kv_heads=2, dim=264, rot=64), 100, [50, 51, 97, 98, 99]),
                             (par(heads=3, kv_heads=3, dim=12, rot=4), 90, [50, 51, 88])):          # dim % 8 != 0: the wave kernel
        _mixer_alone("hip", layer, T, splits, dtype="bfloat16", width=32)


def _talking_case(g, H, G, d, L, dev, dtype):
    page, npages = 64, (L + 63) // 64
    cache = PagedCache([(G, 2 * d)], npages + 3, 2, dtype, dev, page=page)
    cache.free_pages = torch.randperm(npages + 3, generator=g).tolist()     # pages out of order, not the first ones
    cache.admit()
    slot = cache.admit()
    k, v = (torch.randn(L, G, d, generator=g).bfloat16().double() for _ in range(2))
    b = cache_batch(cache, slot, 0, L, dev)
    cache.pools[0][:, b.slot] = torch.cat([v, k], dim=-1).transpose(0, 1).to(dtype).to(dev)
    return cache, slot, k, v


@pytest.mark.parametrize("dtype,tol", STORAGE)
def test_talking_attention_forms(backend, dtype, tol):
    """The operation alone: last tokens of a sequence as one batch, several launch forms, windows, caps, with and without the gate."""
    dev = device_of(backend)
    ops = make_ops(backend, dtype, dev)
    g = torch.Generator().manual_seed(4)
    for H, G, d, L, nq, cap, window, gated in ((8, 4, 16, 200, 1, 3.0, None, True), (8, 4, 16, 200, 37, 3.0, None, True), (6, 2, 8, 300, 5, 0.0, 70, False),
                                               (6, 6, 48, 130, 66, 45.0, None, True), (4, 1, 64, 520, 1, 20.0, None, True), (18, 1, 8, 90, 3, 1.0, 33, True),
                                               (32, 8, 128, 200, 20, 30.0, None, True), (16, 4, 128, 170, 33, 0.0, None, True),
                                               (12, 6, 72, 300, 18, 60.0, 100, False), (32, 32, 16, 140, 17, 2.0, None, True), (21, 7, 40, 97, 16, 8.0, None, True)):
        cache, slot, k, v = _talking_case(g, H, G, d, L, dev, dtype)
        q = torch.randn(nq, H, d, generator=g).bfloat16().double()
        talk, gate = torch.randn(H, H, generator=g).bfloat16().double(), torch.randn(nq, H, generator=g).bfloat16().double()
        ref = torch.empty(nq, H, d, dtype=torch.float64)
        for i in range(nq):
            p = L - nq + i
            lo = max(0, p - window + 1) if window else 0
            s = torch.stack([k[lo:p + 1, h // (H // G)] @ q[i, h] for h in range(H)])
            w = talk @ torch.softmax(cap * torch.tanh(s / cap) if cap else s, dim=-1)
            ref[i] = torch.stack([w[h] @ v[lo:p + 1, h // (H // G)] for h in range(H)])
        if gated:
            ref = ref * torch.sigmoid(gate)[:, :, None]
        b = run_batch(L - nq, L, dev, slot)
        b.seq, b.block_table = torch.full((nq,), slot, dtype=torch.int32, device=dev), cache.block_table()
        forms = [dict(), dict(variant=1)]
        if backend == "hip":
            forms += [dict(key_splits=s, decode=m) for s in (1, 2, 5) for m in (False, True)] + [dict(variant=2, key_splits=s, decode=m) for s in (1, 3) for m in (False, True)]
        for kw in forms:
            out = ops.talking_attention(q.float().to(dev), cache.pools[0], b, talk.to(dtype).to(dev), gate.to(dtype).to(dev) if gated else None,
                                        d, 64, cap=cap, window=window, **kw)
            assert_close(out.double().cpu(), ref.reshape(nq, H * d), tol, f"{H} heads over {G}, {nq} tokens, cap {cap}, window {window}, {kw}")


def test_delta_rule_with_one_decay_per_head_and_a_straight_gate(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(6)
    for H, G, d, dv, taps, D, T, cuts in ((4, 2, 6, 10, 3, 20, 50, [1, 2, 3, 17, 49]), (3, 1, 16, 4, 1, 12, 33, [32]), (2, 2, 1, 5, 2, 9, 12, [4])):
        w = {n: torch.randn(s, generator=g).double() / math.sqrt(s[-1]) for n, s in (
            ("q", (G * d, D)), ("k", (G * d, D)), ("v", (H * dv, D)), ("q_conv", (G * d, taps)), ("k_conv", (G * d, taps)), ("v_conv", (H * dv, taps)),
            ("b", (H, D)), ("a", (H, D)), ("g", (H * dv, D)), ("o", (D, H * dv)))}
        w.update(A_log=torch.randn(H, generator=g).double(), dt_bias=torch.randn(H, generator=g).double(), norm=torch.rand(dv, generator=g).double() + 0.5)
        h = torch.randn(T, D, generator=g)
        ref = P.right_mixer(h.double().numpy(), {k: v.numpy() for k, v in w.items()}, {"heads": H, "kv_heads": G, "dim": d, "vdim": dv}, 1e-5)
        layer = GatedDeltaRule(ops, heads=H, kv_heads=G, dim=d, vdim=dv, taps=taps, eps=1e-5, gate="silu",
                               weights={k: v.float().to(dev) for k, v in w.items()})
        cache = PagedCache([], 2, 3, torch.float32, dev, states=layer.state_specs)
        for s in cache.states:
            s.fill_(9.0)
        slot, outs, lo = 2, [], 0
        for hi in cuts + [T]:
            rd, wr = cache.step_rows(slot)
            outs.append(layer(h[lo:hi].to(dev), run_batch(lo, hi, dev, slot, rd if lo else -1, wr), [], cache.states).double().cpu())
            lo = hi
        assert_close(torch.cat(outs), ref, 3e-5, f"{H} heads over {G} cut at {cuts}")
        assert float(cache.states[0][:2].min()) == 9.0                     # other slots' states are not touched


def test_retention_keeps_an_old_token_by_its_decay(backend):
    """One loud token, then silence: after n more tokens the read-out is decay^n of it, per head, over portions and single tokens."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    H, d, dv, T = 3, 4, 4, 300
    decay = [0.9995, 0.97, 1.0]
    qkv = torch.zeros(T, H, 2 * d + dv)
    q, k, v = torch.zeros(T, H, d), torch.zeros(T, H, d), torch.zeros(T, H, dv)
    q[..., 0], k[0, :, 0] = 1.0, 2.0
    v[0] = torch.tensor([3.0, -1.0, 0.5, 4.0])
    state = torch.full((2, H, d, dv), 4.0, device=dev)
    outs, lo = [], 0
    dec = torch.tensor(decay, device=dev)
    for hi in (1, 2, 3, 200, 299, T):
        f = [t[lo:hi].reshape(hi - lo, -1).contiguous().to(dev) for t in (q, k, v)]
        outs.append(ops.recurrent_scan(*f, dec, None, state, run_batch(lo, hi, dev, 1), H, H, d, dv, 0.5).double().cpu())
        lo = hi
    out = torch.cat(outs)
    want = torch.stack([torch.tensor([dc ** t for dc in decay], dtype=torch.float64)[:, None] * v[0].double() for t in range(T)])
    assert_close(out, want, 2e-5, "decayed read-out")
    assert float(state[0].min()) == 4.0 and qkv.numel() > 0


def test_clamped_feed_forward_alone(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(2)
    h = torch.randn(9, 24, generator=g) * 3
    gate, up, down = (torch.randn(s, generator=g).double() / 4 for s in ((14, 24), (14, 24), (24, 14)))
    for limit in (0.3, 1.0, 7.0):
        layer = GatedFeedForward(ops, gate=gate.float().to(dev), up=up.float().to(dev), down=down.float().to(dev), act="clamped", limit=limit)
        ref = P.clamped_ff(h.double().numpy(), gate.numpy(), up.numpy(), down.numpy(), limit)
        assert_close(layer(h.to(dev)).double().cpu(), ref, 2e-5, f"limit {limit}")
    with pytest.raises(ValueError):
        GatedFeedForward(ops, gate=gate.float(), up=up.float(), down=down.float(), act="clamped")


# ---- keys that stand out: window edges, page borders, far keys heard through another head, the sink ------------------------------------

def _selector(backend, L, dtype, nq, *, spike=None, size=50, sink=-30.0, cuts=(), scale=6.0):
    """Sloped attention alone with selector weights: the layer input IS [q | k], values are the keys.  All keys point off the queries'
    direction but the one at `spike`.  -> (layer output of the last nq positions, plain statement, the keys)."""
    H, G, d = 2, 1, 8
    D = H * d + d
    eye = np.eye(D)
    W = {"q": eye[:16], "k": eye[16:], "o": np.ascontiguousarray(eye[:, :16]), "sink": np.full(H, float(sink)), "q_norm": np.ones(8), "k_norm": np.ones(8)}
    g = torch.Generator().manual_seed((spike or 0) * 7 + L)
    h = (torch.randn(L, D, generator=g) * 0.05).bfloat16().double()
    h[:, 16:23] = torch.randn(L, 7, generator=g).bfloat16().double()        # the values differ from token to token ...
    h[:, 7] = 2.0
    h[:, 8 + 7] = 2.0
    if spike is not None:
        h[spike, 16 + 7] = 24.0                                             # ... one points along the queries
    hn = h.numpy()
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "scale": scale, "mask": {"size": size}}
    ref = P.attention_mixer(hn, W, m, 1e-5)
    dev = device_of(backend)
    ops = make_ops(backend, dtype, dev)
    page, npages = 64, (L + 63) // 64
    layer = SinkWindowAttention(ops, heads=H, kv_heads=G, dim=d, vdim=d, scale=scale, eps=1e-5, window=size, tied_values=True,
                                slopes=distance_slopes(H), weights={k: torch.from_numpy(v).to(dtype).to(dev) for k, v in W.items()})
    cache = PagedCache(layer.cache_rows, npages + 3, 2, dtype, dev, page=page)
    cache.free_pages = torch.randperm(npages + 3, generator=g).tolist()     # pages out of order, not the first ones
    cache.admit()
    slot = cache.admit()
    out, lo = None, 0
    for hi in list(cuts) + [L - nq, L]:
        if hi <= lo:
            continue
        b = cache_batch(cache, slot, lo, hi, dev)
        out = layer(h[lo:hi].to(dtype).to(dev), b, cache.pools, [])
        lo = hi
    return out.double().cpu(), torch.from_numpy(ref[L - nq:]), h[:, 16:]


@pytest.mark.parametrize("dtype,tol", STORAGE)
@pytest.mark.parametrize("nq", [1, 20], ids=["decoded", "prompt"])
def test_window_edges_stand_out(backend, nq, dtype, tol):
    """A window of 50, a sequence of 330: the last query sees [280, 330).  A loud key just inside (280, 281) carries head 1's output (its
    slope is 2^-8) and must not be heard at 279, 278 or far back; with 20 queries in the step the later ones' windows start past the
    first key tile."""
    L, size = 330, 50
    for spike in (0, 63, 64, 278, 279, 280, 281, 319, 320, L - 1):
        out, ref, v = _selector(backend, L, dtype, nq, spike=spike, size=size)
        heard = (ref[-1, 8:16] - v[spike]).abs().max() < 0.25 * v[spike].abs().max()
        assert bool(heard) == (spike >= L - size), f"the key at {spike}"
        assert_close(out, ref, tol, f"spike at {spike}")
    for L2, spike, cuts in ((68, 17, (30,)), (69, 19, ()), (130, 80, (64, 100)), (200, 150, (128, 150, 190)), (51, 0, ()), (52, 2, (2,)), (50, 0, (3,))):
        out, ref, _ = _selector(backend, L2, dtype, min(nq, 7), spike=spike, size=size, cuts=cuts)
        assert_close(out, ref, tol, f"length {L2}, spike at {spike}")


@pytest.mark.parametrize("dtype,tol", STORAGE)
def test_distance_slopes_against_the_sink(backend, dtype, tol):
    """With a sink the bias is slope (i - j), not slope * j: both heads' outputs shrink with the distance of the only loud key.  A sink well
    above every score takes most of the weight, one far below changes nothing."""
    for sink, scale, kw in ((4.0, 2.0, dict(spike=60)), (4.0, 2.0, dict(spike=100)), (8.0, 0.5, {}), (-30.0, 6.0, {}), (0.0, 1.0, {})):
        for L, nq in ((1, 1), (3, 3), (140, 1), (140, 9)):
            if kw.get("spike", 0) >= L:
                continue
            out, ref, v = _selector(backend, L, dtype, nq, sink=sink, scale=scale, size=100, **kw)
            assert_close(out, ref, tol, f"sink {sink}, length {L}, {kw}")
            if sink == 8.0 and L == 1:
                assert ref.abs().max() < 0.3 * v[0].abs().max()
            if sink == -30.0 and L == 1:
                assert (ref[0, :8] - v[0]).abs().max() < 1e-6


@pytest.mark.parametrize("dtype,tol", STORAGE)
@pytest.mark.parametrize("nq", [1, 20], ids=["decoded", "prompt"])
def test_a_far_key_is_heard_through_another_head(backend, nq, dtype, tol):
    """Head 0's query points at one loud key (first tokens, page borders, far back); the talk matrix routes head 0's weights to head 3,
    which holds another key / value head: head 3 returns ITS pool's value at the loud position, head 0 nothing."""
    dev = device_of(backend)
    ops = make_ops(backend, dtype, dev)
    H, G, d, L = 4, 2, 8, 340
    talk = torch.zeros(H, H)
    talk[3, 0], talk[1, 2], talk[2, 1] = 1.0, -1.0, 0.5
    for spike in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 318, 319):
        g = torch.Generator().manual_seed(spike)
        cache, slot, k, v = _talking_case(g, H, G, d, L, dev, dtype)
        k[:, :, 7] = 0.0
        k[spike, 0, 7] = 6.0
        rows = cache.pages[slot]
        at = torch.tensor([rows[j // 64] * 64 + j % 64 for j in range(L)], device=dev)
        cache.pools[0][:, at] = torch.cat([v, k], dim=-1).transpose(0, 1).to(dtype).to(dev)
        q = (torch.randn(nq, H, d, generator=g) * 0.2).bfloat16().double()
        q[:, 0, 7] = 4.0
        ref = torch.empty(nq, H, d, dtype=torch.float64)
        for i in range(nq):
            p = L - nq + i
            s = torch.stack([k[:p + 1, h // 2] @ q[i, h] for h in range(H)])
            w = talk.double() @ torch.softmax(30.0 * torch.tanh(s / 30.0), dim=-1)
            ref[i] = torch.stack([w[h] @ v[:p + 1, h // 2] for h in range(H)])
        assert (ref[-1, 3] - v[spike, 1]).abs().max() < 0.05 and float(ref[:, 0].abs().max()) == 0.0
        b = run_batch(L - nq, L, dev, slot)
        b.seq, b.block_table = torch.full((nq,), slot, dtype=torch.int32, device=dev), cache.block_table()
        out = ops.talking_attention(q.float().to(dev), cache.pools[0], b, talk.to(dtype).to(dev), None, d, 64, cap=30.0)
        assert_close(out.double().cpu(), ref.reshape(nq, H * d), tol, f"loud key at {spike}")


def test_the_soft_cap_bounds_loud_scores(backend):
    """Scores of +-400 under a cap of 4 weigh e^(+-4), not everything or nothing; the same with a cap above the bound that serves as the
    maximum."""
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        dev = device_of(backend)
        ops = make_ops(backend, dtype, dev)
        g = torch.Generator().manual_seed(8)
        for cap in (4.0, 41.0):
            cache, slot, k, v = _talking_case(g, 2, 1, 8, 70, dev, dtype)
            q = torch.zeros(1, 2, 8, dtype=torch.float64)
            q[0, 0, 0], q[0, 1, 0] = 400.0, -400.0
            s = torch.stack([k[:, 0] @ q[0, h] for h in range(2)])
            ref = torch.softmax(cap * torch.tanh(s / cap), dim=-1) @ v[:, 0]
            b = run_batch(69, 70, dev, slot)
            b.seq, b.block_table = torch.full((1,), slot, dtype=torch.int32, device=dev), cache.block_table()
            out = ops.talking_attention(q.float().to(dev), cache.pools[0], b, torch.eye(2).to(dtype).to(dev), None, 8, 64, cap=cap)
            assert_close(out.double().cpu().view(2, 8), ref, tol, f"cap {cap}")


# ---- the whole model ---------------------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def std():
    cfg = standard_config()
    W = P.random_weights(cfg, seed=1)
    seqs = {"a": tokens_for(cfg, 150, 1), "b": tokens_for(cfg, 37, 2), "c": tokens_for(cfg, 1, 3), "d": tokens_for(cfg, 81, 4)}
    ref, layers = {}, {}
    for k, v in seqs.items():
        taps = []
        ref[k] = plain_logits(cfg, W, v, taps)
        layers[k] = [torch.from_numpy(t) for t in taps]
    return cfg, W, seqs, ref, layers


def test_layers_one_by_one(backend, std):
    cfg, W, seqs, _, layers = std
    eng = build_engine(cfg, f32(W), backend)
    slot = eng.open_sequence()
    b = eng.layout([(slot, seqs["d"])])
    seen = []
    eng.model.forward(b, eng.cache.pools, states=eng.cache.states, tap=lambda i, x: seen.append(x.double().cpu().clone()))
    assert len(seen) == len(cfg["layers"])
    for i, x in enumerate(seen):
        assert_close(x, layers["d"][i], F32_TOL, f"residual stream after layer {i}")


def test_whole_prompts(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    for k in seqs:
        got = run_schedule(eng, seqs, [[(k, len(seqs[k]))]])
        assert_close(got[k], ref[k], F32_TOL, f"whole prompt {k}")


def test_prefill_then_token_by_token(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    for k, first in (("a", 60), ("b", 1), ("d", 64)):
        n = len(seqs[k])
        got = run_schedule(eng, seqs, [[(k, first)]] + [[(k, 1)]] * (n - first))
        assert_close(got[k], ref[k], F32_TOL, f"{k}: {first} tokens, then one by one")


def test_portions_of_several_sizes(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    for sizes in ([2] * 75, [64, 64, 22], [63, 2, 2, 61, 22], [3, 1, 1, 2, 5, 7, 45, 64, 1, 19, 2], [149, 1], [20, 13, 7, 26, 33, 51]):
        assert sum(sizes) == 150
        got = run_schedule(eng, seqs, [[("a", s)] for s in sizes])
        assert_close(got["a"], ref["a"], F32_TOL, f"portions {sizes[:6]}...")


def test_unequal_batches_match_each_alone(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    steps = [[("a", 29), ("b", 2), ("c", 1)],
             [("a", 64), ("b", 1), ("d", 17)],
             [("b", 30), ("d", 1), ("a", 2)],
             [("d", 63), ("a", 1), ("b", 1)]]
    steps += [[("a", 1), ("b", 1)]] * 3 + [[("a", 1)]] * 51
    got = run_schedule(eng, seqs, steps)
    for k in seqs:
        assert_close(got[k], ref[k], F32_TOL, f"mixed batch, sequence {k}")


def test_a_sequence_left_out_of_steps_goes_on_later(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    steps = [[("b", 10), ("d", 3)], [("d", 2)], [("d", 1)], [("b", 1), ("d", 1)], [("d", 70)], [("b", 26), ("d", 4)]]
    got = run_schedule(eng, seqs, steps)
    for k in ("b", "d"):
        assert_close(got[k], ref[k], F32_TOL, f"sequence {k}")


def test_pages_slots_and_states_are_used_again(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend, max_tokens=256, max_seqs=2)          # 4 pages, 2 slots: a (3 pages) + one more
    assert eng.cache.num_pages == 4
    seen_pages = []
    for rnd in range(3):
        order = [("a", "b"), ("d", "b"), ("b", "a")][rnd]
        steps = [[(order[0], 30), (order[1], 5)], [(order[0], len(seqs[order[0]]) - 30), (order[1], len(seqs[order[1]]) - 5)]]
        got = run_schedule(eng, seqs, steps)
        for k in order:
            assert_close(got[k], ref[k], F32_TOL, f"pass {rnd}, sequence {k}")
        assert len(eng.cache.free_pages) == 4 and len(eng.cache.free_slots) == 2
        seen_pages.append(tuple(eng.cache.free_pages))
        assert all(float(s.abs().max()) > 0 for s in eng.cache.states)            # the slots' states are left as they were: stale
        assert all(float(p.abs().max()) > 0 for p in eng.cache.pools)
    assert len(set(seen_pages)) > 1
    s0, s1 = eng.open_sequence(), eng.open_sequence()
    with pytest.raises(CacheFull):
        eng.open_sequence()
    eng.close_sequence(s0)
    eng.close_sequence(s1)


def test_first_tokens_and_single_token_sequences(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, f32(W), backend)
    got = run_schedule(eng, seqs, [[("c", 1)]])
    assert_close(got["c"], ref["c"], F32_TOL)
    got = run_schedule(eng, seqs, [[("b", 1)], [("b", 1)], [("b", 2)], [("b", 33)]])
    assert_close(got["b"][:4], ref["b"][:4], F32_TOL, "first tokens")


def test_long_decoding(backend):
    cfg = make_config([par(mlp=dense(12)), att(size=50, mlp=None), ret(mlp=dense(9, 1.5)), att(size=8, mlp=dense(8))], width=32, vocab=29, taps=3)
    W = P.random_weights(cfg, seed=9)
    toks = tokens_for(cfg, 210, 5)
    ref = plain_logits(cfg, W, toks)
    eng = build_engine(cfg, f32(W), backend, max_tokens=256, max_seqs=1)
    got = run_schedule(eng, {"s": toks}, [[("s", 3)]] + [[("s", 1)]] * 207)      # decoded tokens pass window edges and three page borders
    assert_close(got["s"], ref, F32_TOL, "207 decoded tokens")


@pytest.mark.parametrize("variant", range(5))
def test_other_sizes(backend, variant):
    layers, kw = [
        ([par(heads=1, kv_heads=1, dim=2, rot=2, d_heads=1, d_kv=1, d_dim=1, d_vdim=1, conv=1, mlp=dense(1))], dict(width=8, vocab=5, eps=1e-3, taps=1)),
        ([att(heads=6, kv_heads=3, dim=16, size=31, mlp=dense(33, 0.2)), par(heads=4, kv_heads=4, dim=32, rot=32, cap=1.0, d_heads=4, d_kv=4, d_dim=16,
                                                                           d_vdim=16, conv=5, mlp=dense(100)),
          ret(heads=1, dim=32, vdim=24, rot=32, mlp=None)], dict(width=96, vocab=200, taps=2, alpha=1.0)),
        ([ret(heads=7, dim=4, vdim=3, rot=2), par(heads=7, kv_heads=1, dim=70, rot=10, cap=100.0, factor=16.0, d_heads=5, d_kv=1, d_dim=3, d_vdim=20, conv=3)],
         dict(width=41, vocab=33, eps=1e-6, taps=5, alpha=6.0)),
        ([att(heads=1, kv_heads=1, size=5, mlp=dense(8))] * 3, dict(width=48, vocab=61, taps=3)),
        ([ret(mlp=None)], dict(width=20, vocab=9, taps=3, alpha=0.5)),
    ][variant]
    cfg = make_config(layers, **kw)
    W = P.random_weights(cfg, seed=20 + variant)
    toks = tokens_for(cfg, 75, variant)
    ref = plain_logits(cfg, W, toks)
    eng = build_engine(cfg, f32(W), backend)
    got = run_schedule(eng, {"s": toks}, [[("s", 40)], [("s", 30)]] + [[("s", 1)]] * 5)
    assert_close(got["s"], ref, F32_TOL, f"sizes variant {variant}")


def test_bfloat16_storage_stays_near_the_plain_statement(backend, std):
    cfg, W, seqs, ref, _ = std
    eng = build_engine(cfg, bf16(W), backend, dtype="bfloat16")
    got = run_schedule(eng, seqs, [[("a", 70), ("b", 37)], [("a", 80)]])
    for k in ("a", "b"):
        d = got[k] - ref[k]
        rel = (d - d.mean(-1, keepdim=True)).pow(2).mean().sqrt() / ref[k].std()
        assert rel < 0.05, f"bfloat16 run of {k}: relative error {rel:.3f}"
    got2 = run_schedule(eng, seqs, [[("a", 3)], [("a", 147)]])                      # cut differently: the same up to rounding
    rel = (got2["a"] - got["a"]).pow(2).mean().sqrt() / ref["a"].std()
    assert rel < 0.05


def test_key_value_heads_default_to_the_query_heads_and_values_are_tied(backend):
    cfg = make_config([par(heads=3, kv_heads=3, dim=6, rot=2, d_heads=2, d_kv=2), att(heads=2, kv_heads=2)])
    W = P.random_weights(cfg, seed=5)
    toks = tokens_for(cfg, 20, 1)
    ref = plain_logits(cfg, W, toks)
    short = json.loads(json.dumps(cfg))
    del short["layers"][0]["mixer"]["left"]["kv_heads"], short["layers"][0]["mixer"]["right"]["kv_heads"], short["layers"][1]["mixer"]["kv_heads"]
    got = run_schedule(build_engine(short, f32(W), backend), {"s": toks}, [[("s", 20)]])
    assert_close(got["s"], ref, F32_TOL)
    ops = make_ops("unfused", torch.float32, "cpu")
    for edit in (lambda c: c["layers"][1]["mixer"].update(vdim=4), lambda c: c["layers"][0].update(type="unknown"),
                 lambda c: c["canon"].update(taps=3), lambda c: c["canon"].update(taps=0)):
        bad = json.loads(json.dumps(cfg))
        edit(bad)
        with pytest.raises(ValueError):
            Sagupel.from_config(bad, f32(W), ops, "cpu", torch.float32)
    with pytest.raises(KeyError):
        Sagupel.from_config(cfg, {k: v for k, v in f32(W).items() if k != "l0.mix.left.talk"}, ops, "cpu", torch.float32)
    with pytest.raises(ValueError):
        Retention(ops, heads=2, dim=4, vdim=4, decay=[0.5], rotary=None, eps=1e-5,
                  weights={k: torch.zeros(s) for k, s in (("q", (8, 5)), ("k", (8, 5)), ("v", (8, 5)), ("g", (8, 5)), ("o", (5, 8)))})


# ---- generation through the engine's own entry point and scheduler ---------------------------------------------------------------

def plain_greedy(cfg, W, prompt, n):
    toks, margins = list(prompt), []
    for _ in range(n):
        lg = plain_logits(cfg, W, toks)[-1]
        top2 = lg.topk(2).values
        margins.append(float(top2[0] - top2[1]))
        toks.append(int(lg.argmax()))
    return toks[len(prompt):], margins


def test_greedy_generation_through_the_scheduler(backend, std):
    cfg, W, _, _, _ = std
    prompts = [tokens_for(cfg, n, 40 + n) for n in (5, 70, 1, 33, 12, 64)]
    eng = build_engine(cfg, f32(W), backend, max_tokens=512, max_seqs=3, max_batch_tokens=48, prefill_chunk=20)
    outs = eng.generate(prompts, SamplingParams(max_new=6))
    assert not eng.has_work() and len(eng.cache.free_pages) == eng.cache.num_pages and len(eng.cache.free_slots) == 3
    for p, o in zip(prompts, outs):
        ref, margins = plain_greedy(cfg, W, p, 6)
        for i, (a, b) in enumerate(zip(o, ref)):
            if a != b:
                assert margins[i] < 1e-3, f"prompt of {len(p)}: token {i} is {a}, plain statement {b} (margin {margins[i]:.2e})"
                break
        else:
            assert len(o) == 6


def _save_model(tmp_path, cfg, W):
    from safetensors.torch import save_file
    with open(tmp_path / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in bf16(W).items()}, str(tmp_path / "model.safetensors"))


def test_registry_and_checkpoint_directory(tmp_path, backend, std):
    from qserve_amd.serving import registry
    assert registry.architectures()["Sagupel"] == "paged"
    cfg, W, seqs, ref, _ = std
    _save_model(tmp_path, cfg, W)
    eng = Engine.from_pretrained(str(tmp_path), dtype="float32", device=device_of(backend), max_tokens=128, backend=backend)
    got = run_schedule(eng, seqs, [[("b", 37)]])
    assert_close(got["b"], ref["b"], F32_TOL)


# ---- GPU only ---------------------------------------------------------------------------------------------------------------------

@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_command(tmp_path, dtype, std):
    """bin/trace_run on a checkpoint directory: portions, single tokens, a mixed batch, a sequence ended and its slot used again."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg, W, seqs, ref, _ = std
    _save_model(tmp_path, cfg, W)
    out = tmp_path / "out"
    a, b, d = seqs["a"], seqs["b"], seqs["d"]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:70], "want": [0, 69]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [34]}, {"id": "a", "tokens": a[70:71], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[71:], "want": [78]}, {"id": "d", "tokens": d, "want": [80]}], "end": ["a", "d"]},
             {"step": 3, "entries": [{"id": "e", "tokens": b, "want": [36]}], "end": ["e"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "320"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                       timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    V = cfg["vocab"]
    want = {0: [ref["a"][0], ref["a"][69]], 1: [ref["b"][36], ref["a"][70]], 2: [ref["a"][149], ref["d"][80]], 3: [ref["b"][36]]}
    for i, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V).astype(np.float64))
        assert got.shape[0] == len(rows)
        for g_, r_ in zip(got, rows):
            if dtype == "float32":
                assert_close(g_, r_, F32_TOL, f"step {i}")
            else:
                assert ((g_ - r_).pow(2).mean().sqrt() / r_.std()) < 0.05


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_steps_from_a_graph_match_eager_steps(dtype, std):
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg, W, seqs, _, _ = std
    outs = []
    for graphs in (False, True):
        eng = build_engine(cfg, f32(W) if dtype == "float32" else bf16(W), "hip", dtype=dtype, max_tokens=512, max_seqs=2, decode_graphs=graphs)
        steps = [[("a", 100), ("b", 30)]] + [[("a", 1), ("b", 1)]] * 7 + [[("a", 1)]] * 43
        outs.append(run_schedule(eng, seqs, steps))
        if graphs:
            assert any(g for g in eng._graphs.values()), "no decode step was replayed from a graph"
    for k in ("a", "b"):
        assert_close(outs[1][k], outs[0][k], 1e-5 if dtype == "float32" else 2e-2, f"graph replay, sequence {k}")
