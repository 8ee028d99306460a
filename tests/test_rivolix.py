"""The Rivolix model and its mechanisms through the serving engine against the plain float64 statement (tests/_rivolix_plain.py).

Every test runs with the unfused tensor-op backend on the CPU (host logic: pages, state rows, runs, the layers' composition) and,
marked `gpu`, with the HIP kernels.  Configurations and weights are made here: small, random, sizes unlike each other so that a mixed-up
dimension shows; where random weights would hide a fault (one key among hundreds, a map that is left out, a lost convolution state, a weight
on the wrong side of an expert) the weights or inputs are made so that it shows.
"""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

import _rivolix_plain as P
from qserve_amd.layers.moe import CorrectedSigmoidMoE, GatedFeedForward, SigmoidMoE
from qserve_amd.layers.ops import make_ops
from qserve_amd.layers.rotary import RotaryTable
from qserve_amd.models.rivolix import Rivolix
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


def diff(heads=6, kv_heads=2, dim=10, vdim=14, conv=3, lam=0.4, coef=0.3, every=17, scale=None, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "diff": lam, "scale": scale if scale is not None else 1.3 / math.sqrt(dim)}
    if coef is not None:
        m["q_temp"] = {"coef": coef, "every": every}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def tied(heads=6, kv_heads=3, dim=12, rot=8, base=3000.0, factor=4.0, original=64, fast=8.0, slow=0.5, scale=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": rot}, "scale": scale if scale is not None else 2.0 / math.sqrt(dim)}
    if factor is not None:
        m["rot"]["scaling"] = {"factor": factor, "fast": fast, "original": original, "slow": slow}
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def moe(experts=5, top=2, ff=11, shared=7):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, **({"shared": {"ff": shared}} if shared else {})}


def make_config(layers, width=36, vocab=53, eps=1e-5):
    return {"architecture": "Rivolix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def standard_config():
    return make_config([diff(mlp=moe()), tied(mlp=moe(4, 1, 20, None)), diff(heads=4, kv_heads=2, kv_from=0, conv=2, lam=0.2, mlp=moe(3, 3, 8, 24)),
                        diff(heads=2, kv_heads=2, dim=6, vdim=5, conv=5, coef=None, mlp=None), tied(heads=4, kv_heads=1, dim=8, rot=8, factor=None, mlp=moe()),
                        diff(heads=2, kv_heads=2, dim=6, vdim=5, conv=1, kv_from=3, every=64, mlp=moe(7, 2, 6, 6)), tied(heads=3, kv_heads=3, dim=10, rot=2, mlp=None)])


def t64(W):
    return {k: torch.from_numpy(np.asarray(v)) for k, v in W.items()}


def f32(W):
    return {k: v.float() for k, v in t64(W).items()}


def bf16(W):
    return {k: v.bfloat16() for k, v in t64(W).items()}


def build_engine(cfg, W, backend, dtype="float32", max_tokens=1024, max_seqs=4, **kw):
    return Engine(Rivolix, cfg, W, dtype=dtype, device=device_of(backend), max_tokens=max_tokens, max_seqs=max_seqs, backend=backend, **kw)


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


def assert_near(got, ref, what="", overall=0.012, worst=0.12):
    """bfloat16: by root mean squares (a head's output that happens to be small is blown up by its norm, rounding and all)."""
    ref = torch.as_tensor(ref)
    d, size = (got - ref).pow(2), ref.pow(2).mean().sqrt()
    assert d.mean().sqrt() < overall * size and d.mean(-1).sqrt().max() < worst * size, \
        f"{what}: {d.mean().sqrt() / size:.4f} overall, {d.mean(-1).sqrt().max() / size:.4f} in row {int(d.mean(-1).argmax())}"


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
    rd, wr = cache.step_rows(slot)
    b = run_batch(lo, hi, dev, slot, rd if lo else -1, wr)
    b.seq = torch.full((hi - lo,), slot, dtype=torch.int32, device=dev)
    b.slot, b.block_table = torch.tensor(rows, dtype=torch.int64, device=dev), cache.block_table()
    return b


# ---- mechanisms alone ---------------------------------------------------------------------------------------------------------

def test_scaled_sum_with_two_norms(backend):
    """One statistic, two gains around one; up to three scaled outputs; the embedding as a start; the sum alone."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(0)
    for D in (7, 40, 300, 1024 + 36):
        table = torch.randn(11, D, generator=g) + 0.5                          # a mean far from zero: RMS, not a variance
        w1, w2 = (torch.randn(D, generator=g) * 0.3 for _ in range(2))
        toks = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32)
        gains = [(1.0 + w).to(dev) for w in (w1, w2)]
        x, (h1, h2) = ops.scaled_sum_rms_norms(None, [], gains, 1e-2, tokens=toks.to(dev), table=table.to(dev))
        ref = table.double().numpy()[toks.numpy()]
        for h, w in ((h1, w1), (h2, w2)):
            assert_close(h.double().cpu(), P.norm(ref, w.double().numpy(), 1e-2), 3e-6, f"norms of the embedding, width {D}")
        parts, scales = [torch.randn(5, D, generator=g) for _ in range(3)], [torch.randn(D, generator=g) for _ in range(3)]
        for n in (0, 1, 2, 3):
            use = [(parts[k].to(dev), None if k == 1 else scales[k].to(dev)) for k in range(n)]
            new = ref + sum(((1.0 if k == 1 else scales[k].double().numpy()) * parts[k].double().numpy() for k in range(n)), np.zeros_like(ref))
            xd = x.clone()
            _, hs = ops.scaled_sum_rms_norms(xd, use, gains[:1], 1e-2)
            assert len(hs) == 1
            assert_close(xd.double().cpu(), new, 3e-6, f"{n} parts")
            assert_close(hs[0].double().cpu(), P.norm(new, w1.double().numpy(), 1e-2), 5e-6, f"norm after {n} parts")
            xd = x.clone()
            assert ops.scaled_sum_rms_norms(xd, use, [], 1e-2)[1] == []
            assert_close(xd.double().cpu(), new, 3e-6, "the sum alone")
        out = ops.rms_norm_rows(x, torch.tensor([4, 1], dtype=torch.int32, device=dev), gains[1], 1e-2)
        assert_close(out.double().cpu(), P.norm(ref, w2.double().numpy(), 1e-2)[[4, 1]], 3e-6, "float gains of chosen rows")


def test_gains_keep_what_the_storage_type_cannot_hold(backend):
    """1 + w with w = 2^-12 is 1 in bfloat16: the gain must be float."""
    dev = device_of(backend)
    cfg = make_config([tied(mlp=None)], width=16)
    W = P.random_weights(cfg, seed=3)
    W["l0.norm1"] = np.full(16, 2.0 ** -12)
    eng = build_engine(cfg, bf16(W), backend, dtype="bfloat16", max_tokens=64)
    assert eng.model.layers[0]["norm1"].dtype == torch.float32
    assert float((eng.model.layers[0]["norm1"] - 1.0).min()) == 2.0 ** -12 and str(eng.model.layers[0]["norm1"].device) == str(torch.device(dev))


def test_convolved_heads_carry_their_last_rows(backend):
    """Queries, keys and values through the convolution with runs shorter than the taps, stale history, several sequences in a batch."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(2)
    for Cq, G, kw, dv, taps, pad, cuts in ((10, 1, 3, 2, 3, 1, [1, 2, 3, 9]), (16, 2, 8, 12, 4, 4, [5]), (8, 2, 4, 4, 4, 0, [1, 3, 20]), (6, 0, 0, 5, 2, 3, []),
                                          (1024, 2, 16, 8, 4, 8, [16]), (4, 3, 8, 4, 2, 0, [1, 2, 3]), (12, 1, 4, 4, 5, 0, [2, 3, 4, 30]),
                                          (12, 1, 4, 8, 1, 0, [4, 5]), (8, 2, 4, 4, 3, 0, [1, 2, 3, 4, 5, 6, 7]), (8, 0, 0, 4, 4, 8, [17])):
        T, C = 41, Cq + G * (kw + dv)
        proj, w = torch.randn(T, C + pad, generator=g), torch.randn(C, taps, generator=g)
        ref = P.causal_conv(proj[:, :C].double().numpy(), w.double().numpy())
        coef, every = (0.7, 9) if Cq != 8 else (None, None)
        qref = ref[:, :Cq] * 0.6 * (P.temperature(np.arange(T), coef, every)[:, None] if coef else 1.0)
        cache = PagedCache([(G, dv + kw)] if G else [], 3, 3, torch.float32, dev, states=[StateSpec((taps - 1, C), copies=2)] if taps > 1 else [])
        hist = cache.states[0] if taps > 1 else None
        if taps > 1:
            hist.fill_(7.0)
        cache.admit()
        slot, outs, lo = cache.admit(), [], 0
        for hi in cuts + [T]:
            b = cache_batch(cache, slot, lo, hi, dev)
            outs.append(ops.conv_heads_cache(proj[lo:hi].to(dev).contiguous(), w.t().contiguous().to(dev), hist, b, Cq, G, kw, dv,
                                             cache.pools[0] if G else None, 0.6, (coef, every) if coef else None).cpu())
            lo = hi
        assert_close(torch.cat(outs).double(), qref, 5e-6, f"{taps} taps cut at {cuts}: queries")
        if G:
            rows = cache.pages[slot]
            at = torch.tensor([rows[j // 64] * 64 + j % 64 for j in range(T)], device=dev)
            got = cache.pools[0][:, at].transpose(0, 1).double().cpu()                           # [T, G, dv + kw]
            assert_close(got[..., dv:], ref[:, Cq:Cq + G * kw].reshape(T, G, kw), 5e-6, "cached keys")
            assert_close(got[..., :dv], ref[:, Cq + G * kw:].reshape(T, G, dv), 5e-6, "cached values")
        if taps > 1:
            assert float(hist[:2].min()) == 7.0                                                   # other slots' states are not touched


def test_query_temperature_steps(backend):
    """The factor's steps sit exactly at (p + 1) / every integral, also far from the start."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    pos = torch.tensor([0, 62, 63, 64, 126, 127, 128, 100000, 64 * 3000 - 2, 64 * 3000 - 1], dtype=torch.int32)
    b = run_batch(0, len(pos), dev)
    b.pos, b.slot = pos.to(dev), torch.zeros(len(pos), dtype=torch.int64, device=dev)
    proj, w = torch.ones(len(pos), 4, device=dev), torch.ones(1, 4, device=dev)
    for coef, every in ((0.7, 64), (2.0, 63), (0.1, 1)):
        q = ops.conv_heads_cache(proj, w, None, b, 4, 0, 0, 4, None, 1.0, (coef, every))
        assert_close(q[:, 0].double().cpu(), P.temperature(pos.numpy(), coef, every), 1e-6, f"every {every}")
    q = ops.conv_heads_cache(proj, w, None, b, 4, 0, 0, 4, None, 1.0, (0.7, 64))[:, 0].cpu()
    assert q[1] < q[2] and q[2] == q[3] == q[4] and q[4] < q[5] and q[8] < q[9]


def test_norm_behind_the_rotation(backend):
    """Partly rotated heads under YaRN: cos and sin carry a magnitude, so the norm behind the rotation is not the norm in front of it."""
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(3)
    pos = torch.tensor([5, 0, 64, 129, 1], dtype=torch.int32)
    for H, G, d, rot, pad, factor, store in ((4, 2, 12, 8, 0, 4.0, True), (6, 3, 8, 8, 8, 16.0, False), (3, 1, 6, 2, 3, 2.0, False), (5, 5, 16, 4, 0, None, True), (2, 1, 20, 6, 20, 3.0, False)):
        T, s = 5, {"base": 77.0, "dims": rot}
        if factor:
            s["scaling"] = {"factor": factor, "original": 40, "fast": 6.0, "slow": 0.3}
        proj = torch.randn(T, (H + G) * d + 4, generator=g)
        table = RotaryTable(rot, 77.0, s.get("scaling"), dev, positions=130)
        assert abs(table.magnitude - P.frequencies(s)[1]) < 1e-12 and np.allclose(table.freq.numpy(), P.frequencies(s)[0], rtol=1e-12)
        cache = PagedCache([(G, 2 * d)], 4, 1, torch.float32, dev)
        b = cache_batch(cache, cache.admit(), 0, T, dev)
        b.pos, b.max_pos = pos.to(dev), 129
        pd = proj.to(dev)
        k = pd[:, H * d:(H + G) * d]
        qf = ops.qk_norm_rope_prep(pd[:, :H * d], k, k, H, G, d, d, None, None, True, 1e-2, table.table, rot, 0.6, cache.pools[0], b, halves=True,
                                   q_pad=pad, rot_gain=table.magnitude ** 2, q_store=store)
        q64, k64 = (proj[:, a:z].double().numpy().reshape(T, n, d) for a, z, n in ((0, H * d, H), (H * d, (H + G) * d, G)))
        assert qf.shape == (T, H, pad + d) and (pad == 0 or float(qf[..., :pad].abs().max()) == 0.0)
        assert_close(qf[..., pad:].double().cpu(), P.rms(P.rotate(q64, pos.numpy(), s), 1e-2) * 0.6, 1e-5, "queries")
        rows = cache.pools[0][:, b.slot].transpose(0, 1).double().cpu()
        assert_close(rows[..., d:], P.rms(P.rotate(k64, pos.numpy(), s), 1e-2), 1e-5, "cached keys")
        assert_close(rows[..., :d], k64, 1e-6, "cached values: the projection, neither turned nor normed")
        if factor:                                                             # (the two orders differ: the test can tell them apart)
            assert np.abs(P.rms(P.rotate(k64, pos.numpy(), s), 1e-2) - P.rotate(P.rms(k64, 1e-2), pos.numpy(), s)).max() > 1e-2


def _mixer_alone(backend, layers, T, splits, seed=3, width=24, tol=5e-5, dtype="float32", tweak=None):
    """The last layer's mixer through its layer object, the engine's cache and state, the tokens cut at `splits`, against the plain statement.  A
    layer in front of it (if any) provides the keys and values."""
    layers = layers if isinstance(layers, list) else [layers]
    cfg = make_config(layers, width=width)
    W = P.random_weights(cfg, seed=seed)
    if tweak:
        tweak(W)
    eng = build_engine(cfg, f32(W) if dtype == "float32" else bf16(W), backend, dtype=dtype, max_tokens=max(256, T + 64), max_seqs=3)
    dev, st = eng.device, torch.float32 if dtype == "float32" else torch.bfloat16
    g = torch.Generator().manual_seed(seed + 100)
    h = torch.randn(T, width, generator=g).bfloat16().float()
    h64, eps, kv = h.double().numpy(), cfg["norm"]["eps"], None
    if len(layers) > 1:
        kv = P.differential_kv(h64, {n.replace(".", "_"): W["l0.mix." + n] for n in ("k", "v", "k.conv", "v.conv")}, layers[0]["mixer"])
    ref = P.mixer(layers[-1]["type"], h64, W, f"l{len(layers) - 1}.mix.", layers[-1]["mixer"], eps, kv)
    eng.open_sequence()                                                    # (not slot 0)
    slot = eng.open_sequence()
    for s in eng.cache.states:
        s.fill_(5.0)                                                       # stale state: a new sequence must not read it
    for p in eng.cache.pools:
        p.fill_(3.0)
    outs, lo = [], 0
    for hi in list(splits) + [T]:
        b = eng.layout([(slot, [0] * (hi - lo))])
        for i, L in enumerate(eng.model.layers):
            p0, p1, s0, s1 = eng.model.slices[i]
            y = L["mixer"](h[lo:hi].to(st).to(dev), b, eng.cache.pools[p0:p1], eng.cache.states[s0:s1])
        outs.append(y.double().cpu())
        lo = hi
    got, ref = torch.cat(outs), torch.from_numpy(ref)
    what = f"{layers[-1]['mixer']} cut at {splits}"
    return assert_close(got, ref, tol, what) if dtype == "float32" else assert_near(got, ref, what)


def test_differential_attention_layer_alone(backend):
    _mixer_alone(backend, diff(), 70, [])
    _mixer_alone(backend, diff(), 70, [1, 2, 3, 5, 16, 17, 31, 32, 33, 63, 64, 65, 69])
    _mixer_alone(backend, diff(heads=5, kv_heads=1, dim=6, vdim=16, conv=1, lam=0.8, every=1), 140, [63, 64, 65, 128, 129])
    _mixer_alone(backend, diff(heads=2, kv_heads=2, dim=16, vdim=32, conv=4, coef=None, lam=0.05), 20, [1, 2, 7])
    _mixer_alone(backend, diff(heads=3, kv_heads=3, dim=4, vdim=3, conv=6), 90, [2, 4, 6, 8, 10, 80, 82])
    _mixer_alone(backend, diff(heads=1, kv_heads=1, dim=1, vdim=1, conv=2), 10, [5])


def test_shared_keys_and_values_layer_alone(backend):
    _mixer_alone(backend, [diff(), diff(heads=4, kv_from=0, conv=2, lam=0.1, scale=0.2)], 70, [1, 2, 3, 31, 33, 64, 65])
    _mixer_alone(backend, [diff(heads=2, kv_heads=2, dim=16, vdim=32, conv=4), diff(heads=8, kv_heads=2, dim=16, vdim=32, kv_from=0, conv=1, coef=None)], 90, [2, 64, 66])


def test_tied_rotary_attention_layer_alone(backend):
    _mixer_alone(backend, tied(), 70, [])
    _mixer_alone(backend, tied(), 70, [1, 2, 3, 5, 31, 32, 33, 63, 64, 65, 69])
    _mixer_alone(backend, tied(heads=5, kv_heads=1, dim=6, rot=6, factor=None), 140, [63, 64, 65, 128, 129])
    _mixer_alone(backend, tied(heads=4, kv_heads=4, dim=64, rot=64, base=2e5, factor=5.0, original=512, fast=24.0, slow=1.5), 40, [7])
    _mixer_alone(backend, tied(heads=1, kv_heads=1, dim=2, rot=2), 10, [5])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixers_at_the_matrix_core_sizes(dtype):
    """Sizes the matrix-core kernels take, and some that fall back; prompt tiles, short runs beside long ones, head groups beyond 32."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    for layers, T, splits in ((diff(heads=6, kv_heads=3, dim=32, vdim=64, conv=3), 300, [87, 88, 89, 126, 170, 298, 299]),
                              (diff(heads=6, kv_heads=1, dim=16, vdim=32), 330, [43, 47, 53, 54, 126, 170, 328, 329]),
                              (diff(heads=8, kv_heads=2, dim=64, vdim=128, conv=2), 200, [150, 151, 153, 190]),
                              (diff(heads=3, kv_heads=1, dim=64, vdim=64), 140, [100, 101, 102, 139]),
                              (diff(heads=2, kv_heads=2, dim=48, vdim=96), 130, [64, 65, 129]),
                              (diff(heads=2, kv_heads=1, dim=96, vdim=96, conv=1), 130, [64, 65, 129]),
                              (diff(heads=40, kv_heads=1, dim=16, vdim=32), 90, [33, 34, 80]),
                              (diff(heads=2, kv_heads=2, dim=128, vdim=128), 100, [50, 51, 99]),
                              (diff(heads=4, kv_heads=2, dim=24, vdim=40), 100, [50, 51, 99]),         # (wave kernel)
                              ([diff(heads=6, kv_heads=3, dim=32, vdim=64), diff(heads=12, kv_heads=3, dim=32, vdim=64, kv_from=0)], 150, [64, 66, 70, 149]),
                              (tied(heads=6, kv_heads=2, dim=64, rot=64), 300, [87, 88, 89, 126, 170, 298, 299]),
                              (tied(heads=3, kv_heads=1, dim=32, rot=8), 150, [100, 101, 102, 140]),
                              (tied(heads=4, kv_heads=2, dim=96, rot=64), 130, [64, 65, 129]),
                              (tied(heads=8, kv_heads=1, dim=128, rot=128), 130, [64, 65, 129]),
                              (tied(heads=4, kv_heads=2, dim=80, rot=32), 100, [50, 51, 99])):          # (row-attention kernel)
        _mixer_alone("hip", layers, T, splits, dtype=dtype, width=32)


def _paged(g, G, R, L, dev, dtype):
    """A sequence of L random rows in pages out of order, not the first ones, every other row of the pool far from anything sensible."""
    npages = (L + 63) // 64
    cache = PagedCache([(G, R)], npages + 3, 2, dtype, dev)
    cache.pools[0].fill_(50.0)
    cache.free_pages = torch.randperm(npages + 3, generator=g).tolist()
    cache.admit()
    slot = cache.admit()
    rows = torch.randn(L, G, R, generator=g).bfloat16().double()
    b = cache_batch(cache, slot, 0, L, dev)
    cache.pools[0][:, b.slot] = rows.transpose(0, 1).to(dtype).to(dev)
    return cache, slot, rows


def _query_batch(cache, slot, L, nq, dev):
    b = run_batch(L - nq, L, dev, slot)
    b.seq, b.block_table = torch.full((nq,), slot, dtype=torch.int32, device=dev), cache.block_table()
    return b


@pytest.mark.parametrize("dtype,tol", STORAGE)
def test_differential_attention_forms(backend, dtype, tol):
    """The operation alone: the last tokens of a sequence as one batch, every launch form, with and without a gate."""
    dev = device_of(backend)
    ops = make_ops(backend, dtype, dev)
    g = torch.Generator().manual_seed(4)
    for H, G, d, dv, L, nq, lam, gated in ((4, 2, 32, 64, 200, 1, 0.5, True), (4, 2, 32, 64, 200, 37, 0.5, True), (6, 1, 16, 32, 330, 5, 0.2, False),
                                           (8, 2, 64, 128, 150, 66, 0.9, True), (8, 8, 64, 64, 520, 1, -0.4, True), (40, 1, 16, 32, 97, 3, 0.3, True),
                                           (3, 3, 48, 96, 33, 33, 0.3, True), (2, 1, 128, 128, 140, 20, 0.6, False), (2, 2, 96, 96, 64, 64, 0.1, True),
                                           (2, 2, 32, 32, 1, 1, 0.1, True), (3, 1, 20, 12, 70, 9, 0.3, True), (12, 4, 32, 64, 300, 30, 0.3, True)):
        cache, slot, rows = _paged(g, G, dv + 2 * d, L, dev, dtype)
        q = (torch.randn(nq, H, 2, d, generator=g) / d ** 0.5 * 2).bfloat16().double()
        gate = torch.randn(nq, H * dv + 8, generator=g).bfloat16().double()
        k, v = rows[..., dv:].reshape(L, G, 2, d), rows[..., :dv]
        ref = P.differential(q.numpy(), k.numpy(), v.numpy(), 1.0, lam, 0.25, 1e-5).reshape(nq, H * dv)
        if gated:
            ref = ref * P.sigmoid(gate[:, 8:].numpy())
        b = _query_batch(cache, slot, L, nq, dev)
        gd = gate.to(dtype).to(dev)[:, 8:] if gated else None
        forms = [dict(), dict(variant=1)] + ([dict(key_splits=s) for s in (1, 2, 5)] if backend == "hip" else [])
        for kw in forms:
            out = ops.diff_attention(q.to(dtype).to(dev).reshape(nq, -1), cache.pools[0], b, H, d, dv, lam, 0.75, 1e-5, gd, 64, **kw).double().cpu()
            what = f"{H} heads over {G}, {d} / {dv}, {nq} of {L} tokens, {kw}"
            if dtype == torch.float32:
                assert_close(out, ref, tol, what)
            else:
                assert_near(out, ref, what)


@pytest.mark.gpu
def test_single_map_attention_forms():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    dev, dtype = "cuda:0", torch.bfloat16
    ops = make_ops("hip", dtype, dev)
    g = torch.Generator().manual_seed(5)
    for H, G, d, L, nq in ((8, 4, 64, 200, 1), (8, 4, 64, 200, 37), (6, 1, 32, 330, 5), (16, 2, 128, 150, 66), (8, 8, 96, 520, 1), (40, 1, 32, 97, 3), (4, 4, 64, 1, 1), (33, 1, 64, 100, 64)):
        cache, slot, rows = _paged(g, G, 2 * d, L, dev, dtype)
        q = (torch.randn(nq, H, d, generator=g) / d ** 0.5 * 2).bfloat16().double()
        ref = P.attention(q.numpy(), rows[..., d:].numpy(), rows[..., :d].numpy(), 1.0).reshape(nq, H * d)
        b = _query_batch(cache, slot, L, nq, dev)
        for kw in [dict()] + [dict(key_splits=s) for s in (1, 2, 5)]:
            out = ops.single_map_attention(q.to(dtype).to(dev), cache.pools[0], b, H, d, d, 64, **kw)
            assert_close(out.double().cpu(), ref, 1e-2, f"{H} heads over {G} of {d}, {nq} of {L} tokens, {kw}")


# ---- keys that stand out: first tokens, page and block borders, far back, through one map or the other ----------------------------------

@pytest.mark.parametrize("dtype,tol", STORAGE)
@pytest.mark.parametrize("nq", [1, 20], ids=["decoded", "prompt"])
def test_a_loud_key_is_heard_through_its_map(backend, nq, dtype, tol):
    """Head 0's map 1 points at one key of its pool, head 2's map 2 at the same place of the other pool: head 0 returns that value (normed), head
    2 minus lambda times it on top of its own average; a key that comes after the query is not heard."""
    dev = device_of(backend)
    ops = make_ops(backend, dtype, dev)
    H, G, d, dv, L, lam = 4, 2, 32, 64, 340, 0.5
    for spike in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, 318, 319, 320, 339):
        g = torch.Generator().manual_seed(spike)
        cache, slot, rows = _paged(g, G, dv + 2 * d, L, dev, dtype)
        for pool, m in ((0, 0), (1, 1)):
            rows[:, pool, dv + m * d + 7] = 0.0
            rows[spike, pool, dv + m * d + 7] = 8.0
        at = torch.tensor([cache.pages[slot][j // 64] * 64 + j % 64 for j in range(L)], device=dev)
        cache.pools[0][:, at] = rows.transpose(0, 1).to(dtype).to(dev)
        q = (torch.randn(nq, H, 2, d, generator=g) * 0.1).bfloat16().double()
        q[:, 0, 0, 7], q[:, 2, 1, 7] = 4.0, 4.0
        ref = torch.from_numpy(P.differential(q.numpy(), rows[..., dv:].reshape(L, G, 2, d).numpy(), rows[..., :dv].numpy(), 1.0, lam, 0.0, 1e-5))
        v = rows[spike, 0, :dv] / rows[spike, 0, :dv].pow(2).mean().sqrt()
        w = -rows[spike, 1, :dv] / rows[spike, 1, :dv].pow(2).mean().sqrt()
        if spike <= L - 1:
            assert (ref[-1, 0] - v).pow(2).mean().sqrt() < 0.25 and (ref[-1, 2] - w).pow(2).mean().sqrt() < 0.5
        b = _query_batch(cache, slot, L, nq, dev)
        out = ops.diff_attention(q.to(dtype).to(dev).reshape(nq, -1), cache.pools[0], b, H, d, dv, lam, 1.0, 1e-5, None, 64)
        assert_close(out.double().cpu().view(nq, H, dv), ref, tol, f"loud key at {spike}")


def test_lambda_comes_from_its_vectors(backend):
    """Each of the four vectors and the constant moves lambda as it should."""
    cfg = make_config([diff(dim=8)], width=24)
    W = P.random_weights(cfg, seed=8)
    eng = build_engine(cfg, f32(W), backend, max_tokens=64)
    m = eng.model.layers[0]["mixer"]
    assert abs(m.lam - P.lambda_of(*(W["l0.mix." + n] for n in ("lq1", "lk1", "lq2", "lk2")), 0.4)) < 1e-12 and abs(m.out_scale - 0.6) < 1e-12
    for n in ("lq1", "lk1", "lq2", "lk2"):
        _mixer_alone(backend, diff(dim=8), 12, [5], tweak=lambda W, n=n: W.update({"l0.mix." + n: W["l0.mix." + n] * 2.0}))


# ---- experts -------------------------------------------------------------------------------------------------------------------------

def _expert_layer(ops, dev, dtype, E, top, ff, D, shared, seed, weigh="input"):
    g = torch.Generator().manual_seed(seed)
    gate, up, down = ([(torch.randn(s, generator=g) / math.sqrt(s[1]) * f).bfloat16().double() for _ in range(E)] for s, f in
                      (((ff, D), 2.0), ((ff, D), 2.0), ((D, ff), 1.0)))
    router = (torch.randn(E, D, generator=g) / math.sqrt(D)).bfloat16().double()
    sh = [(torch.randn(s, generator=g) / math.sqrt(s[1])).bfloat16().double() for s in ((shared, D), (shared, D), (D, shared))] if shared else None

    def put(t):
        return t.to(dtype).to(dev)

    layer = SigmoidMoE(ops, router=put(router), gate=[put(t) for t in gate], up=[put(t) for t in up], down=[put(t) for t in down], top_k=top, weigh=weigh,
                       shared=GatedFeedForward(ops, gate=put(sh[0]), up=put(sh[1]), down=put(sh[2])) if shared else None)
    return layer, router, gate, up, down, sh


def test_weights_on_the_experts_input(backend):
    dev = device_of(backend)
    ops = make_ops(backend, torch.float32, dev)
    g = torch.Generator().manual_seed(1)
    for E, top, ff, D, shared, T in ((8, 1, 16, 24, 12, 9), (5, 3, 11, 20, None, 7), (4, 4, 8, 32, 8, 40), (3, 2, 5, 9, 6, 3), (6, 2, 64, 64, 24, 130)):
        layer, router, gate, up, down, sh = _expert_layer(ops, dev, torch.float32, E, top, ff, D, shared, E)
        h = torch.randn(T, D, generator=g).bfloat16().double()
        idx, wt = P.route(h.numpy(), router.numpy(), top)
        ref = P.experts(h.numpy(), idx, wt, *([t.numpy() for t in ts] for ts in (gate, up, down)))
        other = sum(w * P.unit(h[0:1].numpy(), *(ts[e].numpy() for ts in (gate, up, down))) for e, w in zip(idx[0], wt[0]))
        assert np.abs(other - ref[0]).max() > 1e-2                          # (weights on the output would be seen)
        ys = layer(h.float().to(dev))
        assert len(ys) == (2 if shared else 1)
        assert_close(ys[0].double().cpu(), ref, 3e-5, f"{E} experts, top {top}, {T} tokens")
        if shared:
            assert_close(ys[1].double().cpu(), P.unit(h.numpy(), *(t.numpy() for t in sh)), 3e-5, "shared expert")


@pytest.mark.gpu
@pytest.mark.parametrize("weigh", ["input", "output"])
def test_expert_kernel_forms_in_bfloat16(weigh):
    """Per token, expert-major, grouped matrix cores, vendor products per expert: the same weighting in each."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    dev, dtype = "cuda:0", torch.bfloat16
    ops = make_ops("hip", dtype, dev)
    g = torch.Generator().manual_seed(2)
    forms = {"per token": dict(moe_token_slots=10 ** 9, moe_sorted_above=10 ** 9), "expert-major": dict(moe_token_slots=0, moe_expert_major_slots=10 ** 9),
             "grouped": dict(moe_token_slots=0, moe_expert_major_slots=0, moe_sorted_above=0),
             "vendor": dict(moe_token_slots=0, moe_expert_major_slots=0, moe_sorted_above=0, moe_grouped_kernel=False)}
    for E, top, ff, D, T in ((8, 2, 64, 128, 37), (4, 1, 128, 64, 150), (5, 3, 72, 88, 20)):
        layer, router, gate, up, down, _ = _expert_layer(ops, dev, dtype, E, top, ff, D, None, 10 + E, weigh)
        h = torch.randn(T, D, generator=g).bfloat16().double()
        idx, wt = P.route(h.numpy(), router.numpy(), top)
        mats = [[t.numpy() for t in ts] for ts in (gate, up, down)]
        if weigh == "input":
            ref = P.experts(h.numpy(), idx, wt, *mats)
        else:
            ref = np.stack([sum(w * P.unit(h[t:t + 1].numpy(), *(m[e] for m in mats))[0] for e, w in zip(idx[t], wt[t])) for t in range(T)])
        for name, knobs in forms.items():
            for k, v in knobs.items():
                setattr(ops, k, v)
            y = layer(h.to(dtype).to(dev))[0].double().cpu()
            for k in knobs:
                delattr(ops, k)
            assert_near(y, ref, f"{name}, {E} experts, top {top}", overall=0.01, worst=0.03)


def test_router_parameters_are_checked():
    ops = make_ops("unfused", torch.float32, "cpu")
    z = [torch.zeros(4, 6)] * 3
    kw = dict(router=torch.zeros(3, 6), gate=z, up=z, down=[torch.zeros(6, 4)] * 3)
    for bad in (dict(top_k=0), dict(top_k=4), dict(top_k=1, weigh="both"), dict(top_k=1, correction=torch.zeros(2)), dict(top_k=1, groups=2)):
        with pytest.raises(ValueError):
            SigmoidMoE(ops, **{**kw, **bad})
    assert CorrectedSigmoidMoE(ops, correction=torch.zeros(3), top_k=2, **kw).weigh == "output"


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


def test_layers_without_keys_share_their_sources_pools(backend, std):
    cfg, W, _, _, _ = std
    eng = build_engine(cfg, f32(W), backend, max_tokens=64)
    s = eng.model.slices
    assert s[2][:2] == s[0][:2] and s[5][:2] == s[3][:2] and len(eng.cache.pools) == 5
    assert [L["mixer"].shared_kv for L in eng.model.layers if hasattr(L["mixer"], "shared_kv")] == [False, True, False, True]


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
    cfg = make_config([diff(every=20, mlp=moe(3, 1, 12, 5)), tied(mlp=None), diff(heads=2, kv_from=0, every=70, coef=0.9, mlp=moe(2, 2, 9, None))], width=32, vocab=29)
    W = P.random_weights(cfg, seed=9)
    toks = tokens_for(cfg, 210, 5)
    ref = plain_logits(cfg, W, toks)
    eng = build_engine(cfg, f32(W), backend, max_tokens=256, max_seqs=1)
    got = run_schedule(eng, {"s": toks}, [[("s", 3)]] + [[("s", 1)]] * 207)      # decoded tokens pass temperature steps and three page borders
    assert_close(got["s"], ref, F32_TOL, "207 decoded tokens")


@pytest.mark.parametrize("variant", range(5))
def test_other_sizes(backend, variant):
    layers, kw = [
        ([diff(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, every=1, mlp=moe(1, 1, 1, 1))], dict(width=8, vocab=5, eps=1e-3)),
        ([tied(heads=6, kv_heads=3, dim=16, rot=16, mlp=moe(33, 5, 3, 40)), diff(heads=4, kv_heads=4, dim=32, vdim=32, conv=5, mlp=moe(6, 6, 20, None)),
          diff(heads=4, kv_heads=4, dim=32, vdim=32, conv=4, kv_from=1, mlp=None)], dict(width=96, vocab=200)),
        ([diff(heads=7, kv_heads=1, dim=70, vdim=12, conv=3), diff(heads=7, kv_heads=1, dim=70, vdim=12, kv_from=0), diff(heads=2, kv_heads=1, dim=70, vdim=12, kv_from=0, conv=2)],
         dict(width=41, vocab=33, eps=1e-6)),
        ([tied(heads=2, kv_heads=2, dim=4, rot=4, factor=30.0, original=4096, fast=20.0, slow=2.0, base=9e5, mlp=moe())] * 3, dict(width=48, vocab=61)),
        ([diff(mlp=None, lam=0.0, coef=0.0)], dict(width=20, vocab=9)),
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


@pytest.mark.gpu
def test_bfloat16_at_matrix_core_sizes_whatever_the_cut():
    """A model whose layers run on the matrix-core kernels: whole, in portions, decoded, mixed with others - each near the plain statement.  (All
    experts are used: a choice that flips on a rounding would show as more than it is.)"""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = make_config([diff(heads=4, kv_heads=1, dim=32, vdim=64, conv=4, mlp=moe(2, 2, 64, 64)), tied(heads=4, kv_heads=2, dim=32, rot=32, mlp=moe(1, 1, 64, 64)),
                       diff(heads=8, kv_heads=1, dim=32, vdim=64, conv=2, kv_from=0, mlp=moe(2, 2, 64, 64))], width=128, vocab=96)
    W = P.random_weights(cfg, seed=31)
    seqs = {"a": tokens_for(cfg, 300, 1), "b": tokens_for(cfg, 90, 2)}
    ref = {k: plain_logits(cfg, W, v) for k, v in seqs.items()}
    eng = build_engine(cfg, bf16(W), "hip", dtype="bfloat16", max_tokens=512)
    for steps in ([[("a", 300)]], [[("a", 33), ("b", 70)], [("a", 1), ("b", 20)], [("a", 266)]], [[("a", 2)]] * 20 + [[("a", 250)]] + [[("a", 1)]] * 10,
                  [[("b", 3)], [("a", 200), ("b", 1)], [("b", 86), ("a", 1)], [("a", 99)]]):
        for k, got in run_schedule(eng, seqs, steps).items():
            d = got - ref[k]
            rel = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / ref[k].std()
            assert rel.max() < 0.03, f"{k}: relative error {rel.max():.3f} at position {int(rel.argmax())}"


def test_configurations_that_do_not_fit_are_refused(backend):
    cfg = make_config([diff(), tied(), diff(kv_from=0)])
    W = f32(P.random_weights(cfg, seed=5))
    ops = make_ops("unfused", torch.float32, "cpu")
    for edit in (lambda c: c["layers"][1]["mixer"].update(vdim=4), lambda c: c["layers"][0].update(type="unknown"), lambda c: c["layers"][2]["mixer"].update(kv_from=1),
                 lambda c: c["layers"][2]["mixer"].update(kv_from=2), lambda c: c["layers"][2]["mixer"].update(kv_heads=1), lambda c: c["layers"][0]["mixer"].update(conv=4),
                 lambda c: c["layers"][0]["mixer"].update(conv=0), lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=0), lambda c: c.update(vocab=54)):
        bad = json.loads(json.dumps(cfg))
        edit(bad)
        with pytest.raises(ValueError):
            Rivolix.from_config(bad, W, ops, "cpu", torch.float32)
    with pytest.raises(KeyError):
        Rivolix.from_config(cfg, {k: v for k, v in W.items() if k != "l0.mix.lq2"}, ops, "cpu", torch.float32)
    short = json.loads(json.dumps(make_config([diff(heads=3, kv_heads=3), tied(heads=2, kv_heads=2)])))
    W2 = P.random_weights(short, seed=6)
    toks, ref = tokens_for(short, 20, 1), None
    ref = plain_logits(short, W2, toks)
    del short["layers"][0]["mixer"]["kv_heads"], short["layers"][1]["mixer"]["kv_heads"], short["layers"][1]["mixer"]["vdim"]
    got = run_schedule(build_engine(short, f32(W2), backend), {"s": toks}, [[("s", 20)]])
    assert_close(got["s"], ref, F32_TOL, "key / value heads default to the query heads")


def test_step_tiles_split_short_runs_from_long_ones():
    b = run_batch(0, 3, "cpu")
    b.items = [(3, 0, 1), (1, 1, 70), (0, 71, 8), (2, 79, 9)]
    prompt, step = b.split_tiles(8)
    assert step.tolist() == [[3, 0, 1], [0, 71, 8]] and prompt.tolist() == [[1, 1, 32], [1, 33, 32], [1, 65, 6], [2, 79, 9]]
    assert b.split_tiles(8)[0].data_ptr() == prompt.data_ptr()                     # (made once per step)


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
    assert registry.architectures()["Rivolix"] == "paged"
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
@pytest.mark.parametrize("sizes", ["odd", "matrix-core"])
def test_decode_steps_from_a_graph_match_eager_steps(dtype, sizes, std):
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg, W, seqs, _, _ = std
    if sizes == "matrix-core":
        cfg = make_config([diff(heads=6, kv_heads=3, dim=32, vdim=64, conv=3, mlp=moe(4, 2, 64, 64)), tied(heads=4, kv_heads=2, dim=64, rot=32, mlp=moe(4, 1, 64, None)),
                           diff(heads=9, kv_heads=3, dim=32, vdim=64, kv_from=0, mlp=None)], width=64)
        W = P.random_weights(cfg, seed=12)
    outs = []
    for graphs in (False, True):
        eng = build_engine(cfg, f32(W) if dtype == "float32" else bf16(W), "hip", dtype=dtype, max_tokens=512, max_seqs=2, decode_graphs=graphs)
        steps = [[("a", 100), ("b", 30)]] + [[("a", 1), ("b", 1)]] * 7 + [[("a", 1)]] * 43
        outs.append(run_schedule(eng, seqs, steps))
        if graphs:
            assert any(g for g in eng._graphs.values()), "no decode step was replayed from a graph"
    for k in ("a", "b"):
        assert_close(outs[1][k], outs[0][k], 1e-5 if dtype == "float32" else 2e-2, f"graph replay, sequence {k}")
