"""Sisepel on the GPU: each new or widened HIP kernel against its plain torch reference (states
carried over several steps, stale states in the slots), the mixers, the feed-forwards and the
pair of mixers alone against the plain implementation with crafted cases that random weights
would hide (a token just inside and just outside a window, a key that stands out under a cap, a
sink that takes most of a softmax, a write remembered over hundreds of tokens), the engine
against the plain whole-sequence implementation however requests are cut into steps, in
float32 and bfloat16, and greedy generation through LLMEngine."""

import pytest
import torch

import drives
from helpers import (SISE, random_prompt, sisepel_attention, sisepel_config, sisepel_dense,
                     sisepel_layer, sisepel_moe, sisepel_retention, sisepel_scaling,
                     write_sisepel_model)
from kernel_refs import TorchOps
from plain import sisepel_plain as plain
from test_fubepel_gpu import assert_rows_within_rounding, rms_errors
from test_palelix_gpu import Scene, close, load_part, part_context, rnd, run_part_in_steps
from test_zolorax_gpu import close_part
from tokensprint_amd.config import Config, SamplingParams
from tokensprint_amd.engine import ModelRunner
from tokensprint_amd.engine.assemble import load_model
from tokensprint_amd.engine.llm_engine import LLMEngine
from tokensprint_amd.kernels import load_hip_ops
from tokensprint_amd.kernels.stream import NormedPair
from tokensprint_amd.models.spec import PartSpec
from tokensprint_amd.parts.attention import SoftmaxAttention
from tokensprint_amd.parts.base import (FEED_FORWARDS, MIXERS, POSITIONS, PagedKVNeed,
                                        SlotStateNeed, build_part)

pytestmark = pytest.mark.gpu
REF = TorchOps()
SPANS = [[7, 1, 3, 40], [1, 1, 0, 2], [2, 5, 1, 1], [1, 1, 1, 1], [150, 1, 0, 300], [1, 1, 1, 1]]
TIGHT, ROUNDED = dict(rtol=1e-4, atol=1e-4), dict(rtol=1e-2, atol=1e-2)


# ------------------------------------------------------------------ row kernels, gated units


def test_two_normed_outputs_and_the_add_behind_them(gpu_device):
    """The pair alone, added to the stream, and with the next norm or the stream's rows behind
    it: rows of one element, of fewer and of more than a workgroup keeps in registers."""
    ops = load_hip_ops(gpu_device)
    for T, width in ((5, 40), (33, 2304), (1, 1), (3, 7), (2, 9001)):
        w = [(1 + 0.3 * rnd((width,), 10 + i)).to(gpu_device) for i in range(4)]
        for a_dtype in (torch.float32, torch.bfloat16):
            for b_dtype in (torch.float32, torch.bfloat16):
                pair = NormedPair(rnd((T, width), 2, 3.0).to(a_dtype).to(gpu_device), w[0],
                                  rnd((T, width), 3, 0.2).to(b_dtype).to(gpu_device), w[1], 1e-3)
                resid = rnd((T, width), 1).to(gpu_device)
                for dtype, tol in ((torch.float32, TIGHT), (torch.bfloat16, ROUNDED)):
                    close(ops.normed_pair(pair, dtype), REF.normed_pair(pair, dtype), **tol)
                    for norm, out_dtype in ((w[3], dtype), (None, dtype), (None, None)):
                        want, got = resid.clone(), resid.clone()
                        kw = (w[2], 1e-4, norm, 1e-5, out_dtype)
                        want_rows = REF.pair_postnorm_add(want, pair, *kw)
                        rows = ops.pair_postnorm_add(got, pair, *kw)
                        close(got, want, **TIGHT)
                        if out_dtype is None:
                            assert rows is None
                            continue
                        assert rows.dtype == dtype
                        close(rows, want_rows, **tol)
                        if norm is None:
                            assert torch.equal(rows, got.to(dtype))
                # anything else that takes rows sees the sum
                want, got = resid.clone(), resid.clone()
                close(ops.add_rmsnorm(got, pair, w[2], 1e-5, torch.float32),
                      REF.add_rmsnorm(want, REF.normed_pair(pair, torch.float32), w[2], 1e-5, torch.float32), **TIGHT)
                ops.stream_add(got, pair, None, None)
                REF.stream_add(want, REF.normed_pair(pair, torch.float32), None, None)
                close(got, want, **TIGHT)
    with pytest.raises(ValueError, match="second output"):
        ops.normed_pair(NormedPair(torch.zeros(2, 4, device=gpu_device), w[0], torch.zeros(2, 5, device=gpu_device),
                                   w[0], 1e-5), torch.float32)


def test_gelu_gated_unit_in_every_product(gpu_device):
    """The activation alone, and inside the paired products of every layout: few rows and
    many, a short and a long reduction, the tiled product for prompts, sizes that are
    multiples of nothing; gates far on either side."""
    ops = load_hip_ops(gpu_device)
    for dtype in (torch.float32, torch.bfloat16):
        tol = dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else ROUNDED
        for rows, inner in ((5, 24), (3, 7), (130, 512)):
            gu = rnd((rows, 2 * inner), 1, 2.0).to(dtype)
            gu[0, :3] = torch.tensor([60.0, -60.0, 0.0]).to(dtype)
            gu = gu.to(gpu_device)
            close(ops.silu_mul(gu, act="gelu_tanh"), REF.silu_mul(gu, act="gelu_tanh"), **tol)
    for M, K, inner in ((1, 256, 64), (8, 40, 24), (16, 512, 96), (20, 256, 48), (40, 1024, 200),
                        (64, 2048, 256), (8, 2048, 512), (100, 256, 128), (600, 512, 192),
                        (2048, 256, 128), (12, 30, 10)):
        for dtype in (torch.float32, torch.bfloat16):
            x = rnd((M, K), 3).to(dtype)
            x[0] *= 8.0
            x = x.to(gpu_device)
            w = rnd((2 * inner, K), 4, 2.0 * K ** -0.5).to(dtype).to(gpu_device)
            got = ops.linear_silu_mul(x, w, dtype, act="gelu_tanh")
            want = REF.linear_silu_mul(x, w, dtype, act="gelu_tanh")
            assert got.dtype == dtype and bool(torch.isfinite(got).all())
            close(got, want, **(dict(rtol=2e-4, atol=5e-4) if dtype == torch.float32
                                else dict(rtol=2e-2, atol=4e-2)))
    for more in (dict(act="relu"), dict(act="gelu_tanh", limit=1.0)):
        with pytest.raises(ValueError, match="gated unit"):
            ops.silu_mul(torch.zeros(2, 4, device=gpu_device), **more)


def test_router_with_a_bias(gpu_device):
    ops = load_hip_ops(gpu_device)
    for T, E, top in ((1, 12, 3), (37, 8, 2), (300, 64, 6), (5, 5, 5), (9, 130, 1), (4, 1, 1)):
        logits, bias = rnd((T, E), T, 2.0).to(gpu_device), rnd((E,), 7, 3.0).to(gpu_device)
        got = ops.route_experts(logits, top=top, bias=bias).cpu()
        close(got, REF.route_experts(logits, top=top, bias=bias))
        z = (logits.double() + bias.double()).cpu()
        for t in range(min(T, 20)):
            want = plain.route(z[t], top)
            assert sorted(got[t].nonzero().flatten().tolist()) == sorted(want)
            for e, share in want.items():
                assert float(got[t, e]) == pytest.approx(share, rel=1e-4)
    with pytest.raises(ValueError, match="bias"):
        ops.route_experts(torch.zeros(2, 4, device=gpu_device), top=1, bias=torch.zeros(5, device=gpu_device))


@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_norm_without_a_weight_and_gate(gpu_device, out_dtype):
    ops = load_hip_ops(gpu_device)
    for T, groups, width in ((1, 1, 40), (9, 4, 64), (33, 3, 70), (5, 1, 1030), (2, 5, 1)):
        inner = groups * width
        y, gate = rnd((T, inner), 1, 3.0).to(gpu_device), rnd((T, inner + 5), 2).to(gpu_device)
        for kind in ("sigmoid", "silu"):
            kw = dict(groups=groups, gate=kind, eps=1e-3, out_dtype=out_dtype)
            close(ops.norm_gate(y, gate, 5, None, **kw), REF.norm_gate(y, gate, 5, None, **kw),
                  **(TIGHT if out_dtype == torch.float32 else ROUNDED))


# ------------------------------------------------------------------ the recurrence


def rotation_table(pairs, base, rows=1200):
    freqs = (base ** (-torch.arange(pairs, dtype=torch.float64) / pairs)).float()
    angles = torch.outer(torch.arange(rows, dtype=torch.float32), freqs)
    return torch.stack([angles.cos(), angles.sin()], -1).contiguous()


@pytest.mark.parametrize("heads, dim, vdim, pairs", [(4, 16, 64, 8), (3, 10, 6, 2), (2, 6, 70, 3),
                                                     (1, 132, 9, 66), (2, 64, 48, 20), (16, 32, 128, 16),
                                                     (1, 7, 5, 1), (2, 128, 70, 64), (1, 256, 20, 100)])
def test_recurrence_that_turns_its_operands(gpu_device, heads, dim, vdim, pairs):
    """Over steps with portions and single tokens, portions long enough for chunks (up to 128
    channels) beside short ones, states carried on, stale states in the slots; positions beyond
    a page and a chunk."""
    ops = load_hip_ops(gpu_device)
    qk, inner = heads * dim, heads * vdim
    scene = Scene(gpu_device, SlotStateNeed((heads, dim, vdim), torch.float32, "s"), 8, 4, num_pages=200)
    st = scene.view.states["s"]
    st.fill_(3.0)
    st_ref = st.clone()
    decay = (0.8 + 0.2 * torch.rand(heads, generator=torch.Generator().manual_seed(1))).to(gpu_device)
    table = rotation_table(pairs, 1000.0).to(gpu_device)
    for i, spans in enumerate(SPANS):
        batch = scene.step(spans)
        T = batch.num_tokens
        x = rnd((T, 3 + 2 * qk + inner), 10 + i, 0.5).to(gpu_device)
        kw = dict(heads=heads, kv_heads=heads, dim=dim, vdim=vdim, silu_inputs=False, decay=decay,
                  turn=table, k_scale=dim ** -0.5)
        before = x.clone()
        got = ops.linear_recurrence(x, 3, 3 + qk, 3 + 2 * qk, batch, st, **kw)
        assert torch.equal(x, before)
        want = REF.linear_recurrence(x, 3, 3 + qk, 3 + 2 * qk, batch, st_ref, **kw)
        close(got, want, rtol=2e-4, atol=2e-4)
        close(st, st_ref, rtol=2e-4, atol=2e-4)


def test_a_rotation_of_the_recurrence_is_checked(gpu_device):
    ops = load_hip_ops(gpu_device)
    scene = Scene(gpu_device, SlotStateNeed((1, 8, 4), torch.float32, "s"), 8, 1)
    st, x = scene.view.states["s"], torch.zeros(5, 20, device=gpu_device)
    batch = scene.step([5])
    kw = dict(heads=1, kv_heads=1, dim=8, vdim=4, silu_inputs=False, decay=torch.ones(1, device=gpu_device))
    with pytest.raises(ValueError, match="beyond the rotation"):
        ops.linear_recurrence(x, 0, 8, 16, batch, st, turn=rotation_table(4, 9.0, 4).to(gpu_device), **kw)
    with pytest.raises(ValueError, match="channels"):
        ops.linear_recurrence(x, 0, 8, 16, batch, st, turn=rotation_table(5, 9.0).to(gpu_device), **kw)
    with pytest.raises(RuntimeError, match="plain operands"):
        ops.linear_recurrence(x, 0, 8, 16, batch, st, turn=rotation_table(4, 9.0).to(gpu_device),
                              **dict(kw, silu_inputs=True))
    with pytest.raises(RuntimeError, match="factor on k"):
        ops.linear_recurrence(x, 0, 8, 16, batch, st, k_scale=0.5, **kw)


# ------------------------------------------------------------------ attention kernels


def test_capped_scores_with_a_window_and_a_sink_in_every_attention_kernel(gpu_device):
    """The float32 kernel and the matrix-core kernels (decode steps with keys split and whole,
    short portions, long portions of every form, mixed steps) against the plain torch
    attention, for caps that bend nearly every score and hardly any, and sinks that take a
    small and a large share (a sink is not capped)."""
    ops = load_hip_ops(gpu_device)
    for dtype in (torch.float32, torch.bfloat16):
        for nq, nkv, hd, window, cap, page in (
                (4, 2, 64, 40, 1.0, 16), (8, 8, 128, 300, 4.0, 16), (6, 1, 96, 17, 30.0, 16),
                (2, 2, 48, 5, 2.0, 64), (4, 4, 64, None, 3.0, 32), (4, 1, 128, 1, 0.5, 16),
                (3, 3, 80, 700, 8.0, 16), (2, 1, 32, 33, 1.5, 8), (4, 2, 128, 128, 2.5, 64)):
            sink = torch.tensor([(-1.0, 2.0, 5.0)[j % 3] for j in range(nq)], device=gpu_device)
            for spans in ([[700, 0, 0, 0], [1, 0, 0, 0]], [[500, 3, 40, 1], [1, 1, 1, 1], [1, 1, 1, 1]],
                          [[90, 1, 0, 33], [2, 40, 7, 1], [200, 1, 60, 1]],
                          [[2100, 0, 0, 0], [1, 0, 0, 0]], [[900, 1200, 0, 0]]):
                if spans[0][0] > 800 and dtype == torch.float32 and hd != 64:
                    continue         # (the long prompts are for the matrix-core kernels)
                scene = Scene(gpu_device, PagedKVNeed(nkv, hd, window), page, 4, dtype=dtype,
                              num_pages=2400 // page + 12)
                for step, sp in enumerate(spans):
                    batch = scene.step(sp)
                    T = batch.num_tokens
                    table = batch.tables[0]
                    k = rnd((T, nkv, hd), step).to(dtype).to(gpu_device)
                    v = rnd((T, nkv, hd), 50 + step).to(dtype).to(gpu_device)
                    q = rnd((T, nq, hd), 90 + step, 2.0).to(dtype).to(gpu_device)
                    ops.kv_store(k, v, batch, table, scene.view)
                    kw = dict(num_heads=nq, num_kv_heads=nkv, head_dim=hd, scale=hd ** -0.5,
                              window=window, sink=sink, softcap=cap)
                    got = ops.paged_attention(q, batch, table, scene.view, **kw)
                    edge = window or 1
                    only = sorted({min(T - 1, x) for x in (0, T - 1, T // 2, 17, 63, 64, edge - 1, edge,
                                                           899, 900, 1999)})
                    want = REF.paged_attention(q, batch, table, scene.view, only=only, **kw)
                    tol = dict(rtol=1e-4, atol=1e-5) if dtype == torch.float32 \
                        else dict(rtol=3e-2, atol=2e-2)
                    err = (got[only].float() - want[only].float()).abs().cpu()
                    allowed = tol["atol"] + tol["rtol"] * want[only].float().abs().cpu()
                    assert bool((err <= allowed).all()), \
                        (f"{dtype}, heads {nq}/{nkv} of {hd}, window {window}, cap {cap}, spans "
                         f"{spans}, step {step}: differ by up to {float(err.max()):.3e}")


# ------------------------------------------------------------------ the parts alone


def attention_part(gpu_device, dtype, width, m, eps=1e-5):
    ctx = part_context(gpu_device, dtype, width)
    rot, head = m["rot"], SoftmaxAttention.padded_head(m["dim"], m["vdim"])
    s = rot.get("scaling")
    ctx.positions["rot"] = build_part(POSITIONS, PartSpec("rope_partial", {
        "dims": rot["dims"], "base": rot["base"], "head_dim": head, "pairs": "neighbours",
        "max_position": 512, "scaling": dict(s, kind="wavelength") if s else None}), ctx)
    return build_part(MIXERS, PartSpec("softmax_attention", {
        "prefix": "x.", "heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"],
        "vdim": m["vdim"], "scale": m["scale"], "position": "rot",
        "window": (m.get("mask") or {}).get("size"), "softcap": m.get("softcap"), "sink": True,
        "qk_norm": "plain", "qk_norm_eps": eps, "wide_output": True}), ctx)


def retention_part(gpu_device, dtype, width, m, eps=1e-5, prefix="x."):
    ctx = part_context(gpu_device, dtype, width)
    ctx.positions["turn"] = build_part(POSITIONS, PartSpec("rope_interleaved", {
        "dims": m["rot"]["dims"], "base": m["rot"]["base"], "pairs": "halves", "max_position": 1024}), ctx)
    return build_part(MIXERS, PartSpec("retention", {
        "prefix": prefix, "heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"],
        "decay": m["decay"], "eps": eps, "position": "turn", "state": "r"}), ctx)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [
    sisepel_attention(heads=4, kv_heads=2, dim=12, vdim=20, scale=0.5, window=70, softcap=2.0, base=1e4,
                      rot_dims=8, scaling=sisepel_scaling(4.0, 1.0, 4.0, 64)),
    sisepel_attention(heads=2, kv_heads=2, dim=24, vdim=8, scale=0.3, window=5, softcap=9.0, base=300.0, rot_dims=24),
    sisepel_attention(heads=3, kv_heads=1, dim=16, vdim=16, scale=0.6, window=1, softcap=1.0, base=50.0, rot_dims=2),
    sisepel_attention(heads=8, kv_heads=2, dim=64, vdim=64, scale=0.2, window=33, softcap=4.0, base=5e5,
                      rot_dims=32, scaling=sisepel_scaling(8.0, 1.0, 2.0, 200)),
    sisepel_attention(heads=4, kv_heads=4, dim=40, vdim=96, scale=0.2, window=100, softcap=None, base=1e6, rot_dims=20),
    sisepel_attention(heads=2, kv_heads=1, dim=128, vdim=112, scale=0.1, window=None, softcap=3.0, base=1e4, rot_dims=128),
], ids=lambda m: f"{m['dim']}-{m['vdim']}")
def test_window_attention_alone_whole_and_cut_around_windows_and_pages(gpu_device, dtype, m):
    width, T = 48, 330
    part = attention_part(gpu_device, dtype, width, m)
    w = load_part(part, dtype, gpu_device, 40)
    h = rnd((T, width), 3).to(dtype)
    want = plain.window_attention(h.double(), w, "x.", m, 1e-5).float()
    for cuts in ([T], [15, 1, 1, 31, 16, 2, 34, 28, 1, 1, 1, 36, 1, 2, 160], [2] * 30 + [270]):
        scene = Scene(gpu_device, part.cache_need(), 16, 1, dtype=dtype, num_pages=30)
        got = run_part_in_steps(part, h.to(gpu_device), scene, cuts)
        close_part(got, want, dtype, dict(rtol=5e-3, atol=5e-4))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("decoded", [False, True])
def test_tokens_just_inside_and_just_outside_a_window(gpu_device, dtype, decoded):
    """One token's value is far larger than the others' (through an input channel that only the
    value projection reads): it shows in every row of its window, the last one included, and in
    none behind it; in a prompt and decoded, for windows inside a page and at a page's border."""
    width, T = 32, 200
    for window, marked in ((50, 103), (32, 70), (1, 9), (33, 16), (16, 0), (7, 1), (64, 63)):
        m = sisepel_attention(heads=2, kv_heads=1, dim=16, vdim=16, scale=0.1, window=window, softcap=3.0,
                              base=1e4, rot_dims=8)
        part = attention_part(gpu_device, dtype, width, m)
        w = load_part(part, dtype, gpu_device, 7)
        for name in ("x.q", "x.k"):
            w[name][:, 0] = 0.0
        part.load(lambda n: w[n].to(torch.float32 if n.endswith("sink") else dtype).to(gpu_device))
        h = rnd((T, width), 5).to(dtype)
        h[:, 0] = 0.0
        quiet = plain.window_attention(h.double(), w, "x.", m, 1e-5).float()
        h[marked, 0] = 1000.0
        want = plain.window_attention(h.double(), w, "x.", m, 1e-5).float()
        last_in = marked + window - 1
        changed = (want - quiet).abs().max(-1).values
        assert float(changed[marked:last_in + 1].min()) > 0.5
        assert torch.equal(want[last_in + 1:], quiet[last_in + 1:])
        head = min(marked + 3, T - 1)
        scene = Scene(gpu_device, part.cache_need(), 16, 1, dtype=dtype, num_pages=20)
        got = run_part_in_steps(part, h.to(gpu_device), scene, [head] + [1] * (T - head) if decoded else [T])
        close_part(got, want, dtype, dict(rtol=5e-3, atol=2e-3))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_key_that_stands_out_a_cap_that_levels_it_and_a_sink_that_wins(gpu_device, dtype):
    """One key hundreds of tokens back matches the last queries (its rotation undone by one pair
    of two that turns hardly at all) and its value alone is loud: without a cap it takes the
    softmax, with a small cap it takes a share like the others'; then sinks far above every
    score silence the outputs, uncapped as they are."""
    width, T, far = 32, 420, 11
    outputs = {}
    for cap in (None, 0.5):
        m = sisepel_attention(heads=2, kv_heads=2, dim=16, vdim=8, scale=1.0, window=500, softcap=cap,
                              base=1e4, rot_dims=2)
        part = attention_part(gpu_device, dtype, width, m)
        w = load_part(part, dtype, gpu_device, 9)
        for name in ("x.q", "x.k"):                   # (the turned pair says nothing)
            w[name].view(2, 16, width)[:, :2] = 0.0
            w[name][:, :2] = 0.0
        w["x.v"] *= 0.1
        w["x.v"][:, 1] = 5.0
        for j in range(2):                            # channel 0 asks, channel 1 answers
            w["x.q"].view(2, 16, width)[j, 5, 0] = 30.0
            w["x.k"].view(2, 16, width)[j, 5, 1] = 30.0
        part.load(lambda n: w[n].to(torch.float32 if n.endswith("sink") else dtype).to(gpu_device))
        h = rnd((T, width), 5, 0.3).to(dtype)
        h[:, :2] = 0.0
        h[-3:, 0] = 1.0
        h[far, 1] = 1.0
        want = plain.window_attention(h.double(), w, "x.", m, 1e-5).float()
        outputs[cap] = want
        for cuts in ([T], [T - 5] + [1] * 5, [200, 2, 150, T - 352]):
            scene = Scene(gpu_device, part.cache_need(), 16, 1, dtype=dtype, num_pages=30)
            got = run_part_in_steps(part, h.to(gpu_device), scene, cuts)
            if dtype == torch.float32:
                torch.testing.assert_close(got, want, rtol=5e-3, atol=2e-3)
            else:      # (rows whose quiet values nearly cancel are rounding for the most part)
                err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()
                assert float(err.median()) < 2e-2 and float(err[-3:].max()) < 4e-2
        loud = part.sink
        part.sink = torch.full_like(loud, 200.0)
        for cuts in ([T], [T - 5] + [1] * 5):
            scene = Scene(gpu_device, part.cache_need(), 16, 1, dtype=dtype, num_pages=30)
            got = run_part_in_steps(part, h.to(gpu_device), scene, cuts)
            assert float(got.abs().max()) < 1e-6 and bool(torch.isfinite(got).all())
    assert float(outputs[None][-3:].abs().max()) > 20 * float(outputs[0.5][-3:].abs().max())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("m", [
    sisepel_retention(dim=8, vdim=12, decay=(0.5, 0.97, 1.0), base=500.0, rot_dims=8),
    sisepel_retention(dim=20, vdim=5, decay=(0.9,), base=100.0, rot_dims=6),
    sisepel_retention(dim=64, vdim=128, decay=(0.99, 0.9375), base=1e4, rot_dims=32),
    sisepel_retention(dim=140, vdim=16, decay=(0.99, 0.0), base=1e6, rot_dims=140),
    sisepel_retention(dim=128, vdim=64, decay=(0.998, 0.96, 0.9), base=1e4, rot_dims=128),
], ids=lambda m: f"{m['dim']}-{m['vdim']}")
def test_retention_alone(gpu_device, dtype, m):
    """Whole (long enough for chunks), cut down to single tokens, and decoded over a stale slot."""
    width, T = 40, 330
    part = retention_part(gpu_device, dtype, width, m)
    w = load_part(part, dtype, gpu_device, 60)
    h = rnd((T, width), 5).to(dtype)
    want = plain.retention(h.double(), w, "x.", m, 1e-5).float()
    for cuts in ([T], [1, 1, 70, 2, 256], [2] * 20 + [129] + [1] * 30 + [131], [150] + [1] * 180):
        scene = Scene(gpu_device, part.cache_need(), 16, 1, num_pages=30)
        scene.view.states["r"].fill_(5.0)
        got = run_part_in_steps(part, h.to(gpu_device), scene, cuts)
        close_part(got, want, dtype, dict(rtol=1e-3, atol=1e-3))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_write_remembered_over_hundreds_of_tokens(gpu_device, dtype):
    """Only one early token writes (the others' keys are zero): what a query reads is that
    write's, turned by the distance and faded by the decay; the norm behind it keeps its
    direction, so a lost state, a wrong distance or another's state shows in full."""
    width, T, at = 24, 700, 3
    m = sisepel_retention(dim=16, vdim=8, decay=(0.99951171875, 0.9990234375), base=1e4, rot_dims=12)
    part = retention_part(gpu_device, dtype, width, m, eps=1e-12)
    w = load_part(part, dtype, gpu_device, 60)
    w["x.k"][:, 1:] = 0.0                              # keys come from channel 0 alone
    part.load(lambda n: w[n].to(dtype).to(gpu_device))
    h = rnd((T, width), 5).to(dtype)
    h[:, 0] = 0.0
    h[at, 0] = 2.0
    want = plain.retention(h.double(), w, "x.", m, 1e-12).float()
    assert float(want[at:].abs().mean(-1).min()) > 0.01 and float(want[:at].abs().max()) == 0.0
    for cuts in ([T], [2, 1, 1] + [64] * 10 + [56], [T - 40] + [1] * 40):
        scene = Scene(gpu_device, part.cache_need(), 16, 1, num_pages=60)
        scene.view.states["r"].fill_(-2.0)
        got = run_part_in_steps(part, h.to(gpu_device), scene, cuts)
        # (at some distance a query may be all but orthogonal to the turned key: what is left
        # of it, blown up by the norm, is rounding)
        err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-3)
        assert float(err[at:].quantile(0.97)) < (2e-3 if dtype == torch.float32 else 4e-2)
        assert float(err[at:].median()) < (2e-4 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pair_of_mixers_and_feed_forwards_alone(gpu_device, dtype):
    width, T = 40, 200
    h = rnd((T, width), 4).to(dtype)
    left = sisepel_attention(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.4, window=20, softcap=3.0,
                             base=1e4, rot_dims=8)
    right = sisepel_retention(dim=12, vdim=20, decay=(0.99, 0.8), base=1e3, rot_dims=12)
    ctx = part_context(gpu_device, dtype, width)
    ctx.positions["rot"] = build_part(POSITIONS, PartSpec("rope_partial", {
        "dims": 8, "base": 1e4, "head_dim": 16, "pairs": "neighbours", "max_position": 512}), ctx)
    ctx.positions["turn"] = build_part(POSITIONS, PartSpec("rope_interleaved", {
        "dims": 12, "base": 1e3, "pairs": "halves", "max_position": 512}), ctx)
    part = build_part(MIXERS, PartSpec("side_by_side", {
        "left": PartSpec("softmax_attention", {
            "prefix": "x.left.", "heads": 4, "kv_heads": 2, "dim": 16, "vdim": 12, "scale": 0.4,
            "position": "rot", "window": 20, "softcap": 3.0, "sink": True, "qk_norm": "plain",
            "qk_norm_eps": 1e-5, "wide_output": True}),
        "right": PartSpec("retention", {"prefix": "x.right.", "heads": 2, "dim": 12, "vdim": 20,
                                        "decay": right["decay"], "eps": 1e-5, "position": "turn"}),
        "left_scale": 0.5, "right_scale": 0.5, "norms": ("x.left.out", "x.right.out"), "norm_eps": 1e-5}), ctx)
    w = load_part(part, dtype, gpu_device, 50)
    want = plain.both_mixers(h.double(), w, "x.", {"left": left, "right": right}, 1e-5).float()
    ops = load_hip_ops(gpu_device)
    scene = Scene(gpu_device, part.cache_need(), 16, 1, dtype=dtype, num_pages=30)
    out = part.forward(h.to(gpu_device), scene.step([T]), scene.view, True)
    assert isinstance(out, NormedPair)
    close_part(ops.normed_pair(out, torch.float32).cpu(), want, dtype, dict(rtol=1e-3, atol=1e-3))
    for ff in (24, 64, 17):
        part = build_part(FEED_FORWARDS, PartSpec("swiglu", {
            "prefix": "x.", "inner_dim": ff, "act": "gelu_tanh", "names": ("gate", "up", "down"),
            "wide_output": True}), ctx)
        w = load_part(part, dtype, gpu_device, 60)
        got = part.forward(h.to(gpu_device), None)
        assert got.dtype == torch.float32
        close_part(got.cpu(), plain.gelu_ff(h.double(), w, "x.").float(), dtype)
    for ff, experts, top, shared in ((12, 6, 2, 20), (8, 5, 5, None), (16, 9, 1, 3), (24, 1, 1, 24)):
        part = build_part(FEED_FORWARDS, PartSpec("routed_experts", {
            "prefix": "x.", "inner_dim": ff, "experts": experts, "top": top, "gated": "silu",
            "router_bias": True, "shared_inner": shared}), ctx)
        w = load_part(part, dtype, gpu_device, 70, sharpen=("x.router",))
        mlp = {"router": {"top": top}, "shared": {"ff": shared} if shared else None}
        want = plain.expert_ff(h.double(), w, "x.", mlp).float()
        got = part.forward(h.to(gpu_device), None).float().cpu()
        if dtype == torch.float32:
            torch.testing.assert_close(got, want, rtol=1e-3, atol=1e-3)
        else:        # (a close call between two experts may go the other way on rounded logits)
            err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()
            assert float(err.quantile(0.95)) < 4e-2


# ------------------------------------------------------------------ the engine


TOL = (2e-4, 1e-4)


def rounding_errors(pcfg, w, requests, ref, seed):
    """What changes of a bfloat16 rounding's size in every matrix do to the plain logits, row
    by row (a tiny random model's norms divide by whatever a sub-layer gives, and a router may
    choose another expert: it can be far more sensitive to rounding than a real one)."""
    g = torch.Generator().manual_seed(seed)
    nudged = {n: t * (1 + 2.0 ** -9 * torch.randn(t.shape, generator=g, dtype=t.dtype))
              if t.is_floating_point() and t.dim() == 2 else t for n, t in w.items()}
    return torch.cat([rms_errors(plain.forward(pcfg, nudged, t).float(), ref[rid])
                      for rid, t in requests.items()])


def check(col, ref, dtype, own=None):
    if dtype == torch.float32:
        return drives.compare(col, ref, *TOL)
    return assert_rows_within_rounding(col, ref, own)


@pytest.fixture(scope="module", params=[(n, d) for n in sorted(SISE)
                                        for d in (torch.float32, torch.bfloat16)],
                ids=lambda p: f"{p[0]}-{str(p[1]).split('.')[-1]}")
def setup(request, tmp_path_factory, gpu_device):
    name, dtype = request.param
    cfg, seed, page = SISE[name]
    d = write_sisepel_model(tmp_path_factory.mktemp(f"sise{name}"), cfg, seed, dtype)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, dtype, gpu_device)
    lengths = [5, 11, 17, 40, 64, 1, 23, 100, 180]
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i) for i, n in enumerate(lengths)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = rounding_errors(pcfg, w, requests, ref, seed) if dtype == torch.bfloat16 else None
    return model, page, requests, ref, lambda col: check(col, ref, dtype, own), (pcfg, w, d, dtype)


def runner_for(model, page, num_pages):
    return ModelRunner(model, page_size=page, num_pages=num_pages, num_slots=4)


def test_whole(setup):
    model, page, requests, ref, judge, _ = setup
    judge(drives.drive_whole(runner_for(model, page, 256 // page), requests))


def test_prefill_then_long_decode(setup):
    model, page, requests, ref, judge, _ = setup
    judge(drives.drive_prefill_then_decode(runner_for(model, page, 256 // page), requests,
                                           tail=150))


def test_portions(setup):
    model, page, requests, ref, judge, _ = setup
    judge(drives.drive_portions(runner_for(model, page, 256 // page), requests))


def test_mixed_with_pages_and_slots_used_again(setup):
    model, page, requests, ref, judge, _ = setup
    runner = runner_for(model, page, 480 // page)
    judge(drives.drive_mixed(runner, requests))
    assert all(pool.num_used == 0 for pool in runner.manager.pools)


def test_preempted_and_recomputed(setup):
    model, page, requests, ref, judge, _ = setup
    judge(drives.drive_preempted(runner_for(model, page, 480 // page), requests))


def test_float32_does_not_depend_on_the_cut(setup):
    model, page, requests, ref, _, (_, _, _, dtype) = setup
    if dtype != torch.float32:
        pytest.skip("float32 only")
    a = drives.drive_whole(runner_for(model, page, 256 // page), requests)
    b = drives.drive_portions(runner_for(model, page, 256 // page), requests)
    c = drives.drive_mixed(runner_for(model, page, 480 // page), requests)
    for rid in requests:
        scale = max(1.0, float(ref[rid].abs().max()))
        for other in (b, c):
            torch.testing.assert_close(a.stacked(rid)[0], other.stacked(rid)[0], rtol=1e-4,
                                       atol=1e-4 * scale)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
def test_layer_shapes_of_a_real_model(gpu_device, tmp_path, dtype):
    """Heads of 128 and 64, a width of 512: the instantiations and products the tiny
    configurations do not reach, whole, in portions and decoded."""
    scaling = sisepel_scaling(8.0, 1.0, 4.0, 128)
    cfg = sisepel_config(width=512, vocab=1000, eps=1e-6, side_dim=64, logit_scale=0.7, layers=[
        sisepel_layer(
            sisepel_attention(heads=8, kv_heads=2, dim=128, vdim=128, scale=0.1, window=64, softcap=15.0,
                              base=5e5, rot_dims=64, scaling=scaling),
            sisepel_retention(dim=128, vdim=128, decay=(0.875, 0.96875, 0.99, 0.998), base=1e4, rot_dims=128),
            sisepel_dense(768)),
        sisepel_layer(
            sisepel_attention(heads=4, kv_heads=4, dim=64, vdim=64, scale=0.2, window=100, softcap=5.0,
                              base=1e4, rot_dims=64),
            sisepel_retention(dim=64, vdim=64, decay=(0.9, 0.95, 0.98, 0.99), base=1e4, rot_dims=32),
            sisepel_moe(ff=128, experts=8, top=2, shared=256))])
    d = write_sisepel_model(tmp_path, cfg, 5, dtype, std=0.04)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, dtype, gpu_device)
    requests = {"a": random_prompt(300, 1000, 1), "b": random_prompt(37, 1000, 2)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = rounding_errors(pcfg, w, requests, ref, 5) if dtype == torch.bfloat16 else None
    check(drives.drive_whole(runner_for(model, 16, 24), requests), ref, dtype, own)
    check(drives.drive_prefill_then_decode(runner_for(model, 16, 24), requests, tail=20), ref, dtype, own)
    check(drives.drive_portions(runner_for(model, 16, 24), requests), ref, dtype, own)


def plain_greedy(pcfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(plain.forward(pcfg, w, tokens)[-1].argmax()))
    return tokens[len(prompt):]


def test_greedy_generation_however_the_work_is_cut(setup):
    """LLMEngine.generate: scheduler, captured decode graphs, decode steps launched ahead,
    chunked prefill, preemption by recomputation."""
    model, page, requests, ref, _, (pcfg, w, d, dtype) = setup
    if dtype != torch.float32:
        pytest.skip("greedy tokens are compared in float32")
    prompts = [requests[r] for r in ("r0", "r1", "r2", "r5", "r6", "r3")]
    expected = [plain_greedy(pcfg, w, p, 10) for p in prompts]
    sp = SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True)
    base = dict(model=str(d), max_model_len=128, dtype=dtype, kvcache_block_size=page,
                num_kvcache_blocks=64, max_num_seqs=8, max_num_batched_tokens=64,
                chunked_prefill=True)
    for kw in (dict(), dict(enforce_eager=True), dict(max_num_batched_tokens=7),
               dict(max_num_seqs=1), dict(chunked_prefill=False),
               dict(num_kvcache_blocks=-(-50 // page) + 3)):
        engine = LLMEngine(model, Config(**{**base, **kw}))
        assert engine.generate(prompts, sp, use_tqdm=False) == expected, kw
        assert all(p.num_used == 0 for p in engine.runner.manager.pools)
        if not kw:
            assert engine.runner.graphs, "decode steps were not captured"


def test_greedy_generation_in_bfloat16_through_captured_graphs(gpu_device, tmp_path):
    """The bfloat16 decode path as it serves, over a window's and a page's length and with
    slots and pages used again: captured graphs against the eager step, on later replays too."""
    cfg, seed, page = SISE["A"]
    d = write_sisepel_model(tmp_path, cfg, seed, torch.bfloat16)
    _, model = load_model(d, torch.bfloat16, gpu_device)
    prompts = [random_prompt(n, cfg["vocab"], 7 + n) for n in (9, 30, 2, 17, 1, 5)]
    sp = SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True)
    base = dict(model=str(d), max_model_len=128, dtype=torch.bfloat16, kvcache_block_size=16,
                num_kvcache_blocks=64, max_num_seqs=4, max_num_batched_tokens=64,
                chunked_prefill=True)
    eager = LLMEngine(model, Config(**base, enforce_eager=True)).generate(prompts, sp, use_tqdm=False)
    engine = LLMEngine(model, Config(**base))
    assert engine.runner.graphs or engine.generate(prompts[:1], sp, use_tqdm=False)
    assert engine.generate(prompts, sp, use_tqdm=False) == eager
    assert engine.generate(prompts, sp, use_tqdm=False) == eager


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["float32", "bfloat16"])
def test_sizes_that_are_multiples_of_nothing(gpu_device, tmp_path, dtype):
    """Odd head sizes, a width and inner sizes that are multiples of no tile or vector width:
    the products fall to the multiply-add kernels and heads are padded."""
    cfg = sisepel_config(width=34, vocab=61, eps=1e-6, side_dim=13, logit_scale=1.7, layers=[
        sisepel_layer(
            sisepel_attention(heads=3, kv_heads=3, dim=5, vdim=7, scale=0.8, window=11, softcap=2.0,
                              base=800.0, rot_dims=4),
            sisepel_retention(dim=7, vdim=11, decay=(0.9, 0.97, 0.5), base=90.0, rot_dims=6),
            sisepel_dense(29)),
        sisepel_layer(
            sisepel_attention(heads=3, kv_heads=1, dim=9, vdim=3, scale=0.6, window=40, softcap=6.0,
                              base=80.0, rot_dims=8, scaling=sisepel_scaling(3.0, 1.0, 5.0, 33)),
            sisepel_retention(dim=3, vdim=5, decay=(0.99,), base=90.0, rot_dims=2),
            sisepel_moe(ff=13, experts=3, top=2, shared=7))])
    d = write_sisepel_model(tmp_path, cfg, 12, dtype)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, dtype, gpu_device)
    requests = {"a": random_prompt(90, 61, 1), "b": random_prompt(37, 61, 2), "c": random_prompt(1, 61, 3)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = rounding_errors(pcfg, w, requests, ref, 5) if dtype == torch.bfloat16 else None
    check(drives.drive_whole(runner_for(model, 16, 12), requests), ref, dtype, own)
    check(drives.drive_portions(runner_for(model, 16, 12), requests), ref, dtype, own)
    check(drives.drive_mixed(runner_for(model, 16, 16), requests), ref, dtype, own)
