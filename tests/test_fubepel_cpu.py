"""Fubepel on the CPU: configuration, the model as data, the plain implementation's own pins
(each mechanism against a closed form or a crafted case), the cache manager's kept first
pages, and the engine's cache manager, batch builder and step function (with the plain torch
kernel references in place of the HIP kernels) against the plain whole-sequence
implementation, float32."""

import copy
import math

import pytest
import torch

import drives
from helpers import (FUBE, FUBE_A, FUBE_B, FUBE_C, fubepel_attention, fubepel_config,
                     fubepel_delta, fubepel_dense, fubepel_latent, random_prompt,
                     write_fubepel_model)
from kernel_refs import TorchOps
from plain import fubepel_plain as plain
from tokensprint_amd.cache import CacheManager
from tokensprint_amd.cache.pages import GroupLayout
from tokensprint_amd.cache.storage import group_runs
from tokensprint_amd.config import ConfigError, FubepelConfig
from tokensprint_amd.config.registry import architecture_names, get_architecture
from tokensprint_amd.engine import ModelRunner
from tokensprint_amd.engine.assemble import build_model, load_model
from tokensprint_amd.parts.base import (POSITIONS, BuildContext, PagedKVNeed, PagedLatentNeed,
                                        SlotStateNeed, build_part)
from tokensprint_amd.models.spec import PartSpec


@pytest.fixture(scope="module", params=sorted(FUBE))
def setup(request, tmp_path_factory):
    cfg, seed, page = FUBE[request.param]
    d = write_fubepel_model(tmp_path_factory.mktemp(f"fube{request.param}"), cfg, seed,
                            torch.float32)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, "float32", "cpu", ops=TorchOps())
    lengths = [5, 11, 17, 40, 64, 1, 23]
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i) for i, n in enumerate(lengths)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    return model, page, requests, ref


def runner_for(model, page, num_pages):
    return ModelRunner(model, page_size=page, num_pages=num_pages, num_slots=4)


TOL = (2e-4, 5e-5)


def test_whole(setup):
    model, page, requests, ref = setup
    drives.compare(drives.drive_whole(runner_for(model, page, 64 // page + 1), requests),
                   ref, *TOL)


def test_prefill_then_decode(setup):
    model, page, requests, ref = setup
    drives.compare(drives.drive_prefill_then_decode(runner_for(model, page, 64 // page + 1),
                                                    requests), ref, *TOL)


def test_portions(setup):
    model, page, requests, ref = setup
    drives.compare(drives.drive_portions(runner_for(model, page, 64 // page + 1), requests),
                   ref, *TOL)


def test_mixed_with_pages_and_slots_used_again(setup):
    model, page, requests, ref = setup
    runner = runner_for(model, page, 160 // page)
    drives.compare(drives.drive_mixed(runner, requests), ref, *TOL)
    assert all(pool.num_used == 0 for pool in runner.manager.pools)
    assert runner.manager.slots.num_free == 4


def test_preempted_and_recomputed(setup):
    model, page, requests, ref = setup
    runner = runner_for(model, page, 160 // page)
    drives.compare(drives.drive_preempted(runner, requests), ref, *TOL)


# ------------------------------------------------------------------ configuration, spec


def test_config_reads_every_size():
    cfg = FubepelConfig.from_dict(FUBE_A)
    assert (cfg.width, cfg.vocab_size, cfg.eps, cfg.embed_scale, cfg.side_dim, len(cfg.layers)) == \
        (40, 97, 1e-5, 2.5, 6, 4)
    m = cfg.layers[0].mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, m.rot_base, m.rot_dims,
            m.kv_from) == (3, 8, 4, 10, 20, 0.4, 10000.0, 4, None)
    a = cfg.layers[1].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.keep_first) == \
        (4, 2, 12, 20, 0.6, 3, 2)
    d = cfg.layers[2].mixer
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.conv) == (4, 2, 8, 12, 3)
    assert cfg.layers[3].mixer.kv_from == 0
    assert (cfg.layers[0].mlp.ff, cfg.layers[0].mlp.limit) == (24, 0.7) and cfg.layers[2].mlp is None
    assert FubepelConfig.from_dict(FUBE_C).side_dim is None
    assert FubepelConfig.from_dict(FUBE_C).layers[2].mixer.window is None
    bare = copy.deepcopy(FUBE_A)
    del bare["embedding"], bare["layers"][1]["mixer"]["mask"]["keep_first"]
    bare["layers"][3]["mixer"]["kv_from"] = None
    cfg = FubepelConfig.from_dict(bare)
    assert cfg.embed_scale == 1.0 and cfg.layers[1].mixer.keep_first == 0
    assert cfg.layers[1].mixer.window == 3 and cfg.layers[3].mixer.kv_from is None
    assert "Fubepel" in architecture_names()


@pytest.mark.parametrize("path, value, message", [
    (("layers", 0, "type"), "mamba2", "Fubepel has"),
    (("layers", 0, "mixer", "kv_rank"), 0, "kv_rank"),
    (("layers", 0, "mixer", "rot", "dims"), 3, "rot.dims"),
    (("layers", 0, "mixer", "rot", "dims"), 6, "rot.dims"),
    (("layers", 0, "mlp", "kind"), "moe", "dense"),
    (("layers", 0, "mlp", "limit"), 0.0, "limit"),
    (("layers", 1, "mixer", "kv_heads"), 3, "multiple"),
    (("layers", 1, "mixer", "mask", "size"), -1, "size"),
    (("layers", 1, "mixer", "mask", "keep_first"), -2, "keep_first"),
    (("layers", 2, "mixer", "conv"), 2.5, "conv"),
    (("layers", 3, "mixer", "kv_from"), 3, "no earlier layer"),
    (("layers", 3, "mixer", "kv_from"), 4, "no earlier layer"),
    (("layers", 3, "mixer", "kv_from"), 1, "no latents of its own"),
    (("layers", 3, "mixer", "kv_rank"), 24, "rank or rotation"),
    (("layers", 3, "mixer", "rot", "base"), 50.0, "rank or rotation"),
    (("token_side", "dim"), 0, "token_side"),
    (("norm", "eps"), 0, "eps"),
])
def test_config_errors(path, value, message):
    cfg = copy.deepcopy(FUBE_A)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=message):
        FubepelConfig.from_dict(cfg)


def test_a_reader_of_a_reader_is_refused():
    cfg = copy.deepcopy(FUBE_B)
    cfg["layers"][4]["mixer"]["kv_from"] = 3
    with pytest.raises(ConfigError, match="no latents of its own"):
        FubepelConfig.from_dict(cfg)


def test_caches_and_tensors_follow_the_mixers():
    arch = get_architecture("Fubepel")
    spec = arch.build_spec(arch.parse_config(FUBE_B))
    assert [run.cache_of for run in spec.order] == [None, None, None, 1, 1, None]
    _, model = build_model(FUBE_B, "float32", "cpu", ops=TorchOps())
    needs = model.cache_needs()
    # heads are laid out in the larger of key and value size rounded up to 16
    assert needs[0] == PagedKVNeed(1, 32, 37, 21)
    assert needs[1] == PagedLatentNeed(48) and needs[5] == PagedLatentNeed(32)
    assert needs[3] is None and needs[4] is None
    assert needs[2] == (SlotStateNeed((0, 2 * 48 + 24), torch.float32, "delta.conv"),
                        SlotStateNeed((3, 16, 8), torch.float32, "delta"))
    groups, _ = group_runs(needs)
    assert [(g.window, g.keep_first, g.runs) for g in groups] == \
        [(37, 21, (0,)), (None, 0, (1,)), (None, 0, (5,))]
    decls = model.tensor_decls()
    assert decls["side.embed"].shape == (131, 6 * 16) and decls["l4.side.gate"].shape == (16, 72)
    assert decls["l1.mix.dkv"].shape == (48, 72) and decls["l4.mix.q"].shape == (24, 72)
    assert {"l3.mix.sink", "l3.mix.uk", "l0.norm2", "l5.side.norm", "embed", "head", "final.norm"} \
        <= set(decls)
    assert not {"l3.mix.dkv", "l3.mix.dkv.norm", "l1.norm2", "l1.mlp.up", "l0.mix.q.norm", "l0.mix.sink"} \
        & set(decls)
    _, without = build_model(FUBE_C, "float32", "cpu", ops=TorchOps())
    assert not [n for n in without.tensor_decls() if "side" in n]


def test_random_weights_fit_the_declarations(tmp_path):
    for name, (cfg, seed, _) in FUBE.items():
        d = write_fubepel_model(tmp_path / name, cfg, seed, torch.bfloat16)
        _, w = plain.read_model_dir(d)
        _, model = load_model(d, "bfloat16", "cpu", ops=TorchOps())
        assert set(w) == set(model.tensor_decls())
        # the side table is no part of what a step reads whole
        assert all(t.data_ptr() != model.blocks[0].side.table.data_ptr()
                   for part in model.parts() for t in part.step_read_tensors()) \
            if cfg.get("token_side") else True


def test_layer_outputs_follow_the_plain_stream(tmp_path):
    """The residual stream after every layer, float32."""
    cfg, seed, page = FUBE["B"]
    d = write_fubepel_model(tmp_path, cfg, seed, torch.float32)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, "float32", "cpu", ops=TorchOps())
    tokens = random_prompt(30, cfg["vocab"], 5)
    want, got = [], []
    plain.forward(pcfg, w, tokens, want)
    for block in model.blocks:
        def wrapped(resid, *a, _forward=block.forward, **k):
            out = _forward(resid, *a, **k)
            got.append(out[0].clone())
            return out
        block.forward = wrapped
    drives.drive_whole(runner_for(model, page, 4), {"a": tokens})
    assert len(got) == len(want) == 6
    for g, x in zip(got, want):
        torch.testing.assert_close(g, x.float(), rtol=3e-4, atol=3e-4)


# ------------------------------------------------------------------ kept first pages


def test_a_window_group_keeps_its_first_pages():
    """Window 10 beside 9 kept tokens on pages of 4: pages 0 to 2 stay for good, later ones go
    back as the window passes, and every position a query sees is on a page all along."""
    layout = GroupLayout(1, 8, 10, (0,), keep_first=9)
    m = CacheManager([layout], 4, 15, 2)
    rc = m.admit("a")
    for n in [3, 2, 9, 1, 1, 5, 20, 1, 1, 1, 30, 7]:
        new = rc.num_tokens + n
        start = rc.num_tokens
        assert m.can_extend(rc, new)
        m.extend(rc, new)
        m.check()
        for q in range(start, new):
            seen = set(range(max(0, q - 9), q + 1)) | set(range(min(9, q + 1)))
            assert all(rc.tables[0][p // 4] >= 0 for p in seen), (start, q)
    # 3 kept pages, and what the last portion's first query could still see
    held = [i for i, p in enumerate(rc.tables[0]) if p >= 0]
    assert held[:3] == [0, 1, 2] and min(h for h in held if h > 2) >= (rc.num_tokens - 7 - 9) // 4
    m.free(rc)
    m.check()
    assert m.pools[0].num_used == 0


@pytest.mark.parametrize("seed", range(4))
def test_kept_pages_in_random_orders_lose_nothing(seed):
    g = torch.Generator().manual_seed(seed)

    def draw(lo, hi):
        return int(torch.randint(lo, hi, (1,), generator=g))
    layouts = [GroupLayout(1, 8, draw(1, 20), (0,), keep_first=draw(0, 15)),
               GroupLayout(1, 8, None, (1,)), GroupLayout(1, 8, draw(1, 6), (2,), keep_first=draw(1, 30))]
    P = draw(1, 6)
    m = CacheManager(layouts, P, 60, 3)
    live = {}
    for i in range(200):
        if len(live) < 3 and draw(0, 3) == 0:
            live[i] = m.admit(i)
        for rid, rc in list(live.items()):
            new = rc.num_tokens + draw(1, 9)
            if not m.can_extend(rc, new):
                continue
            start = rc.num_tokens
            m.extend(rc, new)
            for gi, lay in enumerate(layouts):
                for q in (start, new - 1):
                    lo = 0 if lay.window is None else max(0, q - lay.window + 1)
                    for p in list(range(lo, q + 1)) + list(range(min(lay.keep_first, q + 1))):
                        assert rc.tables[gi][p // P] >= 0
            if draw(0, 4) == 0 and new - start > 1:
                m.shrink(rc, new - 1)
            if draw(0, 12) == 0:
                m.free(live.pop(rid))
        m.check()
    for rc in live.values():
        m.free(rc)
    m.check()
    assert all(p.num_used == 0 for p in m.pools)


# ------------------------------------------------------------------ the plain side's pins


def test_plain_window_with_kept_first_tokens():
    seen = plain.visible(9, 3, 2)
    for i in range(9):
        assert [j for j in range(9) if seen[i, j]] == \
            sorted({j for j in range(i + 1) if j > i - 3 or j < 2})
    assert plain.visible(4)[3].tolist() == [True] * 4 and plain.visible(4)[0].tolist() == [True, False, False, False]


def test_plain_sink_takes_its_share():
    s = torch.tensor([[[0.0, math.log(3.0)], [1.0, 2.0]]], dtype=torch.float64)
    p = plain.softmax_with_sink(s, plain.visible(2), torch.tensor([math.log(2.0)], dtype=torch.float64))
    assert torch.allclose(p[0, 0], torch.tensor([1 / 3, 0.0], dtype=torch.float64))
    e = math.e
    assert torch.allclose(p[0, 1], torch.tensor([e, e * e], dtype=torch.float64) / (e + e * e + 2))
    # without a sink an ordinary softmax
    assert torch.allclose(plain.softmax_with_sink(s, plain.visible(2))[0, 1],
                          torch.softmax(s[0, 1], 0))


def test_plain_rotation_pairs_halves():
    x = torch.arange(12, dtype=torch.float64).view(2, 1, 6)
    y = plain.turn_halves(x, 100.0, 4)
    assert torch.equal(y[0], x[0]) and torch.equal(y[1, 0, 4:], x[1, 0, 4:])
    for i, freq in ((0, 1.0), (1, 100.0 ** -0.5)):
        u, v = x[1, 0, i], x[1, 0, i + 2]
        assert y[1, 0, i] == pytest.approx(float(u * math.cos(freq) - v * math.sin(freq)))
        assert y[1, 0, i + 2] == pytest.approx(float(v * math.cos(freq) + u * math.sin(freq)))


def test_the_engines_layout_of_a_rotation_by_halves():
    ctx = BuildContext(ops=TorchOps(), dtype=torch.float32, device=torch.device("cpu"), width=8)
    enc = build_part(POSITIONS, PartSpec("rope_interleaved", {"dims": 6, "base": 50.0, "pairs": "halves"}), ctx)
    layout = enc.layout(8)
    assert layout == [0, 3, 1, 4, 2, 5, 6, 7]
    x = torch.randn(5, 3, 8, generator=torch.Generator().manual_seed(1), dtype=torch.float64)
    y = x[..., layout].float().contiguous()
    TorchOps().rotate_interleaved_inplace(y, torch.arange(5, dtype=torch.int32), enc.frequencies(), 6)
    torch.testing.assert_close(y, plain.turn_halves(x, 50.0, 6)[..., layout].float(), rtol=1e-5, atol=1e-5)
    with pytest.raises(RuntimeError, match="layout"):
        enc.apply(y, None, torch.arange(5, dtype=torch.int32))
    plain_order = build_part(POSITIONS, PartSpec("rope_interleaved", {"dims": 6, "base": 50.0}), ctx)
    assert plain_order.layout(8) == list(range(8))


def test_plain_delta_rule_by_hand():
    """One head of one key and one value channel: S is a number."""
    q, k = torch.tensor([2.0, 0.5, 1.0]), torch.tensor([1.0, 0.0, 0.5])
    v, beta, g = torch.tensor([3.0, 4.0, -1.0]), torch.tensor([1.0, 0.5, 0.25]), torch.tensor([0.5, 0.5, 0.25])
    S, want = 0.0, []
    for t in range(3):
        S = float(g[t]) * S
        S = S + float(k[t]) * float(beta[t]) * (float(v[t]) - S * float(k[t]))
        want.append(S * float(q[t]))
    got = plain.delta_rule(*(x.view(3, 1, 1).double() for x in (q, k, v)), beta.view(3, 1).double(),
                           g.view(3, 1).double())
    assert got.view(-1).tolist() == pytest.approx(want)


def test_plain_convolution_starts_behind_zeros():
    x = torch.tensor([[1.0], [2.0], [4.0]])
    assert plain.short_conv(x, torch.tensor([[10.0, 100.0, 1.0]])).view(-1).tolist() == [1.0, 102.0, 214.0]
    assert torch.equal(plain.short_conv(x, torch.tensor([[3.0]])), 3 * x)


def test_plain_clamped_unit_and_side_input():
    eye = torch.eye(2, dtype=torch.float64)
    w = {"m.gate": eye, "m.up": eye, "m.down": eye}
    h = torch.tensor([[5.0, -3.0], [0.5, 0.25]], dtype=torch.float64)
    g, u = [[2.0, -3.0], [0.5, 0.25]], [[2.0, -2.0], [0.5, 0.25]]
    got = plain.clamped_ff(h, w, "m.", 2.0)
    for t in range(2):
        for j in range(2):
            want = g[t][j] / (1 + math.exp(-1.702 * g[t][j])) * (u[t][j] + 1)
            assert float(got[t, j]) == pytest.approx(want)
    w = {"side.embed": torch.tensor([[1.0, 2.0, 3.0, 4.0], [5.0, 6.0, 7.0, 8.0]], dtype=torch.float64),
         "l1.side.gate": eye, "l1.side.proj": eye, "l1.side.norm": torch.tensor([1.0, 10.0], dtype=torch.float64)}
    y = plain.side_input(torch.tensor([[1.0, -2.0]], dtype=torch.float64), w, [1], 1, 2, 0.0)
    a = [0.8411919906 * 7, -0.0454023059 * 8]                 # gelu_tanh(1), gelu_tanh(-2)
    rms = math.sqrt((a[0] ** 2 + a[1] ** 2) / 2)
    assert y[0].tolist() == pytest.approx([a[0] / rms, 10 * a[1] / rms], rel=1e-6)


# ------------------------------------------------------------------ odd arrangements


@pytest.mark.parametrize("layers, page", [
    ([fubepel_delta(heads=2, kv_heads=1, dim=6, vdim=5, conv=2, mlp=None)], 4),
    ([fubepel_attention(heads=2, kv_heads=2, dim=6, vdim=6, scale=0.5, window=4, keep_first=40,
                        mlp=fubepel_dense(8, 1.0))], 1),
    ([fubepel_latent(heads=1, dim=2, rot_dim=6, vdim=3, kv_rank=7, scale=0.5, base=30.0, mlp=None)], 16),
    ([fubepel_attention(heads=2, kv_heads=1, dim=4, vdim=4, scale=0.9, window=2, keep_first=5, mlp=None),
      fubepel_attention(heads=4, kv_heads=1, dim=4, vdim=4, scale=0.9, window=2, keep_first=6, mlp=None),
      fubepel_attention(heads=1, kv_heads=1, dim=4, vdim=4, scale=0.9, window=7, keep_first=5, mlp=None)], 3),
], ids=["recurrence only", "kept beyond the request", "latents only", "groups that differ in what they keep"])
def test_models_of_one_kind_of_layer(tmp_path, layers, page):
    cfg = fubepel_config(width=16, vocab=40, eps=1e-6, embed_scale=1.5, side_dim=3, layers=layers)
    d = write_fubepel_model(tmp_path, cfg, 3, torch.float32)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, "float32", "cpu", ops=TorchOps())
    requests = {"a": random_prompt(37, 40, 1), "b": random_prompt(20, 40, 2), "c": random_prompt(1, 40, 3)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    drives.compare(drives.drive_portions(runner_for(model, page, -(-48 // page)), requests), ref, *TOL)
    drives.compare(drives.drive_mixed(runner_for(model, page, -(-100 // page)), requests), ref, *TOL)
