"""Sisepel on the CPU: configuration, the model as data, the plain implementation's own pins
(each mechanism against a closed form or a crafted case), rotations as the engine lays them
out, sandwich-norm layers between blocks of other kinds, and the engine's cache manager, batch
builder and step function (with the plain torch kernel references in place of the HIP
kernels) against the plain whole-sequence implementation, float32."""

import copy
import math

import pytest
import torch

import drives
from helpers import (SISE, SISE_A, SISE_B, SISE_C, random_prompt, sisepel_attention,
                     sisepel_config, sisepel_dense, sisepel_layer, sisepel_moe,
                     sisepel_retention, write_sisepel_model)
from kernel_refs import TorchOps
from plain import sisepel_plain as plain
from tokensprint_amd.cache.storage import group_runs
from tokensprint_amd.config import ConfigError, SisepelConfig
from tokensprint_amd.config.registry import architecture_names, get_architecture
from tokensprint_amd.engine import ModelRunner
from tokensprint_amd.engine.assemble import build_model, load_model
from tokensprint_amd.kernels.stream import NormAhead
from tokensprint_amd.models.model import Model
from tokensprint_amd.models.spec import LayerSpec, ModelSpec, PartSpec, Run
from tokensprint_amd.parts.base import (MIXERS, NORMS, POSITIONS, BuildContext, PagedKVNeed,
                                        SlotStateNeed, build_part)


@pytest.fixture(scope="module", params=sorted(SISE))
def setup(request, tmp_path_factory):
    cfg, seed, page = SISE[request.param]
    d = write_sisepel_model(tmp_path_factory.mktemp(f"sise{request.param}"), cfg, seed,
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
    cfg = SisepelConfig.from_dict(SISE_A)
    assert (cfg.width, cfg.vocab_size, cfg.eps, cfg.logit_scale, cfg.side_dim, len(cfg.layers)) == \
        (40, 97, 1e-5, 0.25, 6, 3)
    a, r = cfg.layers[0].mixer.left, cfg.layers[0].mixer.right
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.softcap) == \
        (4, 2, 12, 20, 0.9, 3, 1.5)
    assert (a.rot.base, a.rot.dims) == (10000.0, 8)
    s = a.rot.scaling
    assert (s.factor, s.low, s.high, s.original) == (3.0, 1.0, 4.0, 40.0)
    assert (r.heads, r.dim, r.vdim, r.decay) == (3, 8, 12, (0.5, 0.97, 1.0))
    assert (r.rot.base, r.rot.dims, r.rot.scaling) == (500.0, 8, None)
    assert cfg.layers[0].mlp.ff == 24 and cfg.layers[2].mlp is None
    m = cfg.layers[1].mlp
    assert (m.ff, m.experts, m.top, m.shared_ff) == (12, 6, 2, 20)
    assert SisepelConfig.from_dict(SISE_B).layers[0].mlp.shared_ff is None
    assert SisepelConfig.from_dict(SISE_B).layers[1].mixer.left.window is None
    assert SisepelConfig.from_dict(SISE_C).side_dim is None
    assert "Sisepel" in architecture_names()


def test_what_a_config_leaves_out_takes_its_mechanism_along():
    bare = copy.deepcopy(SISE_A)
    left = bare["layers"][0]["mixer"]["left"]
    del bare["logit_scale"], bare["token_side"], left["mask"], left["softcap"], left["rot"]
    bare["layers"][1]["mixer"]["left"]["rot"]["scaling"] = None
    bare["layers"][1]["mlp"]["shared"] = None
    del bare["layers"][2]["mlp"]
    cfg = SisepelConfig.from_dict(bare)
    assert cfg.logit_scale == 1.0 and cfg.side_dim is None
    a = cfg.layers[0].mixer.left
    assert a.window is None and a.softcap is None and a.rot is None
    assert cfg.layers[1].mixer.left.rot.scaling is None and cfg.layers[1].mlp.shared_ff is None
    assert cfg.layers[2].mlp is None
    _, model = build_model(bare, "float32", "cpu", ops=TorchOps())
    assert not [n for n in model.tensor_decls() if "side" in n or "shared" in n or "l2.mlp" in n
                or n in ("l2.norm2", "l2.norm2b")]
    assert model.blocks[0].mixer.left.position is None
    assert "softcap" not in model.blocks[0].mixer.left.score_options


@pytest.mark.parametrize("path, value, message", [
    (("layers", 0, "type"), "retention", "Sisepel has"),
    (("layers", 0, "mixer", "left", "kv_heads"), 3, "multiple"),
    (("layers", 0, "mixer", "left", "dim"), 0, "dim"),
    (("layers", 0, "mixer", "left", "scale"), 0.0, "scale"),
    (("layers", 0, "mixer", "left", "softcap"), -1.0, "softcap"),
    (("layers", 0, "mixer", "left", "mask", "size"), 0, "size"),
    (("layers", 0, "mixer", "left", "rot", "dims"), 7, "rot.dims"),
    (("layers", 0, "mixer", "left", "rot", "dims"), 14, "rot.dims"),
    (("layers", 0, "mixer", "left", "rot", "scaling", "factor"), 0, "factor"),
    (("layers", 0, "mixer", "left", "rot", "scaling", "high"), 0.5, "below low"),
    (("layers", 0, "mixer", "right", "decay"), [0.5, 0.9], "one number per head"),
    (("layers", 0, "mixer", "right", "rot", "dims"), 10, "rot.dims"),
    (("layers", 0, "mixer", "right", "rot", "scaling"), {"factor": 2.0, "low": 1.0, "high": 2.0,
                                                         "original": 8}, "has none"),
    (("layers", 0, "mixer", "right", "rot"), None, "right.rot"),
    (("layers", 0, "mlp", "kind"), "glu", "dense and moe"),
    (("layers", 1, "mlp", "router", "top"), 7, "cannot give"),
    (("layers", 1, "mlp", "shared", "ff"), 0, "shared"),
    (("token_side", "dim"), 0, "token_side"),
    (("logit_scale",), "1", "logit_scale"),
    (("norm", "eps"), 0, "eps"),
    (("layers",), [], "non-empty"),
])
def test_config_errors(path, value, message):
    cfg = copy.deepcopy(SISE_A)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError, match=message):
        SisepelConfig.from_dict(cfg)


def test_caches_and_tensors_follow_the_mixers():
    _, model = build_model(SISE_B, "float32", "cpu", ops=TorchOps())
    needs = model.cache_needs()
    # heads are laid out in the larger of key and value size rounded up to 16
    assert needs[0] == (PagedKVNeed(1, 32, 37), SlotStateNeed((4, 16, 24), torch.float32, "retention"))
    assert needs[1] == (PagedKVNeed(5, 16, None), SlotStateNeed((2, 10, 10), torch.float32, "retention"))
    assert needs[3] == (PagedKVNeed(1, 48, 16), SlotStateNeed((1, 6, 9), torch.float32, "retention"))
    groups, _ = group_runs(needs)
    assert [(g.window, g.runs) for g in groups] == [(37, (0,)), (None, (1,)), (50, (2,)), (16, (3,))]
    decls = model.tensor_decls()
    assert decls["side.embed"].shape == (131, 4 * 16) and decls["l3.side.gate"].shape == (16, 72)
    assert decls["l0.mix.left.q"].shape == (144, 72) and decls["l0.mix.left.v"].shape == (16, 72)
    assert decls["l0.mix.right.k"].shape == (64, 72) and decls["l0.mix.right.g"].shape == (96, 72)
    assert decls["l0.mlp.router.b"].shape == (5,) and decls["l2.mlp.shared.down"].shape == (72, 4)
    assert {"l0.mix.left.sink", "l0.mix.left.out", "l0.mix.right.out", "l2.norm2b", "l3.norm1b",
            "l1.side.norm", "embed", "head", "final.norm"} <= set(decls)
    assert not {"l1.norm2", "l1.mlp.up", "l0.mix.left.q.norm", "l0.mlp.shared.up",
                "l0.mix.right.norm"} & set(decls)
    # rotations are shared by the layers that use the same one
    arch = get_architecture("Sisepel")
    twice = copy.deepcopy(SISE_A)
    twice["layers"][1]["mixer"] = twice["layers"][0]["mixer"]
    assert len(arch.build_spec(arch.parse_config(twice)).positions) == 4
    assert len(arch.build_spec(arch.parse_config(SISE_A)).positions) == 6


def test_random_weights_fit_the_declarations(tmp_path):
    for name, (cfg, seed, _) in SISE.items():
        d = write_sisepel_model(tmp_path / name, cfg, seed, torch.bfloat16)
        _, w = plain.read_model_dir(d)
        _, model = load_model(d, "bfloat16", "cpu", ops=TorchOps())
        assert set(w) == set(model.tensor_decls())
        # a step reads both mixers' weights and their norms whole, the tables not
        read = {t.data_ptr() for part in model.parts() for t in part.step_read_tensors()}
        mixer = model.blocks[0].mixer
        assert {mixer.w_left.data_ptr(), mixer.left.w_qkv.data_ptr(), mixer.right.w_in.data_ptr()} <= read
        assert not any(p.table.data_ptr() in read for p in model.ctx.positions.values()
                       if getattr(p, "table", None) is not None)


def test_layer_outputs_follow_the_plain_stream(tmp_path):
    """The residual stream after every layer, float32."""
    cfg, seed, page = SISE["B"]
    d = write_sisepel_model(tmp_path, cfg, seed, torch.float32)
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
    assert len(got) == len(want) == 4
    for g, x in zip(got, want):
        torch.testing.assert_close(g, x.float(), rtol=3e-4, atol=3e-4)


def test_the_factor_on_the_logits_is_in_the_final_norm():
    ctx = BuildContext(ops=TorchOps(), dtype=torch.float32, device=torch.device("cpu"), width=3)
    part = build_part(NORMS, PartSpec("rmsnorm", {"dim": 3, "eps": 0.0, "weight": "n", "scale": 0.5}), ctx)
    part.load(lambda n: torch.tensor([1.0, 2.0, 4.0]))
    x = torch.tensor([[3.0, 3.0, -3.0]])
    torch.testing.assert_close(part.forward(x), torch.tensor([[0.5, 1.0, -2.0]]))


# ------------------------------------------------------------------ the plain side's pins


def test_plain_window():
    seen = plain.visible(9, 3)
    for i in range(9):
        assert [j for j in range(9) if seen[i, j]] == [j for j in range(i + 1) if j > i - 3]
    assert plain.visible(4)[3].tolist() == [True] * 4
    assert plain.visible(3, 1).tolist() == torch.eye(3, dtype=torch.bool).tolist()


def test_plain_cap_bends_scores_and_leaves_the_sink_alone():
    assert plain.capped(torch.tensor(1e9), 3.0) == 3.0 and plain.capped(torch.tensor(7.0), None) == 7.0
    assert float(plain.capped(torch.tensor(2.0), 4.0)) == pytest.approx(4 * math.tanh(0.5))
    s = torch.tensor([[0.0, 9.0], [math.log(3.0), math.log(2.0)]], dtype=torch.float64)
    p = plain.softmax_with_sink(s, plain.visible(2), torch.tensor(math.log(5.0), dtype=torch.float64))
    assert torch.allclose(p, torch.tensor([[1 / 6, 0.0], [0.3, 0.2]], dtype=torch.float64))


def test_plain_rotations_pair_neighbours_and_halves():
    x = torch.arange(12, dtype=torch.float64).view(2, 1, 6)
    near = plain.turn_neighbours(x, {"base": 100.0, "dims": 4})
    far = plain.turn_halves(x, {"base": 100.0, "dims": 4})
    assert torch.equal(near[0], x[0]) and torch.equal(far[1, 0, 4:], x[1, 0, 4:])
    for y, pairs in ((near, ((0, 1), (2, 3))), (far, ((0, 2), (1, 3)))):
        for (a, b), f in zip(pairs, (1.0, 100.0 ** -0.5)):
            u, v = x[1, 0, a], x[1, 0, b]
            assert y[1, 0, a] == pytest.approx(float(u * math.cos(f) - v * math.sin(f)))
            assert y[1, 0, b] == pytest.approx(float(v * math.cos(f) + u * math.sin(f)))


def test_plain_stretched_waves():
    """original 100, low 1, high 4: waves shorter than 25 stay, longer than 100 are stretched in
    full; at the two borders the blend meets both; between them s is linear in 1 / wave."""
    s = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 100.0}
    for wave, share in ((24.9, 1.0), (25.0, 1.0), (40.0, 0.5), (50.0, 1 / 3), (100.0, 0.0), (101.0, 0.0)):
        f = 2 * math.pi / wave
        assert plain.stretch_long_waves([f], s)[0] == pytest.approx(f * (share + (1 - share) / 8.0))
    assert plain.stretch_long_waves([0.3], None) == [0.3]


def test_plain_memory_fades_by_its_decay():
    """S_t^T q = sum over s of decay^(t - s) (k_s . q_t) v_s."""
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(6, 2, n, generator=g, dtype=torch.float64) for n in (3, 3, 4))
    got = plain.fading_memory(q, k, v, (0.5, 1.0))
    for t in range(6):
        for j, d in enumerate((0.5, 1.0)):
            want = sum(d ** (t - s) * (k[s, j] @ q[t, j]) * v[s, j] for s in range(t + 1))
            torch.testing.assert_close(got[t, j], want)
    alone = plain.fading_memory(q, k, v, (0.0, 0.0))
    torch.testing.assert_close(alone, (q * k).sum(-1, keepdim=True) * v)


def test_plain_router_weighs_the_chosen_logits_alone():
    w = plain.route(torch.tensor([0.0, math.log(3.0), -5.0, math.log(2.0), 0.0]), 3)
    assert w == {1: pytest.approx(0.5), 3: pytest.approx(1 / 3), 0: pytest.approx(1 / 6)}
    assert plain.route(torch.tensor([-900.0, -901.0]), 1) == {0: 1.0}


def test_plain_experts_bias_and_shared_unit():
    eye = torch.eye(2, dtype=torch.float64)
    w = {"m.router": torch.zeros(3, 2, dtype=torch.float64),
         "m.router.b": torch.tensor([0.0, -1.0, math.log(3.0)], dtype=torch.float64)}
    for e, c in (("e0.", 1.0), ("e1.", 100.0), ("e2.", 10.0), ("shared.", 1000.0)):
        w.update({f"m.{e}gate": eye, f"m.{e}up": eye, f"m.{e}down": c * eye})
    h = torch.tensor([[2.0, -1.0]], dtype=torch.float64)
    unit = torch.tensor([2.0 / (1 + math.exp(-2.0)) * 2.0, 1.0 / (1 + math.exp(1.0))])
    mlp = {"router": {"top": 2}, "shared": {}}
    got = plain.expert_ff(h, w, "m.", mlp)[0]
    assert got.tolist() == pytest.approx(((0.25 * 1 + 0.75 * 10 + 1000) * unit).tolist())
    got = plain.expert_ff(h, w, "m.", {"router": {"top": 2}})[0]
    assert got.tolist() == pytest.approx(((0.25 * 1 + 0.75 * 10) * unit).tolist())


def test_plain_gelu_unit_and_both_mixers():
    assert float(plain.gelu_tanh(torch.tensor(1.0, dtype=torch.float64))) == pytest.approx(0.8411919906)
    eye = torch.eye(2, dtype=torch.float64)
    w = {"m.gate": eye, "m.up": eye, "m.down": eye}
    got = plain.gelu_ff(torch.tensor([[1.0, -2.0]], dtype=torch.float64), w, "m.")
    assert got[0].tolist() == pytest.approx([0.8411919906, -2 * -0.0454023059])
    # a single token of one head each: attention gives its share beside the sink of v, retention
    # (k . q) v over its own size; each is then of size one, and half their sum comes out
    m = {"left": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0, "rot": {"base": 10.0, "dims": 2}},
         "right": {"heads": 1, "dim": 2, "vdim": 2, "decay": [0.5], "rot": {"base": 10.0, "dims": 2}}}
    w = {f"x.{side}.{n}": eye for side in ("left", "right") for n in "qkvog"}
    w.update({"x.left.sink": torch.zeros(1, dtype=torch.float64),
              "x.left.out": torch.tensor([1.0, 10.0], dtype=torch.float64),
              "x.right.out": torch.tensor([3.0, 5.0], dtype=torch.float64)})
    h = torch.tensor([[3.0, 3.0]], dtype=torch.float64)
    got = plain.both_mixers(h, w, "x.", m, 0.0)
    assert got[0].tolist() == pytest.approx([0.5 * (1 + 3), 0.5 * (10 + 5)])


# ------------------------------------------------------------------ rotations in the engine


def cpu_context(width=8):
    return BuildContext(ops=TorchOps(), dtype=torch.float32, device=torch.device("cpu"), width=width)


@pytest.mark.parametrize("dims, dim, head, scaling", [
    (6, 10, 16, None), (16, 16, 16, (3.0, 1.0, 4.0, 40)), (2, 6, 32, None), (20, 30, 48, (8.0, 2.0, 2.0, 9))])
def test_the_engines_layout_of_a_rotation_of_neighbours(dims, dim, head, scaling):
    """The whole-head table rotates what the layout brought together; queries times keys are
    those of the plain rotation, and a norm over the head may come before or after it."""
    s = dict(zip(("factor", "low", "high", "original"), scaling)) if scaling else None
    enc = build_part(POSITIONS, PartSpec("rope_partial", {
        "dims": dims, "base": 70.0, "head_dim": head, "max_position": 64, "pairs": "neighbours",
        "scaling": dict(s, kind="wavelength") if s else None}), cpu_context())
    layout = enc.layout(dim)
    assert len(layout) == head and sorted(x for x in layout if x >= 0) == list(range(dim))
    assert layout[:2] == ([0, 2] if dims > 2 else [0, dims]) and layout[head // 2] == 1
    x = torch.randn(50, 2, dim, generator=torch.Generator().manual_seed(1), dtype=torch.float64)
    want = plain.turn_neighbours(x, {"base": 70.0, "dims": dims, "scaling": s})

    def laid(v):
        out = torch.zeros(v.shape[0], v.shape[1], head, dtype=v.dtype)
        for place, src in enumerate(layout):
            if src >= 0:
                out[..., place] = v[..., src]
        return out
    y = laid(x).float().contiguous()
    enc.apply(y, None, torch.arange(50, dtype=torch.int32))
    torch.testing.assert_close(y, laid(want).float(), rtol=1e-4, atol=1e-4)
    torch.testing.assert_close(plain.over_rms(want, 1e-3),
                               plain.turn_neighbours(plain.over_rms(x, 1e-3), {"base": 70.0, "dims": dims, "scaling": s}))


def test_rotation_options_are_checked():
    base = {"dims": 4, "base": 70.0, "head_dim": 16, "max_position": 8}
    for more, message in (({"pairs": "thirds"}, "neighbours or halves"),
                          ({"scaling": {"kind": "linear"}}, "scaling"),
                          ({"scaling": {"kind": "wavelength", "factor": 2.0, "original": 9, "low": 2.0,
                                        "high": 1.0}}, "high >= low")):
        with pytest.raises(ValueError, match=message):
            build_part(POSITIONS, PartSpec("rope_partial", {**base, **more}), cpu_context())
    plain_halves = build_part(POSITIONS, PartSpec("rope_partial", base), cpu_context())
    assert plain_halves.layout(6) == [0, 1, 4, 5] + [-1] * 4 + [2, 3] + [-1] * 6
    no_table = build_part(POSITIONS, PartSpec("rope_interleaved", {"dims": 4, "base": 9.0}), cpu_context())
    with pytest.raises(RuntimeError, match="no table"):
        no_table.pair_table()


def test_the_recurrences_table_turns_pairs_of_halves_laid_side_by_side():
    enc = build_part(POSITIONS, PartSpec("rope_interleaved", {
        "dims": 6, "base": 50.0, "pairs": "halves", "max_position": 40}), cpu_context())
    table = enc.pair_table()
    assert table.shape == (40, 3, 2)
    x = torch.randn(40, 2, 9, generator=torch.Generator().manual_seed(1), dtype=torch.float64)
    want = plain.turn_halves(x, {"base": 50.0, "dims": 6})[..., enc.layout(9)].float()
    y = x[..., enc.layout(9)].float()
    cos, sin = table[:, None, :, 0], table[:, None, :, 1]
    a, b = y[..., 0:6:2], y[..., 1:6:2]
    got = torch.cat([torch.stack([a * cos - b * sin, b * cos + a * sin], -1).flatten(-2), y[..., 6:]], -1)
    torch.testing.assert_close(got, want, rtol=1e-4, atol=1e-4)


# ------------------------------------------------------------------ blocks of several kinds


def mixed_blocks_spec(order, width=16, vocab=30):
    """Layers of block kinds that hand the stream on in different ways, one after the other."""
    positions = {"rot": PartSpec("rope_interleaved", {"dims": 4, "base": 50.0, "pairs": "halves",
                                                      "max_position": 64})}
    layers = []
    for i, kind in enumerate(order):
        def norm(n, i=i):
            return PartSpec("rmsnorm", {"dim": width, "eps": 1e-5, "weight": f"l{i}.{n}"})
        pre = f"l{i}."
        mixer = PartSpec("retention", {"prefix": pre + "x.", "heads": 2, "dim": 4, "vdim": 6,
                                       "decay": (0.9, 0.5), "eps": 1e-5, "position": "rot",
                                       "state": "s"})
        ff = PartSpec("swiglu", {"prefix": pre + "f.", "inner_dim": 12, "act": "gelu_tanh",
                                 "names": ("gate", "up", "down")})
        side = PartSpec("gated_token_table", {"prefix": pre + "side.", "table": f"t{i}", "vocab_size": vocab,
                                              "dim": 3, "parts": 1, "index": 0})
        if kind == "pre":
            layers.append(LayerSpec("pre_norm", mixer_norm=norm("a"), mixer=mixer, ffn_norm=norm("b"),
                                    feed_forward=ff))
        elif kind == "parallel":
            layers.append(LayerSpec("parallel_residual", mixer_norm=norm("a"), mixer=mixer, feed_forward=ff))
        elif kind == "post":
            layers.append(LayerSpec("post_norm", mixer=mixer, mixer_post_norm=norm("a"), feed_forward=ff,
                                    ffn_post_norm=norm("b")))
        elif kind == "shift":
            layers.append(LayerSpec("sandwich_norm", mixer_norm=norm("a"), mixer=mixer, mixer_post_norm=norm("b"),
                                    mixer_filter=PartSpec("token_shift", {"weight": pre + "s", "dim": width})))
        else:
            parts = dict(mixer_norm=norm("a"), mixer=mixer, mixer_post_norm=norm("b"))
            if "f" in kind:
                parts.update(ffn_norm=norm("c"), feed_forward=ff, ffn_post_norm=norm("d"))
            if "s" in kind:
                parts.update(side=side, side_post_norm=norm("e"))
            layers.append(LayerSpec("sandwich_norm", **parts))
    return ModelSpec(
        architecture="Mixed", width=width, vocab_size=vocab,
        embedding=PartSpec("embedding", {"weight": "embed", "vocab_size": vocab}), positions=positions,
        layers=tuple(layers),
        order=tuple(Run(i, enter=("rows", 0) if i == 3 else None) for i in range(len(layers))),
        final_norm=PartSpec("rmsnorm", {"dim": width, "eps": 1e-5, "weight": "final"}),
        head=PartSpec("head", {"weight": "head", "vocab_size": vocab}), max_position=64,
        enter_tables={"rows": 1})


@pytest.mark.parametrize("order", [
    ("-fs", "-f", "-s", "-", "-fs"), ("pre", "-fs", "parallel", "-f", "post", "-s"),
    ("-", "parallel", "-fs", "pre", "-"), ("-f", "shift", "-s", "parallel", "parallel", "-fs"),
    ("post", "-fs", "post", "shift", "-f", "pre")], ids=lambda o: " ".join(o))
def test_sandwich_layers_between_blocks_of_other_kinds(order):
    """What a block tells the one before it (the norm it opens with) is an offer: with every
    offer withdrawn the model gives the same, and a row that enters in front of a layer is
    added first either way."""
    logits = []
    for withdrawn in (False, True):
        ctx = cpu_context(16)
        model = Model(mixed_blocks_spec(order), ctx)
        model.load_tensors({n: torch.randn(d.shape, generator=torch.Generator().manual_seed(len(n) + sum(map(ord, n))))
                            * (0.3 if d.role == "matrix" else 1.0) for n, d in model.tensor_decls().items()})
        offers = [b.entry_hint() for b in model.blocks]
        for kind, offer, block in zip(order, offers, model.blocks):
            if kind.startswith("-"):
                assert isinstance(offer, NormAhead)
            if withdrawn:
                block.entry_hint = lambda: None
        col = drives.drive_portions(runner_for(model, 4, 12), {"a": random_prompt(30, 30, 2)})
        logits.append(col.stacked("a")[0])
    torch.testing.assert_close(*logits, rtol=1e-5, atol=1e-5)


def test_blocks_and_parts_check_what_they_are_given():
    norm = PartSpec("rmsnorm", {"dim": 16, "eps": 1e-5, "weight": "n"})
    spec = mixed_blocks_spec(("-fs",))
    parts = dict(spec.layers[0].parts)
    del parts["side_post_norm"]
    bad = ModelSpec(**{**spec.__dict__, "layers": (LayerSpec("sandwich_norm", **parts),)})
    with pytest.raises(ValueError, match="side input and its norm"):
        Model(bad, cpu_context(16))
    with pytest.raises(ValueError, match="act="):
        ctx = cpu_context(16)
        from tokensprint_amd.parts.base import FEED_FORWARDS
        build_part(FEED_FORWARDS, PartSpec("swiglu", {"prefix": "f.", "inner_dim": 4, "act": "tanh"}), ctx)
    with pytest.raises(ValueError, match="decays"):
        ctx = cpu_context(16)
        build_part(MIXERS, PartSpec("lightning_attention", {
            "prefix": "x.", "heads": 3, "dim": 4, "vdim": 4, "decay": (0.5,), "eps": 1e-5}), ctx)
    assert norm.kind == "rmsnorm"


# ------------------------------------------------------------------ odd arrangements


@pytest.mark.parametrize("mlp, page, window", [
    (None, 1, 4), (sisepel_dense(8), 16, 1), (sisepel_moe(ff=4, experts=1, top=1, shared=None), 3, 50),
    (sisepel_moe(ff=6, experts=3, top=2, shared=5), 8, None)],
    ids=["no feed-forward", "dense", "one expert", "experts and a shared one"])
def test_models_of_one_kind_of_layer(tmp_path, mlp, page, window):
    layer = sisepel_layer(
        sisepel_attention(heads=2, kv_heads=1, dim=6, vdim=5, scale=1.2, window=window, softcap=4.0,
                          base=30.0, rot_dims=4),
        sisepel_retention(dim=5, vdim=7, decay=(0.9, 0.6), base=20.0, rot_dims=4), mlp)
    cfg = sisepel_config(width=16, vocab=40, eps=1e-6, side_dim=3, logit_scale=1.5, layers=[layer, layer])
    d = write_sisepel_model(tmp_path, cfg, 3, torch.float32)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, "float32", "cpu", ops=TorchOps())
    requests = {"a": random_prompt(37, 40, 1), "b": random_prompt(20, 40, 2), "c": random_prompt(1, 40, 3)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    drives.compare(drives.drive_portions(runner_for(model, page, -(-48 // page)), requests), ref, *TOL)
    drives.compare(drives.drive_mixed(runner_for(model, page, -(-100 // page)), requests), ref, *TOL)
