"""Sisepel configurations drawn at random on the GPU: sizes that are no multiples of the kernels'
tiles, windows from one token to beyond the request, rotations with and without stretched
waves, caps, decays, experts, with and without feed-forwards and side input, every run compared
with the plain implementation in float32 however the work is cut, and with itself in bfloat16."""

import random

import pytest
import torch

import drives
from helpers import (random_prompt, sisepel_attention, sisepel_config, sisepel_dense,
                     sisepel_layer, sisepel_moe, sisepel_retention, sisepel_scaling,
                     write_sisepel_model)
from plain import sisepel_plain as plain
from test_fubepel_gpu import assert_rows_within_rounding, rms_errors
from test_sisepel_gpu import rounding_errors
from tokensprint_amd.engine import ModelRunner
from tokensprint_amd.engine.assemble import load_model

pytestmark = pytest.mark.gpu


def draw(case):
    rnd = random.Random(5000 + case)
    layers = []
    for _ in range(rnd.choice([1, 2, 3, 4])):
        kind = rnd.choice(["none", "dense", "moe", "moe"])
        mlp = None
        if kind == "dense":
            mlp = sisepel_dense(rnd.choice([8, 12, 40, 100]))
        elif kind == "moe":
            experts = rnd.choice([1, 3, 8, 13])
            mlp = sisepel_moe(ff=rnd.choice([4, 8, 20, 33]), experts=experts,
                              top=rnd.randint(1, min(experts, 4)), shared=rnd.choice([None, 8, 10, 40]))
        kv = rnd.choice([1, 2, 3])
        dim, rdim = rnd.choice([6, 16, 40, 64, 96, 128]), rnd.choice([4, 12, 32, 64, 100, 132])
        low = rnd.choice([0.5, 1.0, 2.0])
        scaling = rnd.choice([None, sisepel_scaling(rnd.choice([2.0, 8.0]), low, low * rnd.choice([1.0, 2.0, 4.0]),
                                                    rnd.choice([16, 100, 4096]))])
        layers.append(sisepel_layer(
            sisepel_attention(heads=kv * rnd.choice([1, 2, 4]), kv_heads=kv, dim=dim,
                              vdim=rnd.choice([4, 16, 48, 100, 128]), scale=rnd.choice([0.05, 0.2, 0.5]),
                              window=rnd.choice([1, 2, 7, 16, 31, 64, 100, 1000, None]),
                              softcap=rnd.choice([None, 0.7, 3.0, 30.0]), base=rnd.choice([100.0, 1e4, 1e6]),
                              rot_dims=rnd.choice([2, dim // 2 // 2 * 2 or 2, dim]), scaling=scaling),
            sisepel_retention(dim=rdim, vdim=rnd.choice([5, 16, 64, 96]),
                              decay=[rnd.choice([0.0, 0.5, 0.9, 0.96875, 0.99, 0.9995, 1.0])
                                     for _ in range(rnd.choice([1, 2, 5]))],
                              base=rnd.choice([100.0, 1e4]), rot_dims=rnd.choice([2, rdim])), mlp))
    cfg = sisepel_config(width=rnd.choice([20, 36, 64, 100]), vocab=rnd.choice([50, 97, 300]),
                         eps=rnd.choice([1e-6, 1e-5]), side_dim=rnd.choice([None, 1, 6, 16, 40]),
                         logit_scale=rnd.choice([1.0, 0.3, 4.0]), layers=layers)
    return cfg, rnd.choice([4, 16, 32])


LENGTHS = [5, 17, 40, 1, 70, 131]


@pytest.mark.parametrize("case", range(14))
def test_a_drawn_configuration(case, tmp_path, gpu_device):
    """A drawn model may be sensitive by itself (its norms divide by whatever a sub-layer gives):
    the error is held against what float32 arithmetic costs the plain implementation."""
    cfg, page = draw(case)
    d = write_sisepel_model(tmp_path, cfg, case, torch.float32, std=0.15)
    pcfg, w = plain.read_model_dir(d)
    w32 = {n: t.float() if t.is_floating_point() else t for n, t in w.items()}
    _, model = load_model(d, torch.float32, gpu_device)
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i) for i, n in enumerate(LENGTHS)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = max(float(rms_errors(plain.forward(pcfg, w32, t), ref[rid]).max()) for rid, t in requests.items())

    def check(col):
        for rid in requests:
            got, positions = col.stacked(rid)
            assert positions == list(range(len(requests[rid])))
            worst = rms_errors(got, ref[rid])
            assert float(worst.max()) < 3e-5 + 12 * own, \
                f"request {rid}, position {int(worst.argmax())}: {float(worst.max()):.2e}, plain float32 {own:.2e}"

    def runner(pages):
        return ModelRunner(model, page_size=page, num_pages=pages, num_slots=4)

    roomy = 160 // page + 4
    check(drives.drive_whole(runner(roomy), requests))
    check(drives.drive_prefill_then_decode(runner(roomy), requests))
    check(drives.drive_portions(runner(roomy), requests))
    check(drives.drive_mixed(runner(448 // page), requests))


@pytest.mark.parametrize("case", range(14))
def test_a_drawn_configuration_runs_in_bfloat16(case, tmp_path, gpu_device):
    """The same draws in bfloat16: whole prompts and mixed steps agree with each other (what
    differs between them is which kernel serves a row) and with the plain logits, both within
    what rounding every matrix to bfloat16 once more costs the plain implementation."""
    cfg, page = draw(case)
    d = write_sisepel_model(tmp_path, cfg, case, torch.bfloat16, std=0.15)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, torch.bfloat16, gpu_device)
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i) for i, n in enumerate(LENGTHS)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = rounding_errors(pcfg, w, requests, ref, case)

    def runner(pages):
        return ModelRunner(model, page_size=page, num_pages=pages, num_slots=4)

    for col in (drives.drive_whole(runner(160 // page + 4), requests),
                drives.drive_mixed(runner(448 // page), requests)):
        assert_rows_within_rounding(col, ref, own)
