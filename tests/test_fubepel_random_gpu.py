"""Fubepel configurations drawn at random on the GPU: layer orders, sizes that are no multiples
of the kernels' tiles, windows from one token to beyond the request beside kept first tokens,
latents read by later layers, with and without feed-forwards and side input, every run
compared with the plain implementation in float32 however the work is cut, and with itself in
bfloat16."""

import random

import pytest
import torch

import drives
from helpers import (fubepel_attention, fubepel_config, fubepel_delta, fubepel_dense,
                     fubepel_latent, random_prompt, write_fubepel_model)
from plain import fubepel_plain as plain
from test_fubepel_gpu import assert_rows_within_rounding, rms_errors, rounding_errors
from tokensprint_amd.engine import ModelRunner
from tokensprint_amd.engine.assemble import load_model

pytestmark = pytest.mark.gpu


def draw(case):
    rnd = random.Random(4000 + case)
    layers, owners = [], []
    for i in range(rnd.choice([1, 2, 3, 4, 5])):
        mlp = None if rnd.random() < 0.25 else \
            fubepel_dense(rnd.choice([8, 12, 40, 100]), rnd.choice([0.2, 1.0, 7.0]))
        kind = rnd.choice(["delta", "attention", "latent", "latent"])
        kv = rnd.choice([1, 2, 3])
        heads = kv * rnd.choice([1, 2, 4])
        if kind == "delta":
            layers.append(fubepel_delta(heads=heads, kv_heads=kv, dim=rnd.choice([4, 12, 32, 64, 100]),
                                        vdim=rnd.choice([5, 16, 64, 96]), conv=rnd.choice([1, 2, 4, 6]), mlp=mlp))
        elif kind == "attention":
            layers.append(fubepel_attention(
                heads=heads, kv_heads=kv, dim=rnd.choice([6, 16, 40, 64, 96, 128]),
                vdim=rnd.choice([4, 16, 48, 100, 128]), scale=rnd.choice([0.05, 0.2]),
                window=rnd.choice([1, 2, 7, 16, 31, 64, 100, 1000, None]),
                keep_first=rnd.choice([0, 1, 4, 17, 40, 300]), mlp=mlp))
        else:
            sizes = dict(rot_dim=rnd.choice([2, 8, 16, 64]), kv_rank=rnd.choice([12, 24, 64, 160]),
                         base=rnd.choice([100.0, 1e4, 1e6]))
            source = rnd.choice(owners + [None]) if owners else None
            if source is not None:
                m = layers[source]["mixer"]
                sizes = dict(rot_dim=m["rot_dim"], kv_rank=m["kv_rank"], base=m["rot"]["base"])
            else:
                owners.append(i)
            layers.append(fubepel_latent(heads=rnd.choice([1, 3, 4, 8, 17]), dim=rnd.choice([2, 8, 24, 64]),
                                         vdim=rnd.choice([3, 16, 40]), scale=rnd.choice([0.02, 0.05]),
                                         kv_from=source, mlp=mlp, **sizes))
    cfg = fubepel_config(width=rnd.choice([20, 36, 64, 100]), vocab=rnd.choice([50, 97, 300]),
                         eps=rnd.choice([1e-6, 1e-5]), embed_scale=rnd.choice([1.0, 8.0, 2.7]),
                         side_dim=rnd.choice([None, 1, 6, 16, 40]), layers=layers)
    return cfg, rnd.choice([4, 16, 32])


@pytest.mark.parametrize("case", range(14))
def test_a_drawn_configuration(case, tmp_path, gpu_device):
    """A drawn model may be sensitive by itself (its norms divide by whatever a sub-layer gives):
    the error is held against what float32 arithmetic costs the plain implementation."""
    cfg, page = draw(case)
    d = write_fubepel_model(tmp_path, cfg, case, torch.float32, std=0.15, sharpen=1.0)
    pcfg, w = plain.read_model_dir(d)
    w32 = {n: t.float() if t.is_floating_point() else t for n, t in w.items()}
    _, model = load_model(d, torch.float32, gpu_device)
    lengths = [5, 17, 40, 1, 70, 131]
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i) for i, n in enumerate(lengths)}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = max(float(rms_errors(plain.forward(pcfg, w32, t), ref[rid]).max()) for rid, t in requests.items())

    def check(col):
        for rid in requests:
            got, positions = col.stacked(rid)
            assert positions == list(range(len(requests[rid])))
            worst = rms_errors(got, ref[rid])
            assert float(worst.max()) < 2e-5 + 12 * own, \
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
    d = write_fubepel_model(tmp_path, cfg, case, torch.bfloat16, std=0.15, sharpen=1.0)
    pcfg, w = plain.read_model_dir(d)
    _, model = load_model(d, torch.bfloat16, gpu_device)
    requests = {f"r{i}": random_prompt(n, cfg["vocab"], 100 + i)
                for i, n in enumerate([5, 17, 40, 1, 70, 131])}
    ref = {rid: plain.forward(pcfg, w, t).float() for rid, t in requests.items()}
    own = rounding_errors(pcfg, w, requests, ref, case)

    def runner(pages):
        return ModelRunner(model, page_size=page, num_pages=pages, num_slots=4)

    for col in (drives.drive_whole(runner(160 // page + 4), requests),
                drives.drive_mixed(runner(448 // page), requests)):
        assert_rows_within_rounding(col, ref, own)
