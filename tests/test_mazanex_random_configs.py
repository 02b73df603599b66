"""Mazanex configurations drawn at random (widths, head counts, key and value widths, the order of the
layers, chunks shorter and longer than the sequences and the 16-token pages, taps, how many channels
turn and with which base, decay exponents and caps, ranks, feed-forwards present or not): mixed
batches through the engine against the plain implementation, float32 tight and bfloat16 by the root
mean square."""
import copy
import random

import pytest
import torch

import helpers as H
import mazanex_cases as M
import plain_mazanex
from emu_ops import EmuOps

BACKENDS = ["emu", pytest.param("hip", marks=pytest.mark.gpu)]


def draw_config(seed):
    rng = random.Random(seed)
    width = rng.choice([32, 40, 48, 64, 96, 136])
    layers = []
    for _ in range(rng.randint(2, 5)):
        ff = rng.choice([None, rng.randint(20, 160)])
        kind = rng.choice(["parallel", "parallel", "gla", "mlstm"])
        heads, dim, vdim = rng.choice([1, 2, 3, 5]), rng.choice([6, 8, 16, 20, 24, 48, 64]), rng.choice([4, 8, 12, 24, 32, 56, 80])
        if kind == "gla":
            layers.append(M.gla(heads, dim, vdim, rng.choice([1.0, 2.0, 16.0, 40.0]), ff))
        elif kind == "mlstm":
            layers.append(M.mlstm(heads, dim, vdim, rng.choice([2.0, 8.0, 15.0]), ff))
        else:
            kv = rng.choice([1, 2, 3])
            dims = rng.choice([0, 2, dim // 4 * 2, dim // 2 * 2])
            layers.append(M.parallel(
                (kv * rng.choice([1, 2, 4]), kv, dim, vdim, rng.choice([0.1, 0.4, 1.0]), rng.choice([1, 2, 3, 4, 6]),
                 (dims, rng.choice([10.0, 1e4, 5e5])) if dims else None, rng.choice([None, 1, 3, 16, 17, 30, 64, 500])),
                (rng.choice([1, 2, 3, 4]), rng.choice([6, 8, 16, 20, 32])), ff))
    return dict(architecture="Mazanex", vocab=rng.choice([50, 131, 257]), width=width,
                norm=dict(eps=rng.choice([1e-6, 1e-5, 1e-3])), layers=layers)


def with_ranks(cfg, tensors, seed):
    """Decay projections of ranks of their own (no two layers' alike; the files decide, not the configuration)."""
    g = torch.Generator().manual_seed(seed)
    for name in list(tensors):
        if name.endswith((".w1", ".a1")):
            rank = int(torch.randint(1, 40, (1,), generator=g))
            up = name[:-1] + "2"
            down, other = tensors[name], tensors[up]
            tensors[name] = (torch.randn(rank, down.shape[1], generator=g) * 1.5 / down.shape[1] ** 0.5).to(torch.bfloat16)
            tensors[up] = (torch.randn(other.shape[0], rank, generator=g) * 1.5 / rank ** 0.5).to(torch.bfloat16)
    return tensors


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("seed", range(20))
def test_drawn_configuration(backend, seed):
    raw = draw_config(seed)
    cfg = H.lab.MazanexConfig.from_dict(raw)
    tensors = with_ranks(cfg, M.make_tensors(cfg, seed), seed)
    seqs = {f"r{i}": M.random_ids(cfg, n, 100 * seed + i) for i, n in enumerate([3, 45, 70, 20])}
    want = {rid: plain_mazanex.forward(cfg.to_dict(), tensors, ids) for rid, ids in seqs.items()}
    for dtype in ("f32", "bf16"):
        kw = dict(ops=EmuOps(), device="cpu") if backend == "emu" else {}
        engine = H.lab.Engine(config=cfg, tensors=tensors.items(), dtype=dtype, page_size=16, num_pages=16,
                              max_requests=3, max_batch_tokens=128, max_seq_len=128, **kw)
        got = H.run_trace(engine, seqs, H.steps_mixed(seqs, seed=seed, max_live=3, budget=64))
        diff = torch.cat([got[rid].double() - want[rid] for rid in got])
        assert not torch.isnan(diff).any()
        size = max(1.0, float(torch.cat(list(want.values())).std()))
        if dtype == "f32":
            bad = H.first_wrong(got, want, 4e-4 * size)
            assert bad is None, f"{raw}\nfirst wrong logits at (request, position, error) = {bad}"
        else:
            rms = float(diff.pow(2).mean().sqrt())
            assert rms < 0.08 * size, (raw, rms)
        engine.cache.check()
        assert engine.cache.metrics()["rows_used"] == 0


# Two configurations at the sizes of small real models: head sizes that the matrix-core attention
# kernels take (groups of 4 heads and of 3 share their keys) and one that is laid out for them, states
# of 64 x 128 and 128 x 64 (products of 64-row chunks), one too wide for those, chunks that cross the
# 64-token pages.
REAL = {
    "M": dict(architecture="Mazanex", vocab=1000, width=256, norm=dict(eps=1e-6), layers=[
        M.mlstm(3, 64, 128, 15.0, ff=520),
        M.parallel((8, 2, 64, 64, 0.125, 4, (64, 1e4), 100), (4, 64), ff=512),
        M.gla(2, 128, 64, 16.0, ff=512),
    ]),
    "N": dict(architecture="Mazanex", vocab=777, width=384, norm=dict(eps=1e-5), layers=[
        M.parallel((6, 2, 80, 128, 0.1, 3, (40, 5e5), 150), (3, 128), ff=576),
        M.mlstm(2, 48, 272, 8.0),
        M.gla(2, 144, 96, 4.0, ff=200),
        M.parallel((12, 12, 32, 48, 0.2, 2, (16, 1e3), 64), (6, 64)),
    ]),
}


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(REAL))
def test_sizes_of_small_real_models(name):
    cfg = H.lab.MazanexConfig.from_dict(REAL[name])
    tensors = M.make_tensors(cfg, 3)
    seqs = {f"r{i}": M.random_ids(cfg, n, 50 + i) for i, n in enumerate([260, 45, 130, 200])}
    want = {rid: plain_mazanex.forward(cfg.to_dict(), tensors, ids) for rid, ids in seqs.items()}
    size = max(1.0, float(torch.cat(list(want.values())).std()))
    for dtype in ("f32", "bf16"):
        for cut in (H.steps_prefill_then_decode, lambda s: H.steps_mixed(s, seed=1, max_live=3, budget=192)):
            engine = H.lab.Engine(config=cfg, tensors=tensors.items(), dtype=dtype, page_size=64, num_pages=20,
                                  max_requests=3, max_batch_tokens=384, max_seq_len=384)
            got = H.run_trace(engine, seqs, cut(seqs))
            diff = torch.cat([got[rid].double() - want[rid] for rid in got])
            assert not torch.isnan(diff).any()
            if dtype == "f32":
                bad = H.first_wrong(got, want, 5e-4 * size)
                assert bad is None, f"first wrong logits at (request, position, error) = {bad}"
            else:
                rms = float(diff.pow(2).mean().sqrt())
                assert rms < 0.08 * size, rms
            engine.cache.check()


def test_configuration_round_trip_and_errors():
    """``to_dict`` gives back what ``from_dict`` read; what cannot be a model of this design is refused
    with the place named."""
    from llm_inference_lab_amd.config import ConfigError
    for seed in range(8):
        raw = draw_config(seed)
        cfg = H.lab.MazanexConfig.from_dict(raw)
        assert H.lab.MazanexConfig.from_dict(cfg.to_dict()) == cfg
    good = copy.deepcopy(M.CONFIGS["P"])
    for breaker, needle in [
        (lambda r: r["layers"].append(dict(type="other", mixer={}, mlp=None)), "unknown layer type"),
        (lambda r: r.pop("norm"), "norm"),
        (lambda r: r["layers"][0]["mixer"]["left"].update(heads=0), "positive"),
        (lambda r: r["layers"][0]["mixer"]["left"].update(heads=5), "multiple"),
        (lambda r: r["layers"][0]["mixer"]["left"].update(mask=dict(size=0)), "mask.size"),
        (lambda r: r["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
        (lambda r: r["layers"][0]["mixer"].pop("right"), "right"),
        (lambda r: r["layers"][1]["mixer"].update(gate_cap=0.0), "gate_cap"),
        (lambda r: r["layers"][2]["mixer"].update(tau=-1.0), "tau"),
        (lambda r: r["layers"][1]["mixer"].pop("vdim"), "vdim"),
        (lambda r: r["layers"][1]["mlp"].update(kind="moe"), "dense"),
    ]:
        bad = copy.deepcopy(good)
        breaker(bad)
        with pytest.raises(ConfigError) as err:
            H.lab.MazanexConfig.from_dict(bad)
        assert needle in str(err.value)


def test_factors_of_a_decay_that_do_not_fit_are_refused():
    cfg = M.config_of("P")
    for name in ("l0.mix.right.w1", "l2.mix.a1"):
        tensors = M.make_tensors(cfg, 1)
        tensors[name] = tensors[name][:-1].contiguous()
        with pytest.raises(ValueError, match="do not fit"):
            H.lab.Engine(config=cfg, tensors=tensors.items(), dtype="f32", ops=EmuOps(), device="cpu", max_seq_len=64,
                         num_pages=4)


def test_a_model_folder_written_and_read(tmp_path):
    """The random-weights mode writes a folder that the registry, the loader and the engine take back."""
    cfg = M.config_of("S")
    path = H.lab.write_random_model(str(tmp_path / "model"), cfg, 3)
    engine = H.lab.Engine(path, dtype="f32", ops=EmuOps(), device="cpu", page_size=16, num_pages=8, max_requests=1,
                          max_seq_len=64)
    assert engine.config == cfg and engine.spec.architecture == "Mazanex"
    from llm_inference_lab_amd.weights.safetensors_io import ModelFiles
    files = ModelFiles(path)
    tensors = {n: files.tensor(n).clone() for n in files.names()}
    files.close()
    ids = M.random_ids(cfg, 20, 1)
    out = engine.step([H.lab.StepEntry(engine.open("a"), ids, list(range(20)))])
    want = plain_mazanex.forward(cfg.to_dict(), tensors, ids)
    assert float((out.double() - want).abs().max()) < 1e-4
