"""Molotar through the command lines as a user runs them: ``bin/generate`` on a configuration
file with random weights, and ``bin/trace_run`` replaying steps over a model folder written by
the random-weights mode, against the plain implementation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers as H
import molotar_cases as M
import plain_molotar
from llm_inference_lab_amd.weights import random_tensors
from llm_inference_lab_amd.weights.safetensors_io import ModelFiles

pytestmark = pytest.mark.gpu
SEED = 4


def test_generate_greedy_tokens(tmp_path):
    cfg = M.config_of("T")
    path = str(tmp_path / "config.json")
    with open(path, "w") as f:
        json.dump(cfg.to_dict(), f)
    tensors = dict(random_tensors(M.expected_tensors(cfg), SEED, torch.bfloat16))
    prompts = [M.random_ids(cfg, n, 20 + n) for n in (6, 33)]
    proc = subprocess.run([sys.executable, os.path.join(H.ROOT, "bin", "generate"), "--random-weights", path, "--seed",
                           str(SEED), "--dtype", "f32", "--prompt-ids",
                           ";".join(",".join(map(str, p)) for p in prompts), "--max-new-tokens", "6", "--page-size", "16",
                           "--max-batch-tokens", "16"], capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-3000:]
    out = json.loads([l for l in proc.stdout.splitlines() if l.startswith("{")][-1])
    assert out["kv_released"] is True
    for prompt, got in zip(prompts, out["output_ids"]):
        ids = list(prompt)
        for n, token in enumerate(got):
            logits = plain_molotar.forward(ids, cfg.to_dict(), tensors)[-1]
            best = int(logits.argmax())
            # (plain random weights give flat logits: a near-tie may fall either way)
            assert token == best or float(logits[best] - logits[token]) < 1e-5, (n, token, best)
            ids.append(token)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["T", "V"])
def test_trace_replay(tmp_path, dtype, name):
    """Three requests in steps of portions and single tokens, one left out of a step, slots and
    pages used again by a fourth; logits at the wanted places."""
    cfg = M.config_of(name)
    model_dir = H.lab.write_random_model(str(tmp_path / "model"), cfg, SEED)
    files = ModelFiles(model_dir)
    tensors = {n: files.tensor(n).clone() for n in files.names()}
    files.close()
    seqs = {rid: M.random_ids(cfg, n, 7 + i) for i, (rid, n) in enumerate([("a", 40), ("b", 9), ("c", 70), ("d", 21)])}
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": seqs["a"][:17], "want": [0, 16]},
                                {"id": "b", "tokens": seqs["b"][:2], "want": []}], "end": []},
        {"step": 1, "entries": [{"id": "c", "tokens": seqs["c"][:64], "want": [63]},
                                {"id": "b", "tokens": seqs["b"][2:3], "want": [0]}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": seqs["a"][17:40], "want": [22]},
                                {"id": "b", "tokens": seqs["b"][3:9], "want": [5]},
                                {"id": "c", "tokens": seqs["c"][64:66], "want": [1]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "c", "tokens": seqs["c"][66:67], "want": []}], "end": []},
        {"step": 4, "entries": [{"id": "d", "tokens": seqs["d"], "want": [20]},
                                {"id": "c", "tokens": seqs["c"][67:70], "want": [0, 2]}], "end": ["c", "d"]},
    ]
    out_dir = str(tmp_path / "out")
    proc = subprocess.run([sys.executable, os.path.join(H.ROOT, "bin", "trace_run"), "--model", model_dir, "--dtype", dtype,
                           "--out", out_dir, "--max-tokens", "256", "--max-requests", "3"],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    plain = {rid: plain_molotar.forward(ids, cfg.to_dict(), tensors) for rid, ids in seqs.items()}
    at = {rid: 0 for rid in seqs}
    worst = 0.0
    for s in steps:
        want = []
        for e in s["entries"]:
            want += [plain[e["id"]][at[e["id"]] + w] for w in e["want"]]
            at[e["id"]] += len(e["tokens"])
        path = os.path.join(out_dir, f"{s['step']}.f32")
        if not want:
            assert not os.path.exists(path)
            continue
        got = np.fromfile(path, dtype="<f4").reshape(len(want), cfg.vocab)
        worst = max(worst, float(np.abs(got - torch.stack(want).numpy()).max()))
    # Plain random weights: logits with a standard deviation well below one.
    assert worst < (2e-5 if dtype == "float32" else 6e-2), worst
