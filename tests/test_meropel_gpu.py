"""The Meropel design in the framework against the plain implementation of ``plain_meropel``: every mechanism alone at
sizes of its own, then whole models through the step function, the cache and state manager, the scheduler and the
engine, for the same requests cut into steps in different ways.  Configurations and weights are made here."""

from __future__ import annotations

import json
import random

import pytest
import torch

import plain_meropel as pm
import traces
from harness import PartCtx, close, off, paged, replay, step_context
from tiny import random_tokens

pytestmark = pytest.mark.gpu
DEV = "cuda"
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def attn(H, G, D, E, scale, dims, base=5000.0):
    return dict(heads=H, kv_heads=G, dim=D, vdim=E, scale=scale, rot={"base": base, "dims": dims})


def parallel(left, inner, state, rank, conv, ls=1.0, rs=1.0):
    return "parallel", {"left": left, "right": dict(inner=inner, state=state, dt_rank=rank, conv=conv), "left_scale": ls, "right_scale": rs}


def parallel_2(left, H, E, N, groups, conv, parts):
    return "parallel_2", {"left": left, "right": dict(heads=H, vdim=E, state=N, groups=groups, conv=conv, norm_groups=parts)}


def gla(H, D, E, tau):
    return "gla", dict(heads=H, dim=D, vdim=E, tau=tau)


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(n, top, ff, identity=0, groups=(1, 1), scale=1.0, shared=0):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top, "scale": scale, "identity": identity,
                                                           "groups": {"count": groups[0], "keep": groups[1]}}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


BIGRAM = {"bigram": {"buckets": 97, "mul_prev": 31, "mul_cur": 7}}
# A: sizes that are no multiples of 8 or 16 (a width that is no multiple of four), values wider and narrower than keys and as wide, a
#    layer without feed-forward, no shared expert, convolutions of one to five taps.
# B: one head, one group, one state, one expert beside one identity expert, no second embedding, no logit scale, one rotated pair.
# C: sizes the matrix-core kernels take in bfloat16 and long portions that run in chunks.
CONFIGS = {
    "A": dict(cfg={"architecture": "Meropel", "vocab": 300, "width": 90, "norm": {"eps": 1e-5}, "logit_scale": 0.5, "embedding": BIGRAM,
                   "layers": [layer(parallel(attn(6, 3, 12, 20, 0.3, 6), 50, 5, 3, 4, 0.8, 1.4), moe(6, 3, 20, 2, (4, 2), 1.7, shared=28)),
                              layer(gla(3, 10, 22, 4.0), dense(50)),
                              layer(parallel_2(attn(4, 2, 14, 10, 0.3, 8, 300.0), 6, 9, 7, 3, 2, 2), None),
                              layer(parallel(attn(2, 1, 10, 10, 0.3, 10), 37, 20, 5, 1, 1.1, 0.6), moe(5, 2, 24, 1, (3, 2)))]},
              seed=3, page=8, lengths=(1, 2, 23, 77, 150, 203)),
    "B": dict(cfg={"architecture": "Meropel", "vocab": 128, "width": 64, "norm": {"eps": 1e-6},
                   "layers": [layer(parallel(attn(1, 1, 16, 24, 0.4, 2, 100.0), 40, 1, 1, 5), moe(1, 1, 48, 1, (2, 1), 0.7)),
                              layer(gla(1, 64, 8, 1.0), moe(1, 1, 24, shared=16)),
                              layer(parallel_2(attn(1, 1, 16, 16, 0.4, 16), 1, 40, 1, 1, 3, 1), dense(40))]},
              seed=4, page=16, lengths=(3, 8, 9, 40, 129)),
    "C": dict(cfg={"architecture": "Meropel", "vocab": 200, "width": 128, "norm": {"eps": 1e-5}, "logit_scale": 2.0, "embedding": BIGRAM,
                   "layers": [layer(parallel_2(attn(8, 2, 32, 32, 0.2, 16, 1e6), 8, 32, 64, 2, 4, 4), moe(14, 3, 32, 2, (4, 2), 1.3, shared=64)),
                              layer(gla(4, 32, 48, 16.0), moe(4, 4, 64, 0, (1, 1), 1.0, shared=96)),
                              layer(parallel(attn(4, 2, 48, 32, 0.15, 32, 1e4), 128, 16, 8, 4, 1.2, 0.8), dense(256)),
                              layer(gla(2, 64, 32, 2.0), moe(16, 3, 32, 4, (5, 2), 2.0))]},
              seed=5, page=16, lengths=(5, 31, 64, 100, 260)),
}
# what random weights of the usual law leave so small that soft-maxes are flat, gates constant and SiLUs linear (the first
# tail of a name that fits)
SHARPEN = {"embed": 25.0, "bigram": 15.0, "left.q": 6.0, "left.k": 6.0, "left.v": 6.0, "left.g": 10.0, ".b": 15.0, "right.in": 8.0, "right.x": 6.0,
           "right.dt": 15.0, "mix.q": 6.0, "mix.k": 6.0, "mix.v": 6.0, "mix.g": 8.0, "a1": 8.0, "a2": 20.0, ".o": 3.0, "router": 10.0, "correction": 4.0,
           ".gate": 6.0, ".up": 6.0, ".down": 3.0}
# bfloat16 bounds (a row, the median row): every sublayer's output is rounded and then normed, the weights here are sharp, and most
# layers ask a router; the 32-bit runs are the sharp test
CAPS = (0.2, 0.12)
KEEP = ("dt.b", "a2.b")  # their laws are theirs


def config_of(cfg):
    """The typed configuration with an inner size for the decay's two matrices, which config.json does not hold."""
    from dataclasses import replace

    from nanospec_amd.config import MeropelConfig

    config = MeropelConfig.from_hf(cfg)
    return replace(config, layers=tuple(l if l.gla is None else replace(l, gla=replace(l.gla, decay_rank=5 + 3 * (i % 2))) for i, l in enumerate(config.layers)))


def sharpened(name):
    return 1.0 if name.endswith(KEEP) else next((by for tail, by in SHARPEN.items() if name.endswith(tail)), 1.0)


def write_folder(folder, cfg: dict, seed: int, change=None):
    """config.json and model.safetensors with random 32-bit weights for the tensors the framework says the model reads."""
    from safetensors.torch import save_file

    from nanospec_amd.parts.model import wanted_tensors
    from nanospec_amd.weights import random_tensors

    folder.mkdir(parents=True, exist_ok=True)
    tensors = random_tensors(wanted_tensors(config_of(cfg).model_spec()), seed, torch.float32)
    for name, t in tensors.items():
        t *= sharpened(name)
    if change is not None:
        change(tensors)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(folder / "model.safetensors"))
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("meropel")
    return {name: write_folder(base / name, c["cfg"], c["seed"]) for name, c in CONFIGS.items()}


def read_folder(folder, dtype):
    from safetensors.torch import load_file

    cfg = json.loads((folder / "config.json").read_text())
    w = {k: v.to(dtype).double() if v.dim() == 2 and not k.endswith(("conv", "A_log", "router")) else v.double()
         for k, v in load_file(str(folder / "model.safetensors")).items()}  # matrices as the engine rounds them
    for k in w:  # ... and what it keeps in the model's precision besides
        if k.endswith(("norm1", "norm1b", "norm2", "norm2b", "final.norm", ".out", "q.norm", "k.norm", "q.b", "k.b", "v.b")):
            w[k] = w[k].to(dtype).double()
    return cfg, w


def sequences(name):
    c = CONFIGS[name]
    return {f"r{i}": random_tokens(n, c["cfg"]["vocab"], 31 * i + n) for i, n in enumerate(c["lengths"])}


_REF, _MODELS = {}, {}


def plain_logits(folder, name, dtype):
    if (name, dtype) not in _REF:
        cfg, w = read_folder(folder, dtype)
        _REF[name, dtype] = {rid: pm.forward(cfg, w, toks).float() for rid, toks in sequences(name).items()}
    return _REF[name, dtype]


def engine_model(folder, name, dtype):
    from nanospec_amd.loader import load_model

    if (name, dtype) not in _MODELS:
        _MODELS[name, dtype] = load_model(folder, dtype=dtype)
    return _MODELS[name, dtype]


# ------------------------------------------------------------------------------------------------ whole models


@BOTH
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "mixed", "mixed7"])
def test_schedules_match_plain(folders, name, dtype, schedule):
    """Whole prompts; prefill then token-by-token decoding (120 tokens, through captured steps); portions down to two
    tokens; mixed batches of unequal requests in a pool so small that pages and state slots are used again."""
    page = CONFIGS[name]["page"]
    seqs, ref, model = sequences(name), plain_logits(folders[name], name, dtype), engine_model(folders[name], name, dtype)
    longest = max(len(t) for t in seqs.values())
    if schedule == "whole":
        steps, where = traces.whole(seqs)
    elif schedule == "tail":
        steps, where = traces.tail_decoded(seqs, tail=120)
    elif schedule == "portions":
        steps, where = traces.portions(seqs, seed=1)
    else:
        steps, where, peak = traces.mixed(seqs, seed=7 if schedule == "mixed7" else 0, max_live=2 if schedule == "mixed7" else 3)
    max_tokens = peak if schedule.startswith("mixed") else -(-longest // 64) * 64
    rep = replay(model, steps, where, ref, dtype, max_tokens, page, caps=CAPS)
    if schedule.startswith("mixed"):
        assert rep.pages_again > 0 and rep.slots_again > 0, "the pool was meant to hand pages and slots out again"
    if schedule == "tail":
        assert rep.graph_steps > 0, "single decoded tokens were meant to replay captured steps"


@BOTH
@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_stream_after_every_layer(folders, name, dtype):
    """The residual stream after each layer, not only the logits: a fault shows in the layer that has it."""
    from nanospec_amd.engine.replay import Replayer

    model = engine_model(folders[name], name, dtype)
    cfg, w = read_folder(folders[name], dtype)
    toks = sequences(name)["r3"]
    ref, got = [], []
    pm.forward(cfg, w, toks, probe=lambda run, x: ref.append(x.clone()))
    model.layer_probe = lambda i, total: got.append(total.clone())
    try:
        Replayer(model, 256, page_size=CONFIGS[name]["page"], use_graphs=False).step([{"id": "a", "tokens": toks, "want": [0]}], ["a"])
    finally:
        model.layer_probe = None
    assert len(got) == len(cfg["layers"]) == len(ref)
    for i, g in enumerate(got):
        err = (g.cpu() - ref[i].float()).abs().amax(-1) / ref[i].abs().max()
        if dtype == torch.float32:
            assert err.max() <= 2e-5, f"after layer {i}: {err.max():.2e}"
        else:  # (a token may take another expert where two router scores lie within rounding of each other)
            assert (err > 0.1).sum() <= max(2, len(toks) // 10) and err.median() <= 0.03, f"after layer {i}: {err}"


@BOTH
@pytest.mark.parametrize("name", list(CONFIGS))
def test_one_position_however_it_is_reached(folders, name, dtype):
    """The logits at one position are the same (beyond rounding) whole, decoded, in portions cut at and around the pages'
    edges and the recurrences' blocks of tokens, and beside other requests."""
    from nanospec_amd.engine.replay import Replayer

    model, seqs = engine_model(folders[name], name, dtype), sequences(name)
    toks = seqs["r4"]
    last = len(toks) - 1
    rep = Replayer(model, 1024, page_size=CONFIGS[name]["page"])
    got = [rep.step([{"id": "w", "tokens": toks, "want": [last]}], ["w"])[0]]
    rep.step([{"id": "d", "tokens": toks[:-1], "want": []}], [])
    got.append(rep.step([{"id": "d", "tokens": toks[-1:], "want": [0]}], ["d"])[0])
    cuts = [0, 2, 4, 5, 7, 8, 9, 10, 15, 16, 17, 23, 24, 26, 63, 64, 65, 113, last - 9, last - 8, last - 5, last - 4, last - 1, len(toks)]
    cuts = sorted({c for c in cuts if 0 <= c <= len(toks)})
    other = seqs["r3"]
    for a, b in zip(cuts, cuts[1:]):
        entries = [{"id": "p", "tokens": toks[a:b], "want": [b - a - 1]}]
        if a < len(other):
            entries.insert(0, {"id": "o", "tokens": other[a : min(b, len(other))], "want": []})
        out = rep.step(entries, ["p"] if b == len(toks) else [])
    got.append(out[-1])
    tol = 2e-5 if dtype == torch.float32 else 0.08
    for g in got[1:]:
        assert (g - got[0]).abs().max() <= tol * got[0].abs().max()


@BOTH
def test_long_portions_beside_decoded_tokens_through_captured_steps(folders, dtype):
    """A portion long enough for the recurrences' chunks beside single tokens of another request, in one captured shape that is
    replayed with other requests and other lengths (long portions, a short one that the scan takes, none)."""
    from nanospec_amd.engine.replay import Replayer

    model, seqs, ref = engine_model(folders["C"], "C", dtype), sequences("C"), plain_logits(folders["C"], "C", dtype)
    long, short = seqs["r4"], seqs["r3"]
    rep = Replayer(model, 512, page_size=CONFIGS["C"]["page"])
    rep.step([{"id": "d", "tokens": short[:40], "want": []}], [])
    at, loose, rows = 40, [], 0
    for trial, cuts in enumerate(([0, 200, 205, 260], [0, 250, 258], [0, 60, 259], [0, 195, 198])):
        for a, b in zip(cuts, cuts[1:]):
            end = b == cuts[-1]
            out = rep.step([{"id": "d", "tokens": [short[at]], "want": [0]}, {"id": f"p{trial}", "tokens": long[a:b], "want": [0, b - a - 1]}],
                           [f"p{trial}"] if end else [])
            assert rep.runner.last_used_graph, "the step was meant to replay a captured graph"
            close(out, torch.stack([ref["r3"][at], ref["r4"][a], ref["r4"][b - 1]]), dtype, (a, b == len(long)), loose)  # (a row that is off is off in every trial)
            at, rows = at + 1, rows + 3
    assert len(set(loose)) <= max(2, rows // 10), loose


def test_long_decoding_keeps_the_state(folders):
    """400 tokens one by one after a short prompt, in 32-bit: every kind of state and the pages carry every token; the last
    logits are those of the whole sequence at once."""
    cfg, w = read_folder(folders["B"], torch.float32)
    toks = random_tokens(420, cfg["vocab"], 99)
    ref = {"a": pm.forward(cfg, w, toks).float()}
    steps, where = traces.tail_decoded({"a": toks}, tail=400)
    replay(engine_model(folders["B"], "B", torch.float32), steps, where, ref, torch.float32, 448, CONFIGS["B"]["page"])


@BOTH
@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_engine(folders, name, dtype):
    """``Engine.generate`` with a token budget and a longest portion, so that the scheduler cuts prompts and batches portions
    beside decoding requests; against the plain implementation's greedy continuation (in bfloat16 a sequence may leave it
    only where the plain logits of the two tokens are within rounding of each other)."""
    from nanospec_amd import Engine, EngineConfig, SamplingParams

    page = CONFIGS[name]["page"]
    model = engine_model(folders[name], name, dtype)
    cfg, w = read_folder(folders[name], dtype)
    prompts = [t for t in sequences(name).values() if len(t) < 100][:4]
    new = 12
    eng = Engine(model, EngineConfig(num_blocks=sum(-(-(len(p) + new) // page) for p in prompts) + 2, block_size=page, max_step_tokens=48,
                                     prefill_chunk=20, max_running=4))
    got = eng.generate(prompts, SamplingParams(max_tokens=new))
    eng.cache.check()
    for prompt, ours in zip(prompts, got):
        seq = list(prompt)
        for k, tok in enumerate(ours):
            row = pm.forward(cfg, w, seq)[-1]
            best = int(row.argmax())
            if tok != best:
                gap = float(row[best] - row[tok]) / float((row - row.mean()).pow(2).mean().sqrt())
                assert dtype == torch.bfloat16 and gap < 0.25, f"{name} {dtype}: token {k} is {tok}, plain {best} (gap {gap:.3f})"
                break
            seq.append(tok)
        assert len(ours) == new


def test_preempted_requests_start_their_state_again(folders):
    """A pool too small for all requests with the policy that releases the newest one and recomputes it later: its states (and the
    token before its first one) start from nothing at its second admission, and the tokens are those of a pool that is large
    enough."""
    from nanospec_amd import Engine, EngineConfig, SamplingParams

    page = CONFIGS["A"]["page"]
    model = engine_model(folders["A"], "A", torch.float32)
    prompts = [t[:20] for t in sequences("A").values() if len(t) >= 20] * 2
    new = 30
    calm = Engine(model, EngineConfig(num_blocks=128, block_size=page)).generate(prompts, SamplingParams(max_tokens=new))
    eng = Engine(model, EngineConfig(num_blocks=23, block_size=page, on_exhaustion="preempt", prefill_chunk=16))
    rough = eng.generate(prompts, SamplingParams(max_tokens=new))
    assert eng.sched.preempted_total > 0, "the pool was meant to run out"
    assert rough == calm
    eng.cache.check()


def test_the_command_lines_generate_and_replay(folders, tmp_path):
    """``python -m nanospec_amd`` continues a prompt greedily; ``bin/trace_run`` replays two steps of the same model."""
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    root = Path(__file__).resolve().parent.parent
    out = subprocess.run([sys.executable, "-m", "nanospec_amd", "--model", str(folders["B"]), "--prompt-ids", "1,2,3,4,5", "--max-tokens", "4",
                          "--dtype", "float32", "--block-size", "16"], cwd=root, capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    row = json.loads(out.stdout.strip().splitlines()[-1])
    cfg, w = read_folder(folders["B"], torch.float32)
    seq = [1, 2, 3, 4, 5]
    for tok in row["output_ids"]:
        assert tok == int(pm.forward(cfg, w, seq)[-1].argmax())
        seq.append(tok)
    assert len(row["output_ids"]) == 4
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [1]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [4, 5], "want": [0, 1]}], "end": ["a"]}]
    out = subprocess.run([str(root / "bin" / "trace_run"), "--model", str(folders["B"]), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert out.returncode == 0 and "done 1" in out.stdout.splitlines(), out.stderr[-2000:]
    ref = pm.forward(cfg, w, [1, 2, 3, 4, 5]).float()
    for step, rows in ((0, [1]), (1, [3, 4])):
        got = torch.from_numpy(np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")).view(len(rows), -1)
        close(got, ref[rows], torch.float32, f"step {step}")


def drawn_config(seed: int) -> dict:
    """A configuration drawn from everything the design lets a model choose."""
    rng = random.Random(2000 + seed)
    layers = []

    def left():
        G = rng.choice([1, 2, 3])
        D = rng.choice([8, 12, 24, 40])
        return attn(G * rng.choice([1, 2, 3]), G, D, rng.choice([8, 20, 24, D]), rng.uniform(0.1, 0.5), rng.choice([2, 4, D]), rng.choice([100.0, 1e4]))

    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["parallel", "gla", "parallel_2"])
        if kind == "gla":
            mixer = gla(rng.choice([1, 2, 5]), rng.choice([4, 9, 16, 36]), rng.choice([5, 16, 40]), rng.choice([1.0, 4.0, 16.0]))
        elif kind == "parallel":
            mixer = parallel(left(), rng.choice([12, 33, 64]), rng.choice([1, 3, 16, 24, 40]), rng.choice([1, 4, 8]), rng.choice([1, 2, 4, 6]),
                             rng.uniform(0.5, 1.5), rng.uniform(0.5, 1.5))
        else:
            g = rng.choice([1, 2, 3])
            H = g * rng.choice([1, 2, 3])
            E = rng.choice([4, 10, 24])
            mixer = parallel_2(left(), H, E, rng.choice([1, 6, 16, 28]), g, rng.choice([1, 3, 4]), rng.choice([1, 2, H]) if E % 2 == 0 else H)
        r = rng.random()
        if r < 0.2:
            mlp = None
        elif r < 0.45:
            mlp = dense(rng.choice([8, 20, 48]))
        else:
            count = rng.choice([1, 2, 3])
            per = rng.randint(1, 4)
            n = count * per
            identity = rng.randint(0, min(3, n - 1))
            keep = rng.randint(1, count)
            mlp = moe(n - identity, rng.randint(1, keep * per), rng.choice([8, 20, 48]), identity, (count, keep), rng.choice([1.0, 2.5]), rng.choice([0, 8, 40]))
        layers.append(layer(mixer, mlp))
    cfg = {"architecture": "Meropel", "vocab": rng.choice([50, 128, 333]), "width": rng.choice([32, 50, 64, 100, 136]),
           "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-3])}, "logit_scale": rng.choice([0.3, 1.0]), "layers": layers}
    if rng.random() < 0.8:
        cfg["embedding"] = {"bigram": {"buckets": rng.choice([1, 7, 1000]), "mul_prev": rng.choice([1, 127, 99991]), "mul_cur": rng.choice([1, 5, 100003])}}
    return cfg


@BOTH
@pytest.mark.parametrize("seed", range(8))
def test_drawn_configurations_match_plain(tmp_path, seed, dtype):
    """Eight configurations drawn at random: in portions, then in a mixed batch, in a small pool.  (Some of them choose one
    expert of two: there a close call that bfloat16 rounding moves changes a row altogether, so more rows may differ by more
    than rounding.)"""
    from nanospec_amd.loader import load_model

    folder = write_folder(tmp_path / "m", drawn_config(seed), seed)
    model = load_model(folder, dtype=dtype)
    cfg, w = read_folder(folder, dtype)
    seqs = {f"r{i}": random_tokens(n, cfg["vocab"], 7 * i + seed) for i, n in enumerate((1, 2, 19, 70, 131))}
    ref = {rid: pm.forward(cfg, w, toks).float() for rid, toks in seqs.items()}
    page = [4, 8, 16][seed % 3]
    steps, where = traces.portions(seqs, seed=seed)
    replay(model, steps, where, ref, dtype, 192, page, loose_share=5, caps=CAPS)
    steps, where, peak = traces.mixed(seqs, seed=seed, max_live=3)
    replay(model, steps, where, ref, dtype, peak, page, loose_share=5, caps=CAPS)


@BOTH
@pytest.mark.parametrize("mark", [0, 15, 16, 17, 131])
def test_a_far_key_decides_the_answer(folders, tmp_path, dtype, mark):
    """The first layer of model B has attention with one head.  Its query matrix is made minus its key matrix where nothing is
    rotated (zero where it is), and two tokens get embeddings of opposite sign: the query of the one at the end then meets the
    key of the other (and not its own), ``mark`` tokens into the sequence, with the largest score there can be, among hundreds
    of others.  The plain logits at the end change when that one token is taken away; the framework's follow them, in a prompt
    and decoded."""
    from nanospec_amd.loader import load_model

    def change(w):
        w["l0.mix.left.q"] = -8.0 * w["l0.mix.left.k"]
        w["l0.mix.left.q"][:2] = 0.0
        w["l0.mix.left.o"] *= 8.0
        w["embed"][4] = torch.randn(w["embed"].shape[1], generator=torch.Generator().manual_seed(1))
        w["embed"][3] = -w["embed"][4]

    X, Y, Z = 3, 4, 5
    folder = write_folder(tmp_path / "far", CONFIGS["B"]["cfg"], CONFIGS["B"]["seed"], change)
    cfg, wd = read_folder(folder, dtype)
    toks = [t if t not in (X, Y) else Z for t in random_tokens(300, cfg["vocab"], 5)]
    toks[mark], toks[-1] = X, Y
    ref = pm.forward(cfg, wd, toks).float()
    without = pm.forward(cfg, wd, toks[:mark] + [Z] + toks[mark + 1 :]).float()[-1]
    spread = (ref[-1] - ref[-1].mean()).pow(2).mean().sqrt()
    assert (ref[-1] - without).pow(2).mean().sqrt() > 0.1 * spread, "the test's far key was meant to matter"
    model = load_model(folder, dtype=dtype)
    for tail in (1, 40):
        steps, where = traces.tail_decoded({"a": toks}, tail=tail)
        replay(model, steps, where, {"a": ref}, dtype, 320, CONFIGS["B"]["page"])


# ------------------------------------------------------------------------------------------------ mechanisms alone


def built(role, spec, dtype, seed, scale=sharpened, prefix=""):
    """A part as the framework builds it, with random weights -> (part, plain weights)."""
    from nanospec_amd.parts import registry
    from nanospec_amd.weights import random_tensors

    part = registry.build(role, spec, prefix)
    tensors = random_tensors(part.wanted(), seed, torch.float32)
    for name, t in tensors.items():
        t *= scale(name)
    stored = {k: v.to(dtype) for k, v in tensors.items()}
    part.load(lambda name: stored[name], dtype, DEV)
    return part, {k: v.double() for k, v in stored.items()}


def in_steps(part, seqs, plain, slots, cuts, floats, dtype, plan=None, reuse=True, tol=(1e-4, 3e-2)):
    """Requests in state slots that are not in order, cut into unequal portions, each step finding the state that the step before
    left; then one more request in a slot that another one had, from zero."""
    ref = [plain(s.double()) for s in seqs]
    state = torch.randn(max(slots) + 2, floats, device=DEV)  # what earlier requests left
    ctx = PartCtx()

    def run(live, parts):
        x = torch.cat([seqs[b][a:e] for b, (a, e) in zip(live, parts)]).to(DEV)
        ctx.requests([e - a for a, e in parts], [slots[b] for b in live], [p for a, e in parts for p in range(a, e)], plan, spare=2)
        mark = ctx.arena.mark()
        y = part.forward(ctx, x, type("V", (), {"state": state})()).cpu()
        ctx.arena.release(mark)
        worst, rms = off(y, torch.cat([ref[b][a:e] for b, (a, e) in zip(live, parts)]))
        assert worst <= tol[0] if dtype == torch.float32 else rms <= tol[1], (live, parts, worst, rms)

    n = len(cuts)
    untouched = state[max(slots) + 1].clone()
    for b in range(n):
        state[slots[b]] = 0  # as at admission
    for step in range(max(len(c) for c in cuts) - 1):
        live = [b for b in range(n) if step + 1 < len(cuts[b])]
        run(live, [(cuts[b][step], cuts[b][step + 1]) for b in live])
    if reuse:
        state[slots[n]] = 0
        run([n], [(0, len(seqs[n]))])
    assert torch.equal(state[max(slots) + 1], untouched), "a slot that no request has was written"


def requests(width, dtype, lengths=(9, 5, 214, 70), seed=7):
    g = torch.Generator().manual_seed(seed)
    return [torch.randn(n, width, generator=g).to(dtype) for n in lengths]


SLOTS = [4, 0, 2, 0]
CUTS = [[0, 4, 5, 9], [0, 1, 2, 3, 4, 5], [0, 2, 19, 150, 214]]


@BOTH
@pytest.mark.parametrize("chunked", [False, True], ids=["scan", "chunks"])
@pytest.mark.parametrize("inner,N,R,K", [(300, 9, 4, 3), (50, 5, 3, 4), (24, 1, 1, 1), (33, 16, 8, 2), (64, 24, 4, 3), (40, 40, 5, 4), (20, 100, 8, 6), (9, 200, 2, 3), (7, 300, 1, 4)])
def test_selective_scan_through_the_part(monkeypatch, dtype, inner, N, R, K, chunked):
    """Mamba alone: states of one lane and of many, taps from one to six; token by token and with long portions in chunks (up to 32
    states)."""
    from nanospec_amd.config.spec import SelectiveScanSpec
    from nanospec_amd.parts import retention
    from nanospec_amd.parts.retention import CHUNKS

    monkeypatch.setattr(retention, "CHUNKED_FROM", 64)
    W = 48
    part, w = built("mixer", SelectiveScanSpec(hidden=W, inner=inner, state=N, dt_rank=R, conv=K), dtype, inner + N)
    assert set(w) == {"in", "conv", "conv.b", "x", "dt", "dt.b", "A_log", "D", "o"}
    assert bool(part.batch_plans()) == (N <= 32)
    m = dict(inner=inner, state=N, dt_rank=R)
    in_steps(part, requests(W, dtype), lambda h: pm.mamba(h, w, "", m), SLOTS, CUTS, part.slot_floats, dtype, CHUNKS if chunked else None)


@BOTH
@pytest.mark.parametrize("chunked", [False, True], ids=["scan", "chunks"])
@pytest.mark.parametrize("H,E,N,G,K,parts", [(6, 9, 7, 3, 2, 2), (1, 40, 1, 1, 3, 1), (4, 64, 128, 1, 4, 4), (4, 100, 36, 2, 4, 8), (8, 48, 64, 4, 1, 2), (2, 10, 200, 2, 5, 1)])
def test_state_space_through_the_part(monkeypatch, dtype, H, E, N, G, K, parts, chunked):
    """Mamba-2 alone, token by token and with long portions in chunks (where the sizes allow it)."""
    from nanospec_amd.config.spec import StateSpaceSpec
    from nanospec_amd.parts import retention
    from nanospec_amd.parts.retention import CHUNKS

    monkeypatch.setattr(retention, "CHUNKED_FROM", 64)
    W = 48
    part, w = built("mixer", StateSpaceSpec(hidden=W, heads=H, value_dim=E, state=N, groups=G, conv=K, norm_groups=parts, norm_eps=1e-5), dtype, H * E + N)
    assert set(w) == {"in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o"}
    assert bool(part.batch_plans()) == (N % 4 == 0 and (H * E) % 4 == 0)
    m = dict(heads=H, vdim=E, state=N, groups=G, norm_groups=parts)
    in_steps(part, requests(W, dtype), lambda h: pm.mamba2(h, w, "", m, 1e-5), SLOTS, CUTS, part.slot_floats, dtype, CHUNKS if chunked else None)


@BOTH
@pytest.mark.parametrize("chunked", [False, True], ids=["scan", "chunks"])
@pytest.mark.parametrize("H,D,E,tau,rank", [(3, 20, 36, 4.0, 5), (1, 64, 8, 1.0, 8), (5, 9, 7, 16.0, 3), (2, 128, 256, 16.0, 16), (2, 16, 300, 0.25, 1), (1, 200, 40, 8.0, 24)])
def test_gated_linear_through_the_part(monkeypatch, dtype, H, D, E, tau, rank, chunked):
    """Gated linear attention alone, token by token and with long portions in chunks; with a small tau single tokens forget all that
    was before them in some channels."""
    from nanospec_amd.config.spec import GatedLinearSpec
    from nanospec_amd.parts import retention
    from nanospec_amd.parts.retention import CHUNKS

    monkeypatch.setattr(retention, "CHUNKED_FROM", 64)
    W = 48
    spec = GatedLinearSpec(hidden=W, heads=H, key_dim=D, value_dim=E, tau=tau, query_scale=D**-0.5, norm_eps=1e-5, decay_rank=rank)
    part, w = built("mixer", spec, dtype, H * D + E, lambda name: 15.0 if name in ("q", "k", "v", "g") else (20.0 if name in ("a1", "a2") else 1.0))
    assert set(w) == {"q", "k", "v", "g", "o", "norm", "a1", "a2", "a2.b"}
    assert bool(part.batch_plans()) == (D % 4 == 0)
    m = dict(heads=H, dim=D, vdim=E, tau=tau)
    in_steps(part, requests(W, dtype), lambda h: pm.gla(h, w, "", m, 1e-5), SLOTS, CUTS, -(-H * D * E // 4) * 4, dtype, CHUNKS if chunked else None)


@pytest.mark.parametrize("per", ["head", "channel"])
@pytest.mark.parametrize("H,G,D,E", [(2, 2, 16, 24), (4, 2, 128, 64), (3, 1, 36, 65)])
@pytest.mark.parametrize("gap", [63, 64, 65, 127, 128, 200])
def test_chunks_read_back_what_the_first_token_wrote(monkeypatch, gap, H, G, D, E, per):
    """One key channel is written by the first token alone and read by the last one alone, ``gap`` tokens later: in the same
    portion, inside the chunk and across chunks, and in the portion behind it; the read-out is what the decays between them
    left of the first token's value (one head or channel forgets nothing, another everything at once in the middle)."""
    from nanospec_amd.kernels import ops
    from nanospec_amd.parts import retention
    from nanospec_amd.parts.retention import CHUNKS, ChunkPlan

    monkeypatch.setattr(retention, "CHUNKED_FROM", 64)
    G = H if per == "channel" else G
    n = gap + 1
    g = torch.Generator().manual_seed(gap)
    q, k, v = torch.zeros(n, G, D), torch.randn(n, G, D, generator=g), torch.randn(n, H, E, generator=g)
    k[:, :, 3] = 0.0
    k[0, :, 3] = 1.0  # only the first token writes channel 3
    q[-1, :, 3] = 1.0  # only the last token reads, and only channel 3
    rates = torch.tensor([0.0, 1.0, 40.0][:H] + [0.01] * (H - 3 if H > 3 else 0))
    width = H if per == "head" else H * D
    logs = -0.02 * torch.rand(n, H, width // H, generator=g) * rates[None, :, None]
    logs[n // 2, -1] = -200.0  # the last head forgets everything half way
    scale, skip = torch.rand(n, H, generator=g) + 0.5, torch.randn(H, generator=g)
    left = torch.exp(logs[1:, :, 3 if per == "channel" else 0].double().sum(0))
    want = v[0].double() * left[:, None]
    if per == "head":
        want = want * scale[0].double()[:, None] + skip.double()[:, None] * v[-1].double()
    row = torch.cat([v.reshape(n, -1), torch.full((n, (4 - H * E % 4) % 4), 7.0), k.reshape(n, -1), q.reshape(n, -1)], dim=1)  # v | gap | k | q
    k_at = row.shape[1] - 2 * G * D
    row = torch.cat([row, torch.zeros(n, (4 - row.shape[1] % 4) % 4)], dim=1).to(DEV).contiguous()
    for cuts in ((0, n), tuple(sorted({0, n - 64, n}))):
        state = torch.zeros(3, -(-H * D * E // 4) * 4, device=DEV)
        out = torch.empty(n, H * E, device=DEV)
        for a, b in zip(cuts, cuts[1:]):
            ctx = PartCtx()
            ctx.requests([b - a], [1], list(range(a, b)), CHUNKS, spare=1)
            extra = dict(value_scale=scale[a:b].to(DEV).contiguous(), skip=skip.to(DEV)) if per == "head" else {}
            rows = ops.DecayRows(row[a:b].contiguous(), (k_at + G * D, k_at, 0), H, D, E, kv_heads=G, log_decay=logs[a:b].reshape(b - a, -1).to(DEV).contiguous(), **extra)
            if b - a >= 64:
                chunks, rest = ChunkPlan.view(ctx)
                assert rest == 0 and chunks.shape[0] == -(-(b - a) // 64) + 1
                ops.decay_chunks(rows, state, chunks, ctx.state_slots, torch.full((chunks.shape[0] * rows.words,), float("nan"), device=DEV), out[a:b])
            elif b > a:
                ops.decay_scan(rows, state, ctx.qo_indptr, ctx.state_slots, out[a:b])
        assert torch.allclose(out[-1].cpu().view(H, E).double(), want, rtol=1e-4, atol=1e-5), cuts
        assert state[0].abs().max() == 0 and state[2].abs().max() == 0


@pytest.mark.parametrize("strength", [0.001, 0.5, 3.0, 30.0, 1000.0])
@pytest.mark.parametrize("n", [64, 100, 193])
def test_chunks_with_decays_of_every_strength(n, strength):
    """Logarithms of the decays per channel from nearly nothing to far beyond what 32-bit exponentials hold over a chunk, weak and
    strong channels side by side: the chunked form against the plain recurrence."""
    from nanospec_amd.kernels import ops
    from nanospec_amd.parts.retention import CHUNKS, ChunkPlan

    H, D, E = 2, 40, 70
    g = torch.Generator().manual_seed(n)
    q, k, v = (torch.randn(n, H, s, generator=g) for s in (D, D, E))
    logs = -strength * torch.rand(n, H, D, generator=g) * (torch.rand(1, H, D, generator=g) < 0.5) - 0.01 * torch.rand(n, H, D, generator=g)
    want = pm.channel_decay_memory(q.double(), k.double(), v.double(), torch.exp(logs.double())).reshape(n, -1)
    row = torch.cat([q.reshape(n, -1), k.reshape(n, -1), v.reshape(n, -1)], dim=1).to(DEV).contiguous()
    ctx = PartCtx()
    from nanospec_amd.parts import retention

    before, retention.CHUNKED_FROM = retention.CHUNKED_FROM, 64
    try:
        ctx.requests([n], [1], list(range(n)), CHUNKS)
        chunks, _ = ChunkPlan.view(ctx)
    finally:
        retention.CHUNKED_FROM = before
    rows = ops.DecayRows(row, (0, H * D, 2 * H * D), H, D, E, log_decay=logs.reshape(n, -1).to(DEV).contiguous())
    out = ops.decay_chunks(rows, torch.zeros(2, H * D * E, device=DEV), chunks, ctx.state_slots, torch.empty(chunks.shape[0] * rows.words, device=DEV),
                           torch.empty(n, H * E, device=DEV))
    assert torch.isfinite(out).all()
    worst, rms = off(out, want)
    assert worst <= 2e-5 and rms <= 2e-6, (worst, rms)


@BOTH
@pytest.mark.parametrize("C,K", [(20, 4), (33, 3), (64, 2), (8, 1), (12, 7)])
def test_convolution_with_a_bias_across_steps(dtype, C, K):
    """Two requests in portions down to one token against the plain convolution over each whole sequence; the copy in the model's
    precision holds the same values."""
    from nanospec_amd.kernels import ops

    g = torch.Generator().manual_seed(C)
    seqs = [torch.randn(n, C + 4, generator=g).to(dtype) for n in (13, 9)]
    taps, bias = torch.randn(C, K, generator=g), torch.randn(C, generator=g)
    ref = [pm.silu(pm.causal_conv(s[:, 4:].double(), taps.double(), bias.double())) for s in seqs]
    state = torch.zeros(4, 8 + (K - 1) * C, device=DEV)
    ctx, slots = PartCtx(), [3, 1]
    for cuts in ((0, 1, 0, 1), (1, 2, 1, 2), (2, 7, 2, 6), (7, 8, 6, 7), (8, 13, 7, 9)):
        parts = [(cuts[0], cuts[1]), (cuts[2], cuts[3])]
        ctx.requests([b - a for a, b in parts], slots, [0] * sum(b - a for a, b in parts))
        x = torch.cat([s[a:b] for s, (a, b) in zip(seqs, parts)]).to(DEV)
        out, copy = torch.empty(len(x), C, device=DEV), torch.empty(len(x), C, dtype=dtype, device=DEV)
        ops.conv_silu_carry(x[:, 4:], taps.to(DEV), state, 8, ctx.token_req, ctx.qo_indptr, ctx.state_slots, out, bias=bias.to(DEV), copy=copy,
                            single=len(x) == 2)
        want = torch.cat([r[a:b] for r, (a, b) in zip(ref, parts)])
        assert (out.cpu().double() - want).abs().max() <= 1e-5 and torch.equal(copy, out.to(dtype))
    assert state[0].abs().max() == 0 and state[2].abs().max() == 0 and state[:, :8].abs().max() == 0


def attention_spec(kind, H, G, D, E, scale, dims, W, eps=1e-5):
    from nanospec_amd.config import MeropelConfig
    from nanospec_amd.config.meropel import MeropelAttention, MeropelLayer, MeropelScan, MeropelStateSpace

    right = MeropelScan(8, 2, 2, 2) if kind == "parallel" else MeropelStateSpace(2, 4, 2, 1, 2, 1)
    l = MeropelLayer(type=kind, left=MeropelAttention(H, G, D, E, scale, dims, 1000.0), right=right)
    return MeropelConfig(vocab=8, width=W, layers=(), norm_eps=eps)._mixer(l).left


@BOTH
@pytest.mark.parametrize("kind", ["parallel", "parallel_2"])
@pytest.mark.parametrize("H,G,D,E,dims", [(6, 3, 12, 20, 6), (1, 1, 16, 16, 2), (4, 2, 48, 32, 32), (8, 2, 32, 32, 32), (4, 4, 10, 10, 10), (9, 3, 24, 8, 4)])
def test_attention_sides_over_six_steps(dtype, kind, H, G, D, E, dims):
    """The two attention mixers alone over a paged cache whose pages are not in order: a prompt portion, a second one, then single
    tokens and short portions, against the plain mixer over the whole sequence.  In the mixer whose keys no norm bounds one
    token's input is made so large that its key stands out, at a page's first or last place or far back; behind norms all keys
    are alike in size, and the token's direction alone makes it stand out for the last query."""
    from nanospec_amd.cache.storage import PagedView

    Wd, T, page = 72, 90, 8
    spec = attention_spec(kind, H, G, D, E, 0.3, dims, Wd)
    part, wd = built("mixer", spec, dtype, H * D + E, lambda name: 1.0 if name.endswith("norm") else (10.0 if name.endswith(".b") else 7.0))
    assert set(wd) == ({"q", "k", "v", "g", "o"} if kind == "parallel" else {"q", "k", "v", "o", "q.b", "k.b", "v.b", "q.norm", "k.norm"})
    m = attn(H, G, D, E, 0.3, dims, 1000.0)
    plain = lambda y: pm.gated_attention(y.double(), wd, "", m) if kind == "parallel" else pm.normed_attention(y.double(), wd, "", m, 1e-5)
    g = torch.Generator().manual_seed(H * D + 1)
    pages = -(-T // page)
    order = list(range(pages))
    random.Random(2).shuffle(order)
    for mark in (0, 7, 8, 40):
        x = torch.randn(T, Wd, generator=g).to(dtype)
        calm, token = plain(x), x[mark].clone()
        for by in (12.0, -12.0, 24.0, -24.0, 48.0, -48.0):  # (one of the signs meets the last query's favour)
            x[mark] = token * by
            ref = plain(x)
            share = (ref[-1] - calm[-1]).abs().max() / calm[-1].abs().max()
            if share > 0.05:
                break
        assert share > 0.05, "the large token was meant to matter far away"
        cache = PagedView(0, torch.zeros(pages, G, page, D, dtype=dtype, device=DEV), torch.zeros(pages, G, E, page, dtype=dtype, device=DEV))
        got, at = [], 0
        for n in (37, 30, 1, 1, 2, 19):
            ctx = step_context([n], [at], [order])
            got.append(part.forward(ctx, x[at : at + n].to(DEV), cache, True).cpu())
            at += n
        worst, rms = off(torch.cat(got), ref)
        # (sharp soft-maxes magnify a rounding in single places: the root mean square is what bfloat16 is held to)
        assert worst <= 3e-5 if dtype == torch.float32 else rms <= 0.03, (mark, worst, rms)


@BOTH
@pytest.mark.parametrize("H,G,hd,vd,page", [(4, 2, 48, 32, 8), (6, 2, 32, 32, 16), (3, 3, 20, 12, 4), (4, 1, 64, 48, 8)])
def test_a_key_that_stands_out_at_the_pages_edges(dtype, H, G, hd, vd, page):
    """All keys small but one, placed far back and at a page's first and last place, in a prompt's rows and for a single decoded
    row, by the kernels that the attention sides run at these sizes (the matrix cores' in bfloat16)."""
    from nanospec_amd.kernels import ops
    from nanospec_amd.parts.attention import launch_plans, wide_attention

    T, scale = 200, 0.3
    g = torch.Generator().manual_seed(page)
    for mark in sorted({0, page - 1, page, 97, T - 2, T - 1, (T // page) * page - 1}):
        keys, vals, q = 0.1 * torch.randn(T, G, hd, generator=g), torch.randn(T, G, vd, generator=g), torch.randn(T, H, hd, generator=g)
        for a in range(G):
            keys[mark, a] = 4.0 * q[T - 1, a * (H // G)] / scale / hd  # the favourite of the last query of each group's first head
        keys, vals, q = keys.to(dtype), vals.to(dtype), q.to(dtype)
        kp, vp, table = paged(keys, vals, page, order_seed=mark)
        want = pm.grouped_attention(q.double(), keys.double(), vals.double(), scale)
        for first in (0, T - 1):
            n = T - first
            ctx = step_context([n], [first], [table[0].tolist()])
            rows, out = q[first:].reshape(n, H * hd).to(DEV).contiguous(), torch.zeros(n, H * vd, dtype=dtype, device=DEV)
            if hd == vd and ops.mfma_attention_takes(dtype, hd, page):
                for plan in launch_plans(ctx, H // G, G, hd):
                    ops.attention_mfma(rows, out, kp, vp, plan.tiles, ctx.block_tables[0], H, G, hd, scale, hp=plan.hp, splits=plan.splits,
                                       workspace=plan.workspace, qt=plan.qt, coop=plan.coop)
            elif ops.wide_attention_takes(dtype, hd, vd, page):
                wide_attention(ctx, rows, out, type("V", (), {"k": kp, "v": vp})(), ctx.block_tables[0], H, G, hd, vd, scale)
            else:
                ops.attention_generic(rows, out, kp, vp, ctx.token_req, ctx.positions, ctx.block_tables[0], H, G, hd, scale, v_dim=vd)
            err = (out.cpu().double().view(n, H, vd) - want[first:]).abs().max()
            assert err <= (2e-5 if dtype == torch.float32 else 3e-2), (mark, first, float(err))


@BOTH
@pytest.mark.parametrize("W,mlp", [(90, moe(6, 3, 20, 2, (4, 2), 1.7, shared=28)), (64, moe(1, 1, 48, 1, (2, 1), 0.7)), (128, moe(14, 3, 32, 2, (4, 2), 1.3, shared=64)),
                                   (128, moe(4, 4, 64)), (72, moe(10, 5, 40, 5, (3, 3), 0.5)), (128, moe(3, 4, 32, 13, (4, 3), 1.1))])
@pytest.mark.parametrize("rows", [1, 7, 300])
def test_mixture_with_identity_experts_through_the_part(dtype, W, mlp, rows):
    """The feed-forward as the framework builds it against the plain one, for one row (streamed experts), a few, and many (the
    sorted, tiled products); with none, some and mostly identity experts."""
    from nanospec_amd.config import MeropelConfig
    from nanospec_amd.config.meropel import MeropelFF

    spec = MeropelConfig(vocab=8, width=W, layers=())._ffn(MeropelFF.from_hf(mlp))
    part, w = built("ffn", spec, dtype, W + mlp["router"]["experts"], lambda name: 30.0 if name == "router" else (4.0 if name == "correction" else 6.0))
    x = torch.randn(rows, W, generator=torch.Generator().manual_seed(rows)).to(dtype)
    y = part.forward(PartCtx(), x.to(DEV)).cpu().double()
    want = pm.moe(x.double(), w, "", mlp)
    if rows == 300 and mlp["router"]["identity"]:
        sel, _ = pm.route(x.double(), w, "", mlp["router"])
        assert (sel >= mlp["router"]["experts"]).any() and (sel < mlp["router"]["experts"]).any(), "both kinds were meant to be chosen"
    if dtype == torch.float32:
        assert (y - want).abs().max() <= 1e-4 * want.abs().max()
    else:  # (a row whose router scores lie within rounding of each other may take another expert)
        err = (y - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
        assert (err > 0.05).sum() <= max(1, rows // 25), err.max()


@pytest.mark.parametrize("n,groups,keep,top", [(12, 1, 1, 4), (12, 3, 2, 5), (12, 12, 5, 5), (14, 2, 1, 7), (64, 8, 3, 6), (1, 1, 1, 1)])
@pytest.mark.parametrize("shift", [0.0, -5.0])
def test_router_scores_groups_and_weights(n, groups, keep, top, shift):
    """Soft-max over all outputs, groups judged by their best choice score (all of them negative with ``shift``), weights from the
    scores without the correction, over their sum, times the scale."""
    from nanospec_amd.kernels import ops

    g = torch.Generator().manual_seed(n + groups)
    for rows in (1, 5, 40):
        h, router = torch.randn(rows, 24, generator=g), 0.5 * torch.randn(n, 24, generator=g)
        corr = 0.2 * torch.randn(n, generator=g) + shift
        sel, wt = torch.empty(rows, top, dtype=torch.int32, device=DEV), torch.empty(rows, top, device=DEV)
        ops.moe_route(h.to(DEV), router.to(DEV), None, top, sel, wt, score="softmax_all", correction=corr.to(DEV), groups=groups, keep=keep, group_best=1, scale=2.5)
        want_sel, want_wt = pm.choose(h @ router.T, corr, top, groups, keep, 2.5)
        assert sel.cpu().tolist() == want_sel.tolist()
        assert torch.allclose(wt.cpu(), want_wt, rtol=1e-4, atol=1e-6)


def test_a_group_is_judged_by_its_best_or_its_two_best():
    from nanospec_amd.kernels import ops

    router = torch.zeros(6, 4)
    router[:, 0] = torch.tensor([5.0, -9.0, -9.0, 4.0, 4.0, -9.0])
    h = torch.tensor([[1.0, 0.0, 0.0, 0.0]])
    for best, score, first in ((1, "softmax_all", 0), (2, "sigmoid", 3)):
        sel, wt = torch.empty(1, 1, dtype=torch.int32, device=DEV), torch.empty(1, 1, device=DEV)
        ops.moe_route(h.to(DEV), router.to(DEV), None, 1, sel, wt, score=score, groups=2, keep=1, group_best=best)
        assert sel.item() == first


@BOTH
@pytest.mark.parametrize("W", [20, 90, 300, 2048])
def test_the_weighted_sum_of_normed_outputs(dtype, W):
    from nanospec_amd.kernels import ops

    g = torch.Generator().manual_seed(W)
    a, b = 3.0 * torch.randn(6, W, generator=g), 0.01 * torch.randn(6, W, generator=g)
    wa, wb, ba, bb = (torch.randn(W, generator=g) for _ in range(4))
    a, b, wa, wb, ba, bb = (t.to(dtype) for t in (a, b, wa, wb, ba, bb))
    d = lambda t: t.to(DEV)
    got = ops.normed_sum(d(a), d(b), 0.5, 0.5, d(wa), d(wb), 1e-5, torch.empty_like(d(a)))
    worst, _ = off(got, pm.mean_of_normed(a.double(), b.double(), wa.double(), wb.double(), 1e-5))
    assert worst <= (1e-5 if dtype == torch.float32 else 1e-2)
    got = ops.normed_sum(d(a), d(b), 0.7, -1.2, d(wa), d(wb), 1e-3, torch.empty_like(d(a)), bias=d(ba), bias_b=d(bb))
    want = 0.7 * pm.rms(a.double() + ba.double(), 1e-3) * wa.double() - 1.2 * pm.rms(b.double() + bb.double(), 1e-3) * wb.double()
    worst, _ = off(got, want)
    assert worst <= (1e-5 if dtype == torch.float32 else 1e-2)


@BOTH
@pytest.mark.parametrize("heads,E", [(1, 40), (6, 20), (3, 1), (4, 128)])
def test_a_gate_per_head(dtype, heads, E):
    from nanospec_amd.kernels import ops

    g = torch.Generator().manual_seed(E)
    x, gate = torch.randn(5, heads * E, generator=g).to(dtype), (3.0 * torch.randn(5, heads + 9, generator=g)).to(dtype)
    xs = x.to(DEV)
    ops.gate_mul(xs, gate.to(DEV)[:, 9:], out=xs)
    want = (x.double().view(5, heads, E) * torch.sigmoid(gate[:, 9:].double())[:, :, None]).reshape(5, -1)
    worst, _ = off(xs, want)
    assert worst <= (1e-6 if dtype == torch.float32 else 4e-3)


@BOTH
@pytest.mark.parametrize("parts,E", [(1, 48), (4, 24), (2, 1000), (8, 64)])
def test_the_gate_in_front_of_a_norm_in_parts(dtype, parts, E):
    from nanospec_amd.kernels import ops

    g = torch.Generator().manual_seed(E)
    o, wn = 5.0 * torch.randn(5, parts * E, generator=g), 1.0 + 0.3 * torch.randn(parts * E, generator=g)
    gate = (2.0 * torch.randn(5, parts * E + 8, generator=g)).to(dtype)
    out = ops.gated_rms(o.to(DEV), gate.to(DEV)[:, 8:], wn.to(DEV), 1e-5, parts, out=torch.empty(5, parts * E, dtype=dtype, device=DEV), silu=True, gate_first=True)
    x = (o.double() * pm.silu(gate[:, 8:].double())).view(5, parts, E)
    worst, _ = off(out, pm.rms(x, 1e-5).reshape(5, -1) * wn.double())
    assert worst <= (1e-5 if dtype == torch.float32 else 8e-3)


@BOTH
def test_the_logarithms_of_decays(dtype):
    """Step sizes and decays over the whole range of their inputs, 32-bit values from inputs in the model's precision."""
    from nanospec_amd.kernels import ops

    H, n = 5, 9
    z = torch.linspace(-90.0, 90.0, n * H).view(n, H).to(dtype)
    bias, a_log = torch.linspace(-1.0, 1.0, H), torch.linspace(-2.0, 2.0, H)
    dt, logs = torch.empty(n, H, device=DEV), torch.empty(n, H, device=DEV)
    ops.log_decay_heads(z.to(DEV), bias.to(DEV), a_log.to(DEV), dt, logs)
    want = pm.softplus(z.double() + bias.double())
    assert torch.allclose(dt.cpu().double(), want, rtol=1e-5, atol=1e-30) and torch.allclose(logs.cpu().double(), -torch.exp(a_log.double()) * want, rtol=1e-5, atol=1e-30)
    proj = torch.zeros(n, 4 * H, dtype=dtype, device=DEV)
    ops.retention_prep(proj, (0, H, 2 * H), torch.zeros(n, dtype=torch.int32, device=DEV), None, 1, H, 2 * H, 0, 1.0, torch.empty(n, 4 * H, device=DEV),
                       decays=(z.to(DEV), bias.to(DEV), 16.0, logs))
    assert torch.allclose(logs.cpu().double(), -pm.softplus(-(z.double() + bias.double())) / 16.0, rtol=1e-5, atol=1e-30)


def test_operands_that_do_not_fit_are_refused():
    from nanospec_amd.kernels import ops

    z = lambda *s: torch.zeros(*s, device=DEV)
    with pytest.raises(ops.KernelRefused):
        ops.DecayRows(z(4, 30), (0, 8, 16), 2, 4, 8, log_decay=z(4, 2))  # the row does not hold v
    with pytest.raises(ops.KernelRefused):
        ops.DecayRows(z(4, 32), (0, 8, 16), 2, 4, 8, log_decay=z(4, 3))
    with pytest.raises(ops.KernelRefused):
        ops.DecayRows(z(4, 32), (0, 8, 16), 2, 4, 8, decay=z(2), skip=z(2))
    with pytest.raises(ops.KernelRefused):
        ops.gate_mul(z(4, 12), z(4, 5), out=z(4, 12))
    with pytest.raises(ops.KernelRefused):
        ops.moe_route(z(2, 8), z(6, 8), None, 2, torch.zeros(2, 2, dtype=torch.int32, device=DEV), z(2, 2), score="max")
    with pytest.raises(ops.KernelRefused):
        ops.SelectiveRows(z(3, 6), z(3, 6), z(3, 7), 0, 4, z(3, 6), z(6), z(6, 4), z(6), z(1, 24), z(3, 6))
