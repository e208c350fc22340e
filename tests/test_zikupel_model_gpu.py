"""The Zikupel decoder in the engine against the plain implementation, under every way of cutting
the work: whole prompts, prompts then single tokens, portions down to two tokens, unequal requests
side by side, pages and slots that are given back and used again, long decoding, keys and states that
stand out far back, and greedy generation through the engine's own entry point and scheduler."""

from __future__ import annotations

import copy
import math

import pytest
import torch

from tests.darovik_helpers import load_model_folder
from tests.helpers import random_tokens
from tests.plain import zikupel as plain
from tests.zikupel_helpers import CONFIGS, attn, layer, lightning, make_model_dir, model
from tests.test_cuts_gpu import collect

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
IDS = ["f32", "bf16"]


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, (config, page) in CONFIGS.items():
        folder = make_model_dir(tmp_path_factory.mktemp(f"zikupel_{name}"), config, seed=71 + len(out))
        cfg, weights = load_model_folder(folder)
        out[name] = (folder, cfg, weights, page)
    return out


_plain: dict = {}


def oracle(name, cfg, weights, tokens, dtype):
    """Logits of the plain model and, position by position, how far they move when every weight is
    moved by a random relative amount of the size of ``dtype``'s rounding; in bfloat16 infinitely far where a
    router has a close call: the last chosen expert's logit and the next one's within a tenth of the spread
    of its logits (sublayers read the stream unnormed, so its rounding reaches the router as it is)."""
    key = (name, tuple(tokens), dtype)
    if key not in _plain:
        size = 2.0 ** -24 if dtype == torch.float32 else 2.0 ** -9
        gen = torch.Generator().manual_seed(99)
        moved = {k: v * (1 + size * torch.randn(v.shape, generator=gen, dtype=v.dtype)) for k, v in weights.items()}
        close = torch.zeros(len(tokens), dtype=torch.bool)
        real = plain.route

        def watched(h, w, top):
            z = (h @ w["router"].T).sort(-1, descending=True).values
            if z.shape[1] > top:
                close.logical_or_((z[:, top - 1] - z[:, top]) < 0.1 * z.std(-1))
            return real(h, w, top)

        plain.route = watched
        try:
            want = plain.forward(cfg, weights, tokens)
        finally:
            plain.route = real
        other = plain.forward(cfg, moved, tokens)
        _plain[key] = want, [math.inf if close[i] and dtype == torch.bfloat16 else row_error(other[i], want[i])
                             for i in range(len(tokens))]
    return _plain[key]


def session_for(folder, dtype, page, max_tokens, **kw):
    from kvcore_amd.engine.replay import TraceSession

    return TraceSession(str(folder), dtype, max_tokens=max_tokens, block_size=page, poison_cache=True, **kw)


def row_error(row, ref) -> float:
    d = row - ref
    d = d - d.mean()
    return float(d.pow(2).mean().sqrt() / (ref - ref.mean()).pow(2).mean().sqrt())


def compare(got, want, dtype, excused=0):
    """Rows of logits against the plain model's (``want[id]`` from ``oracle``): the difference with its
    mean taken off over the row's own size.  In float32 every position must lie within 2e-4; in
    bfloat16 within 4e-2 or five times what rounding the weights does at that place, but for those where a
    router's call is close (``oracle``) and one position in twenty (or ``excused``)."""
    assert got, "nothing was compared"
    base, far, inside = (2e-4 if dtype == torch.float32 else 4e-2), [], 0
    for (rid, pos), row in sorted(got.items()):
        assert torch.isfinite(row).all(), f"non-finite logits at {rid}:{pos}"
        ref, floor = want[rid]
        err = row_error(row, ref[pos])
        inside += err <= max(base, 2 * floor[pos])
        if err > max(base, 5 * floor[pos]):
            far.append(f"{rid}:{pos} differs by {err:.3e} (rounding alone: {floor[pos]:.1e})")
    allowed = max(excused, len(got) // 20) if dtype == torch.bfloat16 else 0
    assert len(far) <= allowed, (len(far), len(got), far[:5])
    assert 2 * inside >= len(got), f"only {inside} of {len(got)} positions lie within {base} or twice what rounding does"


def replay(session, seqs, plan):
    """Steps of ``plan``: a list of (request, number of tokens) a step; every position's logits."""
    at, steps = dict.fromkeys(seqs, 0), []
    for group in plan:
        entries, ended = [], []
        for k, n in group:
            lo, hi = at[k], min(at[k] + n, len(seqs[k]))
            entries.append({"id": k, "tokens": seqs[k][lo:hi], "want": list(range(hi - lo))})
            at[k] = hi
            if hi == len(seqs[k]):
                ended.append(k)
        steps.append({"step": len(steps), "entries": entries, "end": ended})
    assert all(at[k] == len(v) for k, v in seqs.items()), at
    return collect(session, steps)


def test_the_test_weights_make_every_mechanism_count(models, monkeypatch):
    """What the other tests rest on: the plain model's logits move by far more than the limits of the
    comparisons when any one mechanism is left out or bent."""
    folder, cfg, weights, page = models["A"]
    tokens = random_tokens(60, cfg["vocab"], 5)
    base = plain.forward(cfg, weights, tokens)

    def moved(cfg2=cfg, w2=weights, rows=slice(None)):
        other = plain.forward(cfg2, w2, tokens)
        return float((other - base)[rows].pow(2).mean().sqrt() / base[rows].pow(2).mean().sqrt())

    def scaled(factor, *ends):
        return {k: (v * factor if k.endswith(ends) else v) for k, v in weights.items()}

    def bent(path, value):
        out = copy.deepcopy(cfg)
        at = out
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        return out

    for names in (("q.b",), ("k.b",), ("mix.g",), ("norm1",), ("norm2",), ("final.norm",), ("mix.v",), ("shared.up",)):
        assert moved(w2=scaled(0.0, *names)) > 2e-2, names
    for names in (("q.norm", "k.norm"), ("l1.mix.norm",)):
        assert moved(w2={k: (v * 0 + 1 if k.endswith(names) else v) for k, v in weights.items()}) > 2e-2, names
    for path, value in ((("layers", 0, "mixer", "softcap"), 8.0), (("layers", 4, "mixer", "softcap"), 20.0),
                        (("layers", 0, "mixer", "rot", "dims"), 24), (("layers", 4, "mixer", "rot", "base"), 500.0),
                        (("layers", 0, "mixer", "rot", "scaling"), None), (("layers", 0, "mixer", "rot", "scaling", "factor"), 2.0),
                        (("layers", 0, "mixer", "rot", "scaling", "fast"), 2.0), (("layers", 2, "mixer", "scale"), 0.3),
                        (("layers", 1, "mixer", "decay", 0), 0.9), (("layers", 3, "mixer", "decay", 1), 0.97),
                        (("layers", 1, "mlp", "router", "top"), 2), (("layers", 1, "mlp", "shared"), None)):
        assert moved(bent(path, value)) > 2e-2, path

    def bend(name, fn):
        monkeypatch.setattr(plain, name, fn)
        assert moved() > 2e-2, name
        monkeypatch.undo()

    real_ff, real_rope, real_state = plain.routed_ff, plain.frequencies, plain.lightning_state

    def on_outputs(h, w, mlp):
        choice, weight = plain.route(h, w, mlp["router"]["top"])
        out = plain.expert(h, w, "shared") if mlp.get("shared") else torch.zeros_like(h)
        for t in range(h.shape[0]):
            for c in range(choice.shape[1]):
                out[t] += weight[t, c] * plain.expert(h[t: t + 1], w, f"e{int(choice[t, c])}")[0]
        return out

    bend("routed_ff", on_outputs)
    bend("frequencies", lambda rot: (real_rope(rot)[0], 1.0))
    bend("relu_squared", lambda z: torch.clamp(z, min=0.0))
    bend("lightning_state", lambda q, k, v, d: real_state(q, k, v, [0.0] * len(d)))


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts_then_single_tokens_then_portions(models, name, dtype):
    folder, cfg, weights, page = models[name]
    seqs = {"a": random_tokens(75, cfg["vocab"], 5)}
    want = {"a": oracle(name, cfg, weights, seqs["a"], dtype)}
    s = session_for(folder, dtype, page, 256)
    for plan in ([75], [40] + [1] * 35, [1] * 75, [2, 3, 2, 1, 9, 2, 17, 1, 1, 2, 30, 5], [2] * 37 + [1], [33, 42]):
        compare(replay(s, seqs, [[("a", n)] for n in plan]), want, dtype, excused=2)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_unequal_requests_side_by_side_with_slots_used_again(models, name, dtype):
    """Up to three live requests: portions of some beside single tokens of others, requests that
    pause, end and are followed by new ones in the same slots and pages (cache and states are
    poisoned when they are given back)."""
    folder, cfg, weights, page = models[name]
    V = cfg["vocab"]
    seqs = {k: random_tokens(n, V, i) for i, (k, n) in
            enumerate({"a": 61, "b": 33, "c": 9, "d": 47, "e": 2, "f": 1}.items())}
    want = {k: oracle(name, cfg, weights, v, dtype) for k, v in seqs.items()}
    s = session_for(folder, dtype, page, 192, max_num_seqs=3)
    plan = [
        [("a", 20), ("b", 2)], [("a", 1), ("b", 13), ("c", 9)], [("a", 7), ("b", 1)],
        [("b", 1), ("d", 2), ("a", 1)], [("d", 30), ("a", 1), ("b", 1)], [("a", 31)],
        [("b", 15), ("d", 1)], [("d", 14), ("e", 2)], [("f", 1)],
    ]
    compare(replay(s, seqs, plan), want, dtype, excused=3)
    # portions long enough for chunks beside single tokens and short portions
    three = {k: seqs[k] for k in "abd"}
    plan = [[("b", 20)], [("a", 50), ("b", 1), ("d", 2)], [("b", 11), ("a", 11), ("d", 1)], [("d", 44), ("b", 1)]]
    compare(replay(s, three, plan), want, dtype, excused=3)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
def test_long_decoding_through_graphs(models, dtype):
    """Some three hundred single tokens after short prompts, two requests side by side (steps of
    single tokens are captured into a graph and replayed), then one that pauses while the other goes on."""
    folder, cfg, weights, page = models["B"]
    seqs = {"a": random_tokens(330, cfg["vocab"], 7), "b": random_tokens(290, cfg["vocab"], 8)}
    want = {k: oracle("B", cfg, weights, v, dtype) for k, v in seqs.items()}
    s = session_for(folder, dtype, page, 704)
    assert s.model.graph_safe()
    plan = [[("a", 30)], [("a", 1), ("b", 10)]] + [[("a", 1), ("b", 1)]] * 240 + [[("a", 1)]] * 20 + [[("b", 1)]] * 20
    plan += [[("b", 1), ("a", 1)]] * 20 + [[("a", 19)]]
    got = replay(s, seqs, plan)
    assert s.runner.graph_replays > 200
    compare(got, want, dtype, excused=6)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_stream_after_every_layer(models, name, dtype):
    """The float32 stream itself, layer by layer, against the plain model's: a step of one whole
    prompt with a hook on the blocks."""
    folder, cfg, weights, page = models[name]
    tokens = random_tokens(40, cfg["vocab"], 21)
    layers: list = []
    plain.forward(cfg, weights, tokens, layers)
    s = session_for(folder, dtype, page, 64)
    seen = []
    for block in s.model.blocks:
        def hooked(delta, residual, ctx, call, next_block=None, inner=block.forward):
            out = inner(delta, residual, ctx, call, next_block=next_block)
            seen.append(residual[: ctx.num_tokens].double().cpu())
            return out

        block.forward = hooked
    s.run_step({"step": 0, "entries": [{"id": "a", "tokens": tokens, "want": [39]}], "end": ["a"]})
    assert len(seen) == len(layers)
    limit = 2e-5 if dtype == torch.float32 else 4e-2
    for i, got in enumerate(seen):
        per = (got - layers[i]).pow(2).mean(1).sqrt() / layers[i].pow(2).mean(1).sqrt()
        above = int((per >= limit).sum())
        assert above <= (0 if dtype == torch.float32 else 4), f"layer {i}: {above} tokens, worst {float(per.max()):.3e}"
        assert float(per.median()) < limit / 2, f"layer {i}: median {float(per.median()):.3e}"


def probe_model(tmp_path, dim, softcap, page):
    """One attention layer without a feed-forward in which one token's key outscores every other: its
    embedding alone feeds one key channel that is not rotated, and a bias puts every query on that
    channel."""
    V, H, heads, kv = 60, 32, 2, 1
    cfg = model(V, H, 1e-6, [layer(attn(heads, kv, dim, 24.0 / dim, softcap, dim // 2, 500.0), None)])
    folder = make_model_dir(tmp_path, cfg, seed=dim + page)
    from safetensors.torch import load_file, save_file

    t = load_file(str(folder / "model.safetensors"))
    channel = dim - 1
    t["embed"][:, 0] = 0
    t["embed"][V - 1] = 0
    t["embed"][V - 1, 0] = 12.0   # the marked token, never drawn otherwise
    t["l0.mix.k"][channel] = 0
    t["l0.mix.k"][channel, 0] = 8.0
    t["l0.mix.k.b"].zero_()
    t["l0.mix.q.b"].view(heads, dim)[:, channel] = 40.0
    save_file(t, str(folder / "model.safetensors"))
    cfg, weights = load_model_folder(folder)
    return folder, cfg, weights, V - 1


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("dim,softcap,page", [(64, 30.0, 16), (128, 60.0, 16), (64, None, 16), (24, 30.0, 8)])
def test_a_key_that_stands_out_far_back(tmp_path, dim, softcap, page, dtype):
    """The marked token at the start, on either side of a page's edge and inside the prompt, seen
    from 600 tokens on: in a whole prompt, in portions, and from single tokens."""
    folder, cfg, weights, marked = probe_model(tmp_path, dim, softcap, page)
    s = session_for(folder, dtype, page, 704)
    T = 640
    for place in (0, 1, page - 1, page, 333):
        tokens = [t % (marked - 1) for t in random_tokens(T, marked, place + 3)]
        without = plain.forward(cfg, weights, tokens)
        tokens[place] = marked
        want, floor = plain.forward(cfg, weights, tokens), [0.0] * T
        for pos in (place, 500, T - 1):
            assert row_error(without[pos], want[pos]) > 0.3, (place, pos)
        for plan in ([T], [place + 1, 2, T - place - 20] + [1] * 17, [300, 2, 299] + [1] * (T - 601)):
            got = replay(s, {"a": tokens}, [[("a", n)] for n in plan])
            compare(got, {"a": (want, floor)}, dtype)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("dim,vdim", [(64, 64), (20, 30)])
def test_a_state_that_stands_out_far_back(tmp_path, dim, vdim, dtype):
    """One lightning layer whose marked token writes a state a hundred times as large as the others': read
    600 tokens later, across steps, chunks, a slot used again, and from single tokens."""
    from safetensors.torch import load_file, save_file

    V = 60
    cfg = model(V, 32, 1e-6, [layer(lightning(dim, vdim, 0.9995, 0.999), None)])
    folder = make_model_dir(tmp_path, cfg, seed=dim)
    t = load_file(str(folder / "model.safetensors"))
    t["embed"][V - 1] *= 14.0
    save_file(t, str(folder / "model.safetensors"))
    cfg, weights = load_model_folder(folder)
    s = session_for(folder, dtype, 16, 704, max_num_seqs=1)
    T = 640
    for place in (0, 15, 63, 64, 333):
        tokens = [x % (V - 2) for x in random_tokens(T, V - 1, place + 3)]
        without = plain.forward(cfg, weights, tokens)
        tokens[place] = V - 1
        want, floor = plain.forward(cfg, weights, tokens), [0.0] * T
        for pos in (place, 500, T - 1):
            assert row_error(without[pos], want[pos]) > 0.15, (place, pos)
        for plan in ([T], [place + 1, 2, T - place - 20] + [1] * 17, [300, 2, 299] + [1] * (T - 601), [47, 48, 49, 63, 64, 65, 304]):
            got = replay(s, {"a": tokens}, [[("a", n)] for n in plan])
            compare(got, {"a": (want, floor)}, dtype)


@pytest.mark.parametrize("seed", list(range(12)))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Models whose every size, constant and layer order is drawn from a seed, in float32 and in
    bfloat16: two requests side by side, portions, then single tokens."""
    import random

    from tests.zikupel_helpers import random_config

    cfg = random_config(random.Random(seed))
    folder = make_model_dir(tmp_path / "drawn", cfg, seed=seed)
    c, w = load_model_folder(folder)
    seqs = {"a": random_tokens(150, cfg["vocab"], seed + 1), "b": random_tokens(70, cfg["vocab"], seed + 2)}
    plan = [[("a", 37)], [("b", 2)], [("a", 50)], [("b", 33)]] + [[("a", 1), ("b", 1)]] * 30 + [[("a", 33), ("b", 5)]]
    for dtype in DTYPES:
        want = {k: oracle(f"drawn {seed}", c, w, v, dtype) for k, v in seqs.items()}
        got = replay(session_for(folder, dtype, 16, 320, max_num_seqs=4), seqs, plan)
        assert len(got) == 220
        compare(got, want, dtype, excused=22)  # tokens whose call was close move those after them


def test_the_layers_run_the_kernels_they_are_meant_to(models):
    """In bfloat16 keys of 64 and 128 take the matrix-core kernels, in prompts and alone; single tokens need
    no kernel for norm, rotation, cap or gate; lightning layers run in chunks over a prompt and token by token
    for single tokens and short portions."""
    from kvcore_amd.ops import library as ops

    folder, cfg, weights, page = models["B"]
    s = session_for(folder, torch.bfloat16, page, 128)
    names: list = []
    watched = ("prefill_attention", "decode_attention", "paged_attention", "qk_norm_rope_kv_write", "fixed_decay_chunks",
               "linear_state_scan", "head_gate", "moe_combine", "add_rmsnorm")
    real = {n: getattr(ops, n) for n in watched}
    try:
        for n, fn in real.items():
            setattr(ops, n, lambda *a, n=n, fn=fn, **k: (names.append(n), fn(*a, **k))[1])
        tokens = random_tokens(90, cfg["vocab"], 9)

        def run(step, lo, hi, **end):
            del names[:]
            s.run_step({"step": step, "entries": [{"id": "a", "tokens": tokens[lo:hi], "want": [hi - lo - 1]}], "end": end.get("end", [])})
            return {n: names.count(n) for n in sorted(set(names))}

        assert run(0, 0, 60) == {"prefill_attention": 5, "qk_norm_rope_kv_write": 5, "fixed_decay_chunks": 2, "add_rmsnorm": 1}
        assert run(1, 60, 80) == {"prefill_attention": 5, "qk_norm_rope_kv_write": 5, "linear_state_scan": 2, "add_rmsnorm": 1}
        assert run(2, 80, 81, end=["a"]) == {"decode_attention": 5, "linear_state_scan": 2, "add_rmsnorm": 1}
    finally:
        for n, fn in real.items():
            setattr(ops, n, fn)


@pytest.mark.parametrize("dtype", DTYPES, ids=IDS)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_greedy_generation_through_the_engine(models, name, dtype):
    """``LLMEngine.generate`` with the scheduler cutting prompts into portions of 16 tokens and too few
    pages for all requests at once: every generated token is the plain model's greedy choice given the
    tokens before it (skipped where its two best logits lie closer than rounding can tell apart)."""
    from kvcore_amd import CacheConfig, KVCoreConfig, ModelConfig, SamplingParams, SchedulerConfig
    from kvcore_amd.engine.llm_engine import GenerationRequest, LLMEngine

    folder, cfg, weights, page = models[name]
    V = cfg["vocab"]
    engine = LLMEngine(KVCoreConfig(
        model_config=ModelConfig(model=str(folder), dtype="float32" if dtype == torch.float32 else "bfloat16",
                                 max_model_len=128),
        cache_config=CacheConfig(block_size=page, num_gpu_blocks=112 // page + 1),
        scheduler_config=SchedulerConfig(max_num_seqs=3, max_num_scheduled_tokens=24,
                                         long_prefill_token_threshold=16)))
    prompts = {"r0": random_tokens(37, V, 11), "r1": random_tokens(5, V, 12), "r2": random_tokens(50, V, 13),
               "r3": random_tokens(18, V, 14), "r4": random_tokens(1, V, 15)}
    params = SamplingParams(max_tokens=12, temperature=0.0)
    outs = engine.generate([GenerationRequest(k, params, prompt_token_ids=tuple(v)) for k, v in prompts.items()])
    by_id = {o.request_id: list(o.output_token_ids) for o in outs}
    assert set(by_id) == set(prompts)
    margin = 1e-4 if dtype == torch.float32 else 5e-2
    checked = wrong = 0
    for rid, prompt in prompts.items():
        gen = by_id[rid]
        assert len(gen) == 12
        logits = plain.forward(cfg, weights, prompt + gen)
        for i, tok in enumerate(gen):
            row = logits[len(prompt) + i - 1]
            top = torch.topk(row, 2).values
            if float(top[0] - top[1]) < margin * float(row.std()):
                continue
            wrong += int(torch.argmax(row)) != tok
            checked += 1
    assert checked > 40
    assert wrong == 0 if dtype == torch.float32 else wrong <= 1, f"{wrong} of {checked} tokens differ"


def test_command_lines(models, tmp_path):
    """``bin/kvcore_offline_batch`` generates with a Zikupel folder, and ``bin/trace_run`` replays
    steps on it and writes logits that match the plain model's."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    repo = Path(__file__).resolve().parent.parent
    folder, cfg, weights, page = models["A"]
    cmd = [sys.executable, str(repo / "bin" / "kvcore_offline_batch"), "--model", str(folder),
           "--dtype", "float32", "--prompt-lens", "7,16", "--max-tokens", "5", "--seed", "3",
           "--max-num-seqs", "4", "--max-num-scheduled-tokens", "32", "--num-gpu-blocks", "32",
           "--block-size", str(page), "--max-model-len", "128",
           "--ignore-eos", "--log-level", "WARNING", "--no-log-file"]
    proc = subprocess.run(cmd, capture_output=True, text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert proc.stdout.count("finish_reason=length") == 2
    tokens = random_tokens(21, cfg["vocab"], 17)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": tokens[:13], "want": [0, 12]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": tokens[13:15], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": tokens[15:], "want": [5]}], "end": ["x"]}]
    out_dir = tmp_path / "logits"
    cmd = [str(repo / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32", "--out", str(out_dir),
           "--max-tokens", "64", "--block-size", str(page)]
    proc = subprocess.run(cmd, input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True,
                          text=True, timeout=110)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not (out_dir / "1.f32").exists()
    want = {"x": oracle("A", cfg, weights, tokens, torch.float32)}
    first = np.fromfile(out_dir / "0.f32", dtype="<f4").reshape(2, -1)
    last = np.fromfile(out_dir / "2.f32", dtype="<f4").reshape(1, -1)
    compare({("x", 0): torch.from_numpy(first[0]).double(), ("x", 12): torch.from_numpy(first[1]).double(),
             ("x", 20): torch.from_numpy(last[0]).double()}, want, torch.float32)
