"""The sequence engine on small random Zusuvik models against oracle/zusuvik.py: whole prompts with the stream after every layer run,
decoding through the caches and the recurrent states (a set per pass of the looped layers), portions, mixed batches, reuse of pages and
slots, the first tokens, a far token that decides the logits pages later, long decoding, generation through the scheduler, graph replays."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import zusuvik as oz
from tests.seq_helpers import make_engine, rel_err, rows_close, run_portions, run_whole

pytestmark = pytest.mark.gpu

CONFIGS = {
    # both kinds of layer with and without a feed-forward, a loop over two layers in the middle
    "looped": dict(layers=[("retention", None, {}), ("parallel", None, {}), ("retention", {"heads": 2, "vdim": 12}, None), ("parallel", {"left": {"conv": 2}}, {})],
                   loop=(1, 3, 3)),
    # sizes that are no multiples of 4 or 8, one head, one key/value head, one tap, the whole head rotated, every expert chosen, no shared
    # expert, weights and scales of one, the loop covers the whole model
    "odd": dict(width=50, vocab=61, eps=1e-3, logit_scale=1.0, loop=(0, 2, 2),
                layers=[("parallel", {"left": dict(heads=1, kv_heads=1, dim=10, vdim=7, conv=1, rot_dims=10, scaling=None, scale=0.5, softcap=2.0),
                                      "right": dict(heads=1, dim=5, vdim=9, gate_cap=3.0), "scales": (1.0, 1.0)}, dict(experts=3, top=3, ff=10, shared=0)),
                        ("retention", dict(heads=1, dim=6, vdim=7, rot_dims=6, decay=[0.75]), dict(experts=2, top=1, ff=6, shared=9))]),
    # sizes of the matrix-core tiles, as many key/value heads as query heads, no loop, more experts than a wave's lanes
    "tiles": dict(width=64, vocab=130, logit_scale=0.125,
                  layers=[("parallel", {"left": dict(heads=4, kv_heads=4, dim=32, vdim=64, conv=4, rot_dims=16, softcap=30.0),
                                        "right": dict(heads=2, dim=64, vdim=64, gate_cap=15.0), "scales": (0.5, 0.25)}, dict(experts=70, top=4, ff=16, shared=32)),
                          ("retention", dict(heads=4, dim=32, vdim=128, rot_dims=32, base=1e5), dict(experts=8, top=2, ff=32, shared=64)),
                          ("parallel", {"left": dict(heads=8, kv_heads=2, dim=16, vdim=32, conv=5, rot_dims=4, scaling=None),
                                        "right": dict(heads=4, dim=16, vdim=32)}, None)]),
    # one pass only; a decay of one; the last layers looped
    "once": dict(width=52, layers=[("retention", dict(decay=[1.0, 0.5, 0.99]), {}), ("parallel", {"scales": (1.5, -0.5)}, dict(top=1))], loop=(1, 2, 1)),
}

# rows of a 16-bit engine that must lie within the tolerance: a rounding can tip a narrow choice of experts, which swaps the
# feed-forward output of that row (and, weakly, of the rows that read it)
SHARE = {"odd": 0.75, "once": 0.8, "tiles": 0.85}


def model(name, seed=0):
    rng = np.random.default_rng(seed)
    cfg, t = oz.random_zusuvik(rng, **CONFIGS[name])
    return cfg, t, rng


@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_f32_and_bf16(name):
    cfg, t, rng = model(name)
    tokens = rng.integers(0, cfg["vocab"], 150).tolist()
    streams = []
    want = oz.forward(cfg, t, tokens, streams)
    assert len(streams) == len(oz.layer_order(cfg))
    eng = make_engine(cfg, t, torch.float32)
    taps = {}
    got = eng.step([("a", tokens, list(range(len(tokens))))], taps=taps).cpu().numpy()
    for i, s in enumerate(streams):
        assert rel_err(taps[i].cpu().numpy(), s) < 2e-5, f"layer run {i}"
    assert rel_err(got, want) < 5e-5
    eng.release("a")
    assert rel_err(run_whole(eng, "b", tokens), got) < 1e-6                  # without the taps the residual steps run fused
    eng16 = make_engine(cfg, t, torch.bfloat16)
    assert rows_close(run_whole(eng16, "a", tokens), want, 0.08, SHARE.get(name, 0.95))


@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_against_token_by_token_decoding(name):
    cfg, t, rng = model(name, 1)
    tokens = rng.integers(0, cfg["vocab"], 200).tolist()
    want = oz.forward(cfg, t, tokens)
    eng = make_engine(cfg, t, torch.float32)
    whole = run_whole(eng, "w", tokens)                        # the recurrences run in chunks side by side
    dec = run_portions(eng, "d", tokens, [1])
    assert rel_err(whole, want) < 5e-5 and rel_err(dec, want) < 5e-5
    mixed = run_portions(eng, "m", tokens, [70, 1])           # a prompt, then its last tokens one by one
    assert rel_err(mixed, dec) < 2e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    w16 = run_whole(eng16, "w", tokens)
    d16 = run_portions(eng16, "d", tokens, [120, 1])          # decode steps replay graphs; the key walks are split
    assert rows_close(d16, w16, 0.04, SHARE.get(name, 0.95)) and rows_close(d16, want, 0.08, SHARE.get(name, 0.95))


@pytest.mark.parametrize("sizes", [[2], [3, 2, 64, 1, 5, 63, 2], [64], [65, 2, 2, 1, 127], [1, 2, 128, 2], [130, 2], [31, 32, 33, 2]])
def test_portions_of_any_size(sizes):
    cfg, t, rng = model("looped", 2)
    tokens = rng.integers(0, cfg["vocab"], 201).tolist()
    eng = make_engine(cfg, t, torch.float32)
    whole = run_whole(eng, "w", tokens)
    assert rel_err(run_portions(eng, "p", tokens, sizes), whole) < 2e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    w16 = run_whole(eng16, "w", tokens)
    assert rows_close(run_portions(eng16, "p", tokens, sizes), w16, 0.04)


@pytest.mark.parametrize("name", ["looped", "tiles"])
def test_batches_of_unequal_requests_against_each_alone(name):
    cfg, t, rng = model(name, 3)
    lens = [1, 23, 97, 190]
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in lens]
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, None)):
        eng = make_engine(cfg, t, dtype, max_tokens=1024)
        alone = [run_whole(eng, ("a", i), tk) for i, tk in enumerate(toks)]
        got, at = [[] for _ in toks], [0] * len(toks)
        for step in [[20, 20, 20, 20], [0, 1, 40, 2], [0, 1, 1, 64], [0, 1, 36, 1], [0, 0, 0, 103]]:
            ent, who = [], []
            for i, n in enumerate(step):
                n = min(n, lens[i] - at[i])
                if n > 0:
                    ent.append((("b", i), toks[i][at[i]:at[i] + n], list(range(n))))
                    who.append((i, n))
            out, o = eng.step(ent).cpu().numpy(), 0
            for i, n in who:
                got[i].append(out[o:o + n])
                o, at[i] = o + n, at[i] + n
        for i in range(len(toks)):
            assert at[i] == lens[i]
            if tol is None:
                assert rows_close(np.concatenate(got[i]), alone[i], 0.04, SHARE.get(name, 0.95)), f"request {i}"
            else:
                assert rel_err(np.concatenate(got[i]), alone[i]) < tol, f"request {i}"


def test_pages_and_slots_that_are_freed_and_used_again():
    cfg, t, rng = model("looped", 4)
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in (150, 100, 120, 64, 30)]
    fresh = [run_whole(make_engine(cfg, t, torch.float32, max_tokens=256, max_slots=2), "f", tk) for tk in toks]
    eng = make_engine(cfg, t, torch.float32, max_tokens=320, max_slots=2)      # 5 pages, 2 slots
    assert eng.state.num_pages == 5
    a = run_portions(eng, "a", toks[0], [64, 1, 85])                           # 3 pages, released
    assert eng.state.used_pages() == 0
    b = eng.step([("b", toks[1][:90], list(range(90))), ("c", toks[2][:40], list(range(40)))]).cpu().numpy()
    b2 = eng.step([("b", toks[1][90:], list(range(10))), ("c", toks[2][40:], list(range(80)))]).cpu().numpy()
    assert eng.state.used_pages() == 4
    with pytest.raises(RuntimeError):
        eng.step([("d", toks[3], [])])                                         # no slot left
    eng.release("b")
    d = eng.step([("d", toks[3], list(range(64))), ("c", [], [])]).cpu().numpy()   # b's slot (states, convolution tails) and pages, dirty from b
    eng.release("c")
    e = run_whole(eng, "e", toks[4])
    eng.release("d")
    assert eng.state.used_pages() == 0 and len(eng.state.free_slots) == 2
    assert rel_err(a, fresh[0]) < 2e-5 and rel_err(np.concatenate([b[:90], b2[:10]]), fresh[1]) < 2e-5
    assert rel_err(np.concatenate([b[90:], b2[10:]]), fresh[2]) < 2e-5
    assert rel_err(d, fresh[3]) < 2e-5 and rel_err(e, fresh[4]) < 2e-5


def test_the_first_tokens_of_a_sequence():
    cfg, t, rng = model("tiles", 5)
    tokens = rng.integers(0, cfg["vocab"], 6).tolist()
    want = oz.forward(cfg, t, tokens)
    for dtype, tol in ((torch.float32, 5e-5), (torch.bfloat16, 0.08)):
        eng = make_engine(cfg, t, dtype)
        assert rel_err(run_whole(eng, "a", tokens[:1]), want[:1]) < tol      # one key, empty states, a convolution over zeros
        got = run_portions(eng, "b", tokens, [1, 2, 3])
        assert rel_err(got, want) < tol if dtype == torch.float32 else rows_close(got, want, tol, 0.8)
    second = run_whole(eng, "c", tokens[1:2])
    assert rel_err(got[1:2], second) > 1e-3                                  # a token at position 1 is not that token at position 0


def test_every_pass_of_the_loop_has_its_own_cache_and_state():
    """an oracle whose passes shared one state would differ from the second token on; here the passes' caches are shown to differ"""
    cfg, t, rng = model("looped", 9)
    eng = make_engine(cfg, t, torch.float32)
    tokens = rng.integers(0, cfg["vocab"], 40).tolist()
    eng.step([("a", tokens, [])])
    s = eng.state.live["a"]
    k = [eng.state.tables[f"l1.attn.run{r}.k"].rows(s.index, s.pages, 40).float().cpu().numpy() for r in range(3)]
    assert rel_err(k[0], k[1]) > 0.01 and rel_err(k[1], k[2]) > 0.01
    for name in ("l1.memory.run{}.S", "l1.memory.run{}.n", "l1.attn.run{}.tail", "l2.retention.run{}.S"):
        a, b = (eng.state.states[name.format(r)][s.index].cpu().numpy() for r in (0, 2))
        assert np.abs(a).max() > 0 and rel_err(a, b) > 0.01, name


def test_far_tokens_decide_the_logits_pages_later():
    """sharp scores and slow decays: the logits of the last rows change visibly when tokens more than 230 positions (three pages and more)
    back are others"""
    rng = np.random.default_rng(8)
    cfg, t = oz.random_zusuvik(rng, [("parallel", {"left": {"scale": 1.5, "softcap": 25.0}}, None), ("retention", dict(decay=[0.999, 0.9995, 0.998]), {})],
                               loop=(0, 2, 2))
    a = [int(x) for x in rng.integers(0, cfg["vocab"], 330)]
    b = [int(x) for x in rng.integers(0, cfg["vocab"], 100)] + a[100:]
    wa, wb = oz.forward(cfg, t, a)[-20:], oz.forward(cfg, t, b)[-20:]
    assert rel_err(wa, wb) > 1e-2
    eng = make_engine(cfg, t, torch.float32)
    ga = run_portions(eng, "a", a, [310, 1])[-20:]                            # the last 20 tokens decoded alone, 5 pages on
    gb = run_portions(eng, "b", b, [2, 150, 158, 1])[-20:]
    assert rel_err(ga, wa) < 5e-5 and rel_err(gb, wb) < 5e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    assert rows_close(run_portions(eng16, "a", a, [310, 1])[-20:], wa, 0.08, 0.8)


def test_long_decoding():
    cfg, t, rng = model("looped", 10)
    tokens = rng.integers(0, cfg["vocab"], 170).tolist()
    want = oz.forward(cfg, t, tokens)
    eng16 = make_engine(cfg, t, torch.bfloat16)
    assert rows_close(run_portions(eng16, "d", tokens, [10, 1]), want, 0.08)
    eng = make_engine(cfg, t, torch.float32)
    assert rel_err(run_portions(eng, "d", tokens, [10, 1]), want) < 5e-5


def test_greedy_generation_through_the_scheduler():
    cfg, t, rng = model("looped", 6)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (5, 41, 18)]
    new = 12
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(new):
            seq.append(int(np.argmax(oz.forward(cfg, t, seq)[-1])))
        want.append(seq[len(p):])
    eng = make_engine(cfg, t, torch.float32, max_tokens=192, max_slots=2)      # the third prompt waits for a slot
    got = eng.generate(prompts, max_new_tokens=new, token_budget=24, max_chunk=16)
    assert got == want
    assert eng.state.used_pages() == 0 and not eng.state.live
    sampled = eng.generate(prompts[:2], max_new_tokens=4, sampling={"top_k": 5, "top_p": 0.9, "temperature": 0.8, "seed": 3})
    assert all(len(s) == 4 and all(0 <= x < cfg["vocab"] for x in s) for s in sampled)


def test_decode_steps_replayed_as_graphs_equal_eager_steps(monkeypatch):
    cfg, t, rng = model("tiles", 7)
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in (90, 150, 40)]
    def run(eng):
        out = []
        eng.step([("a", toks[0][:50], []), ("b", toks[1][:100], [])])
        for i in range(25):
            out.append(eng.step([("a", [toks[0][50 + i]], [0]), ("b", [toks[1][100 + i]], [0])]).cpu().numpy().copy())
            if i == 10:
                torch.cuda.synchronize()
                eng.step([("c", toks[2][:30], [])])      # a prompt's portion between two replays
        for i in range(10):
            out.append(eng.step([("a", [toks[0][75 + i]], [0]), ("b", [toks[1][125 + i]], [0]), ("c", [toks[2][30 + i]], [0])]).cpu().numpy().copy())
        return out
    graphed = make_engine(cfg, t, torch.bfloat16)
    assert graphed.use_graphs
    got = run(graphed)
    assert any(g["graph"] is not None for g in graphed._graphs.values())
    monkeypatch.setenv("DIHIP_SEQ_GRAPH", "0")
    eager = make_engine(cfg, t, torch.bfloat16)
    assert not eager.use_graphs
    for a, b in zip(got, run(eager)):
        assert np.array_equal(a, b)


def test_a_checkpoint_folder_through_the_reader_and_the_trace_runner(tmp_path):
    """config.json + model.safetensors on disk: the engine's own loader, and bin/trace_run on the same folder"""
    from safetensors.torch import save_file

    cfg, t, rng = model("odd", 11)
    folder = tmp_path / "model"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: torch.from_numpy(np.ascontiguousarray(v)).to(torch.bfloat16) for k, v in t.items()}, str(folder / "model.safetensors"))
    tokens = rng.integers(0, cfg["vocab"], 70).tolist()
    want = oz.forward(cfg, t, tokens)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:66], "want": [0, 65]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[66:69], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": tokens[69:], "want": [0]}], "end": ["a"]}]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(folder), "--dtype", "float32", "--out", str(out), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    read = lambda i: np.fromfile(out / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
    assert not (out / "1.f32").exists()
    assert rel_err(read(0), want[[0, 65]]) < 5e-5 and rel_err(read(2), want[69:]) < 5e-5
