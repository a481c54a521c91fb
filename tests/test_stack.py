"""Decoders through the layer-by-layer engine (tah_amd.stack) against their plain oracles: prompts, portions, decoding, batches,
slots used again, generation through the shared loop, loading through the registry, the trace runner."""
import io
import json
import os

import pytest
import torch

from tests import emu_util
from tests import stack_cases as Z

BF = torch.bfloat16
needs_clang = pytest.mark.skipif(not emu_util.have_host_clang(), reason="host clang++ not available")
BOTH = pytest.mark.parametrize("dtype", ["f32", "bf16"])
CONFIGS = Z.CONFIGS
MODELS = pytest.mark.parametrize("which", sorted(CONFIGS))


def setup(which, dtype, dev, batch, max_len):
    from tah_amd.stack import StackEngine
    cfg = CONFIGS[which] if dtype == "f32" else Z.without_close_calls(CONFIGS[which])
    t = Z.tensors_for(cfg, sharp=2.0 if dtype == "f32" else 1.0)  # (peaked attention magnifies bf16's roundings)
    return cfg, t, StackEngine(Z.load(cfg, t, Z.DTYPES[dtype], dev), batch, max_len, device=dev), Z.Check(cfg, t, Z.DTYPES[dtype])


# ── no device ────────────────────────────────────────────────────────────────────────────────────────────────────────
@MODELS
def test_faults_would_show(which):
    """Window edges, and a state lost half-way, are far outside the float32 tolerance with these weights."""
    cfg = CONFIGS[which]
    Z.wrong_oracles_differ(cfg, Z.tensors_for(cfg), Z.tokens_of(cfg, 100, 1))


def test_checkpoint_reader_and_registry(tmp_path):
    from tah_amd import TahDuoError, checkpoint, registry
    t = {"a": torch.randn(3, 5).to(BF), "b.c": torch.arange(7, dtype=torch.int32), "odd": torch.tensor([1, 2, 3], dtype=torch.uint8),
         "f": torch.randn(2, 2), "empty": torch.zeros(0, 4)}
    checkpoint.write_safetensors(str(tmp_path / "model.safetensors"), t)
    got = checkpoint.read_tensors(str(tmp_path))
    assert set(got) == set(t) and all(torch.equal(got[k], t[k]) and got[k].dtype == t[k].dtype for k in t)
    safetensors = pytest.importorskip("safetensors.torch")
    assert all(torch.equal(v, t[k]) for k, v in safetensors.load_file(str(tmp_path / "model.safetensors")).items())
    with open(tmp_path / "model.safetensors", "r+b") as f:
        f.truncate(os.path.getsize(tmp_path / "model.safetensors") - 3)
    with pytest.raises(TahDuoError):
        checkpoint.read_tensors(str(tmp_path))
    assert {"Zedudra", "Zozosun", "Qwen3ForCausalLM"} <= set(registry.architectures())
    assert registry.of_config({"architecture": "Zozosun"}).name == "Zozosun"
    assert registry.of_config({"architectures": ["Qwen3ForCausalLM"]}).name == "Qwen3ForCausalLM"
    with pytest.raises(TahDuoError):
        registry.of_config({"architecture": "nothing"})
    for cfg in CONFIGS.values():
        assert registry.of_config(cfg).load is Z.design(cfg).load
        with pytest.raises(TahDuoError):
            Z.design(cfg).shapes(dict(cfg, layers=[dict(cfg["layers"][0], type="other")]))


def test_shared_weights_and_sizes_that_do_not_go_together():
    """Layers on another layer's weights bring no tensors, and are the same layer; sizes are checked where weights are read."""
    import copy

    from tah_amd import TahDuoError, zedudra
    cfg = CONFIGS["zedudra odd"]
    t = Z.tensors_for(cfg)
    assert {n.split(".")[0] for n in t if n[0] == "l"} == {"l0", "l1", "l3"}
    m = Z.load(cfg, t, torch.float32, "cpu")
    assert m.layers[2] is m.layers[0] and m.layers[4] is m.layers[1] and m.layers[3] is not m.layers[1]

    def broken(f):
        c = copy.deepcopy(cfg)
        f(c)
        with pytest.raises(TahDuoError):
            Z.load(c, t, torch.float32, "cpu")
    broken(lambda c: c["canon"].update(taps=4))
    broken(lambda c: c["norm"].update(groups=5))
    broken(lambda c: c["layers"][0]["mixer"].update(vdim=8))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4))
    broken(lambda c: c["layers"][2].update(weights_of=2))
    broken(lambda c: c["layers"][2].update(weights_of=9))
    chain = copy.deepcopy(cfg)
    chain["layers"].append(dict(chain["layers"][4], weights_of=4))
    assert zedudra.shapes(chain) == zedudra.shapes(cfg)
    assert len({id(l) for l in Z.load(chain, t, torch.float32, "cpu").layers}) == 3


def test_slot_pool():
    from tah_amd import TahDuoError
    from tah_amd.kv_cache import SlotPool
    p = SlotPool(2, 10)
    a, b = p.alloc(), p.alloc()
    with pytest.raises(TahDuoError):
        p.alloc()
    assert p.grow(a, 4) == 0 and p.grow(a, 6) == 4 and p.grow(b, 1) == 0
    with pytest.raises(TahDuoError):
        p.grow(a, 1)
    p.release(a)
    with pytest.raises(TahDuoError):
        p.release(a)
    assert p.alloc() == a and p.grow(a, 3) == 0


def test_registry_loads_a_qwen3_checkpoint(tmp_path):
    """The engine's older architecture through the same door: tensors by name into the fused layout."""
    from tah_amd import checkpoint, registry
    c = {"architectures": ["Qwen3ForCausalLM"], "hidden_size": 64, "num_hidden_layers": 2, "num_attention_heads": 2, "num_key_value_heads": 1,
         "head_dim": 128, "intermediate_size": 96, "vocab_size": 40, "rms_norm_eps": 1e-6, "rope_theta": 1e6}
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g).to(BF)
    t = {"model.embed_tokens.weight": r(40, 64), "model.norm.weight": r(64)}
    for i in range(2):
        p = f"model.layers.{i}."
        t.update({p + "input_layernorm.weight": r(64), p + "post_attention_layernorm.weight": r(64), p + "self_attn.q_proj.weight": r(256, 64),
                  p + "self_attn.k_proj.weight": r(128, 64), p + "self_attn.v_proj.weight": r(128, 64), p + "self_attn.q_norm.weight": r(128),
                  p + "self_attn.k_norm.weight": r(128), p + "self_attn.o_proj.weight": r(64, 256), p + "mlp.gate_proj.weight": r(96, 64),
                  p + "mlp.up_proj.weight": r(96, 64), p + "mlp.down_proj.weight": r(64, 96)})
    (tmp_path / "config.json").write_text(json.dumps(c))
    checkpoint.write_safetensors(str(tmp_path / "model.safetensors"), t)
    arch, w = registry.load_weights(str(tmp_path), "cpu")
    assert arch.name == "Qwen3ForCausalLM" and w.cfg.hq == 2 and w.cfg.layers == 2 and w.lm_head is w.embed
    assert torch.equal(w.layers[1]["wqkv"][256:384], t["model.layers.1.self_attn.k_proj.weight"])
    assert torch.equal(w.layers[0]["wgu"][96:], t["model.layers.0.mlp.up_proj.weight"])


# ── one engine case for both devices ─────────────────────────────────────────────────────────────────────────────────
def sequence_case(which, dtype, dev, n, all_cuts, max_len=None):
    cfg, t, eng, check = setup(which, dtype, dev, 2, max_len or n)
    tokens = Z.tokens_of(cfg, n, 3)
    for cuts in all_cuts:  # (slots are given back and taken again between the runs)
        Z.run_cut(eng, check, tokens, cuts, f"{which} {dtype}")


@needs_clang
@BOTH
@pytest.mark.parametrize("which", ["zozosun odd", "zedudra odd"])
def test_portions_and_decoding_on_cpu_shim(which, dtype):
    with emu_util.emulated():
        if which.startswith("zozosun"):
            sequence_case(which, dtype, "cpu", 13, [(7, 2, 2)])
        else:
            sequence_case(which, dtype, "cpu", 7, [(4, 2)])


# ── GPU ──────────────────────────────────────────────────────────────────────────────────────────────────────────────
@pytest.mark.gpu
@MODELS
@BOTH
def test_prompt_against_portions_against_decoding_gpu(which, dtype):
    """The same sequence whole, token by token, and in portions of several sizes, two tokens among them: every position."""
    n = 100
    sequence_case(which, dtype, "cuda", n, [(n,), (), (2,) * 30, (37, 2, 3, 40), (64, 33), (5, 11, 9, 30, 2)])


@pytest.mark.gpu
@MODELS
@BOTH
def test_long_decoding_gpu(which, dtype):
    """Several windows' and rings' lengths decoded token by token behind a short prompt."""
    sequence_case(which, dtype, "cuda", 240, [(3,)])


@pytest.mark.gpu
@MODELS
@BOTH
def test_batches_of_unequal_requests_and_slots_used_again_gpu(which, dtype):
    """Requests of different lengths start, continue in portions or single tokens, and end at different times, all in the same
    calls; each position's logits are those of the request alone.  Slots change owners on the way."""
    cfg, t, eng, check = setup(which, dtype, "cuda", 3, 120)
    reqs = [Z.tokens_of(cfg, n, 10 + i) for i, n in enumerate((90, 9, 41, 1, 60, 25, 2))]
    waiting, live, step = list(range(len(reqs))), {}, 0
    while waiting or live:
        while waiting and len(live) < 3:
            live[waiting.pop(0)] = [eng.alloc(), 0]
        entries, places = [], []
        for j, r in enumerate(sorted(live)):
            s, at = live[r]
            n = min((1, 7, 2, 1, 23, 1, 3, 16)[(step + 3 * j) % 8], len(reqs[r]) - at)
            entries.append((s, reqs[r][at:at + n]))
            places.append((r, at, n))
        lg = eng.extend(entries)
        k = 0
        for r, at, n in places:
            check(lg[k:k + n], reqs[r], range(at, at + n), f"{which} request {r} at {at}")
            k += n
            live[r][1] += n
            if live[r][1] == len(reqs[r]):
                eng.release(live.pop(r)[0])
        step += 1


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("which", ["zozosun odd", "zedudra odd"])
def test_wanted_rows_and_refusals_gpu(which, dtype):
    from tah_amd import TahDuoError
    cfg, t, eng, check = setup(which, dtype, "cuda", 2, 20)
    a, b = eng.alloc(), eng.alloc()
    ta, tb = Z.tokens_of(cfg, 12, 5), Z.tokens_of(cfg, 9, 6)
    lg = eng.extend([(a, ta), (b, tb)], want=[[11, 2], []])
    assert lg.shape == (2, cfg["vocab"])
    check(lg[:1], ta, [11], "wanted")
    check(lg[1:], ta, [2], "wanted")
    assert eng.extend([(b, [3])], want=[[]]).shape == (0, cfg["vocab"])
    for bad in ([(a, [1] * 9)], [(a, [1]), (a, [2])], [(5, [1])], [(a, [])]):
        with pytest.raises(TahDuoError):
            eng.extend(bad)
    check(eng.extend([(a, [ta[0]])]), ta + [ta[0]], [12], "after refusals")


def oracle_greedy(cfg, t, prompt, n, eos=-1):
    """Greedy tokens and the smallest gap between the two largest logits on the way."""
    seq, gap = list(prompt), float("inf")
    for _ in range(n):
        z = Z.oracle(cfg).forward(cfg, t, seq)[-1]
        top = z.topk(2).values
        gap = min(gap, float((top[0] - top[1]) / z.pow(2).mean().sqrt()))
        seq.append(int(z.argmax()))
    return seq[len(prompt):], gap


@pytest.mark.gpu
@MODELS
def test_greedy_generation_gpu(which):
    """Prefill and the shared generation loop, float32: the oracle's greedy tokens, eager and from the captured step, with more
    than one prompt length; and through ``generate`` with a tokenizer."""
    from tah_amd.engine import generate
    cfg, t, eng, check = setup(which, "f32", "cuda", 3, 60)
    prompts = [Z.tokens_of(cfg, n, 30 + n) for n in (17, 2, 30)]
    t64 = {k: v.double() for k, v in t.items()}
    want, gaps = zip(*(oracle_greedy(cfg, t64, p, 12) for p in prompts))
    assert min(gaps) > 3e-4, "the case has a near tie: choose other prompts"
    ids = torch.tensor(sum(prompts, [])).cuda()
    cu = torch.tensor([0, 17, 19, 49], dtype=torch.int32).cuda()
    for graph in (False, True):
        for portion in (None, 7):
            first, _ = eng.prefill(ids, cu, portion=portion)
            for b, p in enumerate(prompts):
                check(first[b:b + 1], p, [len(p) - 1], "prefill")
            got = eng.generate(first, 12, use_graph=graph)
            assert got.tolist() == [list(w) for w in want]
    # the slots go on from where the generation left them
    lg = eng.extend([(1, [want[1][-1]])])
    check(lg, prompts[1] + list(want[1]), [2 + 11], "after a generation")

    class Tokenizer:
        eos_token_id = int(want[0][5])
        decode = staticmethod(lambda ids: " ".join(map(str, ids)))
    T = 30
    inp = torch.tensor([[0] * (T - len(p)) + p for p in prompts])
    mask = torch.tensor([[0] * (T - len(p)) + [1] * len(p) for p in prompts])
    out, text = generate(eng, Tokenizer, {"input_ids": inp, "attention_mask": mask}, max_new_tokens=12, do_sample=False)
    for b in range(3):
        w = list(want[b])
        w = w[:w.index(Tokenizer.eos_token_id)] if Tokenizer.eos_token_id in w else w
        assert out[b] == w and text[b] == " ".join(map(str, w))


@pytest.mark.gpu
@MODELS
def test_captured_generation_equals_eager_steps_gpu(which):
    """bf16: the captured step replayed per token gives the tokens of eager single-token calls, and more rows than one pass
    takes run in groups; sampling draws from the same engine."""
    cfg, t, eng, check = setup(which, "bf16", "cuda", 37, 48)
    prompts = [Z.tokens_of(cfg, 1 + i % 9, 50 + i) for i in range(37)]
    cu = torch.tensor([0] + torch.tensor([len(p) for p in prompts]).cumsum(0).tolist(), dtype=torch.int32).cuda()
    ids = torch.tensor(sum(prompts, [])).cuda()
    got = {}
    for graph in (True, False):
        first, _ = eng.prefill(ids, cu)
        got[graph] = eng.generate(first, 20, use_graph=graph).clone()
        torch.cuda.synchronize()
    assert bool((got[True] == got[False]).all())
    first, _ = eng.prefill(ids, cu)
    tok, want = first.argmax(-1), []
    for i in range(20):
        want.append(tok.clone())
        lg = eng.extend([(b, [int(x)]) for b, x in enumerate(tok.tolist())]) if i < 19 else None
        if lg is not None:
            for b in (0, 8, 31, 36):
                check(lg[b:b + 1], prompts[b] + [int(w[b]) for w in want], [len(prompts[b]) + i], "decoding in a batch")
            tok = lg.float().argmax(-1)
    assert bool((got[True] == torch.stack(want, 1)).all())
    first, _ = eng.prefill(ids, cu)
    drawn = eng.generate(first, 6, temperature=0.8, top_p=0.9)
    assert drawn.shape == (37, 6) and int(drawn.min()) >= 0 and int(drawn.max()) < cfg["vocab"]


@pytest.mark.gpu
@BOTH
@pytest.mark.parametrize("which", ["zozosun odd", "zedudra odd", "zedudra even"])
def test_trace_runner_gpu(which, dtype, tmp_path):
    """A checkpoint folder through the command's main: portions, single tokens, requests that end, wanted rows."""
    from tah_amd import checkpoint, trace
    cfg = CONFIGS[which] if dtype == "f32" else Z.without_close_calls(CONFIGS[which])
    t = Z.tensors_for(cfg, sharp=2.0 if dtype == "f32" else 1.0)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    checkpoint.write_safetensors(str(tmp_path / "model.safetensors"), t)
    check = Z.Check(cfg, t, Z.DTYPES[dtype])
    a, b = Z.tokens_of(cfg, 30, 7), Z.tokens_of(cfg, 4, 8)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:29], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[29:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [1, 3]}], "end": ["b"]}]
    out = io.StringIO()
    args = ["--model", str(tmp_path), "--dtype", {"f32": "float32", "bf16": "bfloat16"}[dtype], "--out", str(tmp_path), "--max-tokens", "30"]
    assert trace.main(args, io.StringIO("\n".join(map(json.dumps, steps)) + "\n"), out) == 0
    assert out.getvalue().split("\n")[:4] == [f"done {i}" for i in range(4)]
    read = lambda i: torch.frombuffer(bytearray((tmp_path / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
    check(read(0), a, [0, 19], "step 0")
    check(read(2), a, [29], "step 2")
    check(read(3), b, [1, 3], "step 3")
    assert not (tmp_path / "1.f32").exists()


def test_trace_runner_refuses_a_format_the_model_does_not_run_in(tmp_path):
    from tah_amd import trace
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["Qwen3ForCausalLM"]}))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "4"], io.StringIO(""), io.StringIO()) == 3
