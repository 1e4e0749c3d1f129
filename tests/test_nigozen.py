"""Nigozen (a layer norm before and after each sublayer, chunked attention with one added to the softmax denominator,
interleaved rotation of the leading dims, values blended with the first such layer's, a sigmoid output gate, dense
GELU and routed squared-ReLU feed-forwards without gates, scaled embedding rows, tied logits) in the engine, against
the plain implementation of tests/nigozen_oracle.py.

Small configurations with random weights are written to a temporary folder (config.json +
model.safetensors) and run through ``LLMEngine.replay_step`` / ``add_request`` on the CPU device
(unfused torch forms of the ops) and, marked ``gpu``, on the HIP kernels, in fp32 and bf16.
"""
from __future__ import annotations

import json
import math

import pytest
import torch

import nigozen_oracle as oracle

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]


# ------------------------------------------------------------------------------------ configurations
def _dense(n):
    return {"kind": "dense", "ff": n}


def _moe(experts, top, n):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": n}}


def _att(H, G, D, V, dims, base, size, mix, mlp, scale=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": scale or 0.6 / math.sqrt(D), "v_mix": mix,
                      "rot": {"base": base, "dims": dims}, "mask": {"size": size}}}


def _model(width, vocab, layers, scale, eps=1e-5):
    return {"architecture": "Nigozen", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


def config_a():
    """Unequal everything: sizes that are no multiple of 8 (the fp32-FMA attention kernel in bf16 too), key size !=
    value size, grouped key/value heads, chunks shorter than a page, layers that mix no values before and between
    those that do, a layer without feed-forward, one without rotation, a vocabulary that is no multiple of 4, head
    counts that differ among the mixing layers (the same kv_heads * vdim)."""
    return _model(42, 50, [
        _att(3, 1, 6, 7, 4, 100.0, 9, False, _dense(26)),
        _att(4, 2, 10, 6, 6, 50.0, 5, True, _moe(5, 2, 13)),
        _att(4, 2, 6, 10, 0, 10.0, 21, False, None),
        _att(6, 3, 7, 4, 2, 1000.0, 19, True, _moe(3, 3, 10)),
        _att(2, 2, 12, 6, 12, 10.0, 30, True, _dense(20))], 1.6)


def config_b():
    """Values that are 1 or equal: one head, chunks of a single token in one layer, one expert, every dim rotated, an
    embedding scale of exactly 1, a single layer that mixes values (so nothing is mixed)."""
    return _model(24, 32, [
        _att(1, 1, 4, 4, 4, 10.0, 1, False, _moe(1, 1, 8)),
        _att(1, 1, 4, 4, 4, 10.0, 32, True, _dense(8))], 1.0, eps=1e-6)


def config_c():
    """Page-scale geometry on the MFMA kernels' sizes: chunks that end inside a page, at page borders (one and three
    pages) and one past a border; as many key/value heads as heads, and fewer; a head wider than 64."""
    return _model(64, 96, [
        _att(4, 2, 16, 32, 8, 10000.0, 37, True, _dense(48)),
        _att(2, 2, 24, 32, 24, 500.0, 16, True, _moe(6, 2, 24)),
        _att(4, 1, 8, 64, 4, 100.0, 48, True, _moe(4, 1, 40)),
        _att(2, 2, 72, 32, 16, 10000.0, 17, True, None)], 0.7, eps=1e-6)


def config_d():
    """Sizes in the range the fragment-packed MFMA GEMMs take (width 512, projections in multiples of 64)."""
    return _model(512, 704, [
        _att(8, 2, 64, 64, 32, 10000.0, 33, True, _dense(1024)),
        _att(4, 4, 32, 32, 32, 10000.0, 24, True, _moe(8, 3, 192)),
        _att(8, 2, 64, 64, 32, 10000.0, 33, True, _moe(8, 2, 128))], 2.5, eps=1e-6)


def config_one():
    """A single layer without feed-forward: what a position's logits depend on is exactly its chunk."""
    return _model(32, 40, [_att(2, 1, 8, 16, 4, 50.0, 20, True, None, scale=0.1)], 1.3)


CONFIGS = {"a": config_a, "b": config_b, "c": config_c, "d": config_d, "one": config_one}


def make_tensors(cfg: dict, seed: int) -> dict:
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def mat(o, i, s=1.0):
        return (torch.randn(o, i, generator=g) * s / math.sqrt(i)).to(torch.bfloat16)

    def vec(n, mean=0.0, s=0.5):
        return (mean + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    # rows with a mean that is not 0, so that a norm that keeps it shows
    t = {"embed": (0.4 + torch.randn(V, W, generator=g)).to(torch.bfloat16), "final.norm": vec(W, 1.0, 0.3)}
    for i, L in enumerate(cfg["layers"]):
        p, m, x = f"l{i}.", L["mixer"], f"l{i}.mix."
        H, G, D, Vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        t.update({p + "norm1": vec(W, 1.0, 0.3), p + "norm1b": vec(W, 1.0, 0.3)})
        t.update({x + "q": mat(H * D, W, 2.0), x + "k": mat(G * D, W, 2.0), x + "v": mat(G * Vd, W), x + "g": mat(H * Vd, W, 2.0),
                  x + "o": mat(W, H * Vd)})
        if m["v_mix"]:
            t[x + "vmix"] = torch.tensor(0.3 + 0.5 * float(torch.rand((), generator=g))).to(torch.bfloat16)
        if L.get("mlp"):
            f = L["mlp"]
            t.update({p + "norm2": vec(W, 1.0, 0.3), p + "norm2b": vec(W, 1.0, 0.3)})
            if f["kind"] == "dense":
                t.update({p + "mlp.up": mat(f["ff"], W, 1.5), p + "mlp.down": mat(W, f["ff"])})
            else:
                E, n = f["router"]["experts"], f["expert"]["ff"]
                t[p + "mlp.router"] = mat(E, W, 5.0)
                for e in range(E):
                    t.update({p + f"mlp.e{e}.up": mat(n, W, 1.5), p + f"mlp.e{e}.down": mat(W, n)})
    return t


_MODELS: dict = {}


def model_dir(tmp_path_factory, name: str):
    """(folder, config dict, tensors) of a named test model, written once per session."""
    if name not in _MODELS:
        from safetensors.torch import save_file
        cfg = CONFIGS[name]()
        t = make_tensors(cfg, seed={"a": 3, "b": 5, "c": 7, "d": 9, "one": 11}[name])
        d = tmp_path_factory.mktemp("nigozen_" + name)
        save_file({k: v.contiguous() for k, v in t.items()}, str(d / "model.safetensors"))
        (d / "config.json").write_text(json.dumps(cfg))
        _MODELS[name] = (str(d), cfg, t)
    return _MODELS[name]


_ORACLE: dict = {}


def oracle_run(name, cfg, W, tokens):
    key = (name, tuple(tokens))
    if key not in _ORACLE:
        lg, streams = oracle.forward(cfg, W, list(tokens))
        _ORACLE[key] = (lg.float(), streams.float())
    return _ORACLE[key]


def oracle_logits(name, cfg, W, tokens):
    return oracle_run(name, cfg, W, tokens)[0]


def engine(path, device, dtype, pages=16, seqs=4, **kw):
    from vgate.runtime.engine import EngineConfig, LLMEngine
    cfg = dict(model=path, dtype=dtype, device=device, max_model_len=pages * 16, max_num_seqs=seqs,
               max_num_batched_tokens=pages * 16, num_kv_blocks=pages, enable_prefix_caching=False, enforce_eager=True,
               warmup=False, prefill_autotune=False, async_scheduling=False)
    cfg.update(kw)
    return LLMEngine(EngineConfig(**cfg))


def rel(a: torch.Tensor, b: torch.Tensor) -> float:
    a, b = a.double().cpu(), b.double().cpu()
    return float((a - b).pow(2).mean().sqrt() / b.pow(2).mean().sqrt())


def tol(dtype: str) -> float:
    return 3e-4 if dtype == "float32" else 6e-2


def close(got: torch.Tensor, want: torch.Tensor, dtype: str) -> bool:
    """fp32: the whole result within tol. bf16: per token, the median within tol and four in five within 0.15 (in
    models this small a rounding can turn a router's close call and move that token; a fault of a mechanism moves
    most tokens by O(1))."""
    if dtype == "float32":
        return rel(got, want) < tol(dtype)
    g, w = got.double().cpu(), want.double().cpu()
    e = (g - w).pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt()
    return float(e.median()) < tol(dtype) and float((e < 0.15).double().mean()) >= 0.8


def tokens_of(cfg, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def replay_all(eng, rid, toks, cuts):
    """Run one request in portions of the given sizes (then one token at a time); logits at every place."""
    out, at = [], 0
    sizes = list(cuts)
    while at < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
        lg = eng.replay_step([(rid, toks[at: at + n], list(range(n)))], [rid] if at + n == len(toks) else [])
        out.append(lg.float().cpu())
        at += n
    return torch.cat(out)


# -------------------------------------------------------------------------------------------- engine
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompt_matches_oracle(tmp_path_factory, device, dtype, name):
    path, cfg, W = model_dir(tmp_path_factory, name)
    toks = tokens_of(cfg, 130 if name == "c" else 67, seed=1)
    eng = engine(path, device, dtype)
    lg = replay_all(eng, "w", toks, [len(toks)])
    assert close(lg, oracle_logits(name, cfg, W, toks), dtype)
    one = replay_all(eng, "one", toks[:1], [1])  # a sequence of one token (first position only)
    assert close(one, oracle_logits(name, cfg, W, toks)[:1], dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_layers_match_oracle(tmp_path_factory, device, name):
    path, cfg, W = model_dir(tmp_path_factory, name)
    toks = tokens_of(cfg, 53, seed=2)
    eng = engine(path, device, "float32")
    eng.model.capture_layers = []
    replay_all(eng, "l", toks, [len(toks)])
    want = oracle_run(name, cfg, W, toks)[1]
    assert len(eng.model.capture_layers) == want.shape[0] == len(cfg["layers"])
    for i, got in enumerate(eng.model.capture_layers):
        assert rel(got[: len(toks)], want[i]) < 1e-4, f"stream after layer {i}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [[1], [30], [2, 2, 2, 3, 5, 7, 16, 17], [15, 1, 16, 2, 14], [36, 2, 36, 2], [47, 2]])
def test_portions_and_decoding_match_whole(tmp_path_factory, device, dtype, cuts):
    """Prefill against token-by-token decoding and portions of several sizes down to two tokens (cuts inside
    pages and chunks, at their borders and across them); the tail decodes one token at a time."""
    path, cfg, W = model_dir(tmp_path_factory, "c")
    toks = tokens_of(cfg, 120, seed=3)
    eng = engine(path, device, dtype)
    whole = replay_all(eng, "whole", toks, [len(toks)])
    cut = replay_all(eng, "cut", toks, cuts)
    assert rel(cut, whole) < 2e-5 if dtype == "float32" else close(cut, whole, dtype)
    assert close(cut, oracle_logits("c", cfg, W, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(tmp_path_factory, device):
    """A short prompt and then hundreds of single tokens, across many chunks."""
    path, cfg, W = model_dir(tmp_path_factory, "a")
    toks = tokens_of(cfg, 300, seed=4)
    eng = engine(path, device, "float32", pages=20)
    got = replay_all(eng, "d", toks, [3])
    want = oracle_logits("a", cfg, W, toks)
    assert rel(got, want) < tol("float32") and rel(got[-5:], want[-5:]) < tol("float32")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[64], [5, 2, 13, 7, 33], [1]])
def test_a_position_depends_on_its_chunk_alone(tmp_path_factory, device, cuts):
    """One layer, chunks of 20: replacing a token moves the logits of the later positions of its own chunk and, to
    the last bit, of no position of another chunk, however the prompt is cut."""
    path, cfg, W = model_dir(tmp_path_factory, "one")
    toks = tokens_of(cfg, 64, seed=8)
    size = cfg["layers"][0]["mixer"]["mask"]["size"]
    eng = engine(path, device, "float32")
    base = replay_all(eng, "base", toks, cuts)
    for n, j in enumerate((0, 19, 20, 39, 47, 59)):   # first and last tokens of chunks, a page border
        other = list(toks)
        other[j] = (other[j] + 7) % cfg["vocab"]
        got = replay_all(eng, f"o{n}", other, cuts)
        moved = (got != base).any(-1)
        end = min((j // size + 1) * size, len(toks))
        assert moved[j:end].all(), j
        assert not moved[:j].any() and not moved[end:].any(), j


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["a", "c"])
def test_mixed_batches_and_reuse(tmp_path_factory, device, dtype, name):
    """Unequal requests in one batch (portions beside single tokens) against each alone, with a pool
    so small that pages and state slots are freed and taken again by later requests."""
    path, cfg, W = model_dir(tmp_path_factory, name)
    reqs = {f"q{i}": tokens_of(cfg, n, seed=10 + i) for i, n in enumerate([41, 5, 23, 1, 30, 17, 9, 48])}
    eng = engine(path, device, dtype, pages=8, seqs=3)  # 128 tokens, 3 slots: 8 requests must reuse both
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
    order = list(reqs)
    live, step = [], 0
    plan = [7, 1, 16, 2, 1, 9, 3]
    while order or live:
        while order and len(live) < 3 and sum((len(reqs[k]) + 15) // 16 for k in live + [order[0]]) <= 8:
            live.append(order.pop(0))
        entries, end = [], []
        for j, k in enumerate(live):
            n = min(plan[(step + j) % len(plan)], len(reqs[k]) - at[k])
            if (step + j) % 5 == 4 and len(live) > 1:
                continue  # a request may sit a step out
            entries.append((k, reqs[k][at[k]: at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        step += 1
        if not entries:
            continue
        lg = eng.replay_step(entries, end).float().cpu()
        o = 0
        for k, t, w in entries:
            got[k].append(lg[o: o + len(w)])
            o += len(w)
        live = [k for k in live if k not in end]
    assert eng.kvm.num_free() == 8 and eng.kvm.free_state_slots() == 3
    for k, toks in reqs.items():
        assert close(torch.cat(got[k]), oracle_logits(name, cfg, W, toks), dtype), k


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(tmp_path_factory, device):
    """add_request -> scheduler (chunked prefill, continuous batching) -> sampler: every generated token
    is the oracle's arg-max (or within rounding of it) given the tokens before it."""
    from vgate.runtime.sampling_params import SamplingParams
    path, cfg, W = model_dir(tmp_path_factory, "a")
    eng = engine(path, device, "float32", pages=24, seqs=3, max_num_batched_tokens=24, enforce_eager=False)
    prompts = {"g0": tokens_of(cfg, 29, seed=31), "g1": tokens_of(cfg, 3, seed=32), "g2": tokens_of(cfg, 40, seed=33),
               "g3": tokens_of(cfg, 11, seed=34)}
    done = {}
    for rid, p in prompts.items():
        eng.add_request(rid, prompt_ids=p, params=SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True),
                        callback=lambda kind, seq, payload: done.__setitem__(seq.request_id, seq))
    eng.run_until_idle()
    assert set(done) == set(prompts)
    for rid, p in prompts.items():
        out = done[rid].output_ids
        assert len(out) == 12
        ref = oracle_logits("a", cfg, W, p + out[:-1])
        for i, tok in enumerate(out):
            row = ref[len(p) - 1 + i]
            assert row[tok] >= row.max() - 1e-3 * row.std(), (rid, i, tok, int(row.argmax()))
    assert eng.kvm.free_state_slots() == 3


@pytest.mark.gpu
def test_generation_replays_graphs(tmp_path_factory):
    """Later runs of the same requests replay the hipGraphs captured after the first and sample the same tokens (bf16,
    the serving dtype), also after eager work in between."""
    from vgate.runtime.sampling_params import SamplingParams
    path, cfg, W = model_dir(tmp_path_factory, "c")
    eng = engine(path, "cuda", "bfloat16", pages=32, seqs=4, enforce_eager=False)
    outs = []
    for rnd in range(3):
        done = {}
        for i in range(3):
            eng.add_request(f"r{rnd}_{i}", prompt_ids=tokens_of(cfg, 9 + 17 * i, seed=40 + i),
                            params=SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True),
                            callback=lambda kind, seq, payload: done.__setitem__(seq.request_id[3:], seq.output_ids))
        hits = eng.runner.graph_hits
        eng.run_until_idle()
        outs.append(done)
        torch.randn(64, 64, device="cuda").sum().item()
    assert eng.runner.graph_hits > hits
    assert outs[0] == outs[1] == outs[2]


@pytest.mark.gpu
def test_packed_gemm_path_matches_row_major_and_oracle(tmp_path_factory, monkeypatch):
    """bf16 at sizes whose projections run on the fragment-packed MFMA GEMMs (the dense activation is a row kernel
    behind them): same logits as with every matrix on the row-major GEMM (activation in its epilogue), and the
    oracle's; prompt portions and decoded tokens."""
    from vgate.models import mixers
    path, cfg, W = model_dir(tmp_path_factory, "d")
    toks = tokens_of(cfg, 45, seed=5)
    got = {}
    for packed in (True, False):
        monkeypatch.setattr(mixers, "USE_PACKED", packed)
        eng = engine(path, "cuda", "bfloat16")
        assert all(p.packed == packed for p in (eng.model.layers[0].proj, eng.model.layers[0].ff.up, eng.model.head))
        got[packed] = replay_all(eng, "p", toks, [30, 2, 9])
        del eng
    assert close(got[True], got[False], "bfloat16")
    assert close(got[True], oracle_logits("d", cfg, W, toks), "bfloat16")
    eng = engine(path, "cuda", "float32")
    assert rel(replay_all(eng, "f", toks, [30, 2, 9]), oracle_logits("d", cfg, W, toks)) < tol("float32")


def test_registry_and_config(tmp_path_factory):
    from vgate.models.config import HybridArch, resolve_arch
    from vgate.models.hybrid import tensor_shapes
    path, cfg, W = model_dir(tmp_path_factory, "a")
    a = resolve_arch(path)
    assert isinstance(a, HybridArch) and a.family == "nigozen" and a.arrangement == "sandwich_norm"
    assert a.norm == "layer" and a.embed_scale == 1.6 and a.tie_embeddings and a.rms_eps == 1e-5
    assert all(L.kind == "window_attention" and L.mixer["sink"] == "one" and L.mixer["gate"] == "sigmoid" for L in a.layers)
    assert [L.mixer["chunk"] for L in a.layers] == [9, 5, 21, 19, 30] and all(L.mixer["window"] is None for L in a.layers)
    assert [L.mixer["value_mix"] for L in a.layers] == [False, True, False, True, True]
    assert a.layers[0].mixer["rot"] == {"dims": 4, "base": 100.0, "layout": "pairs"}
    assert a.layers[0].mlp == {"kind": "dense", "ff": 26, "gated": False, "act": "gelu"}
    assert a.layers[1].mlp["router"] == {"experts": 5, "top": 2, "score": "top_softmax", "correction": False}
    assert a.layers[1].mlp["expert"] == {"ff": 13, "gated": False, "act": "relu2"} and a.layers[2].mlp is None
    shapes = tensor_shapes(a, nominal=None)
    assert set(shapes) == set(W) and all(tuple(W[k].shape) == s for k, s in shapes.items())
    t = resolve_arch("nigozen-tiny")
    assert t.family == "nigozen" and t.num_params() > 0


def test_mixing_layers_must_agree_on_their_values(tmp_path):
    from safetensors.torch import save_file
    cfg = _model(16, 20, [_att(2, 1, 4, 4, 4, 10.0, 8, True, None), _att(2, 2, 4, 4, 4, 10.0, 8, True, None)], 1.0)
    save_file(make_tensors(cfg, 1), str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match="mix values"):
        engine(str(tmp_path), "cpu", "float32")


@pytest.mark.parametrize("device", DEVICES)
def test_preset_runs(device):
    eng = engine("nigozen-tiny", device, "bfloat16")
    lg = eng.replay_step([("x", list(range(40)), [0, 39])], ["x"])
    assert lg.shape == (2, 300) and bool(torch.isfinite(lg).all())


# --------------------------------------------------------------------------------- mechanisms alone
def _step_meta(new, ctx, table, d):
    """Device tensors of one step of one sequence: ``new`` tokens that end at context ``ctx``."""
    pos = list(range(ctx - new, ctx))
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=d)  # noqa: E731
    return i32(pos), i32([table[j // 16] * 16 + j % 16 for j in pos]), i32([0, new]), i32([ctx])


STEPS_310 = ([310], [61, 2, 35, 1, 1, 210], [240] + [1] * 70)
SCATTERED = [7, 2, 9, 4, 11, 0, 5, 13, 1, 8, 3, 6, 10, 12, 14, 15, 16, 17, 18, 19]


def _chunk_reference(q, k, v, other, lam, gate, H, G, D, V, scale, dims, base, size, one=True):
    """float64, one sequence: rotated q / k, values blended with ``other``, chunked attention, sigmoid gate."""
    T = q.shape[0]
    pos = torch.arange(T)
    q3 = oracle.turn_pairs(q.double().view(T, H, D), pos, dims, base)
    k3 = oracle.turn_pairs(k.double().view(T, G, D), pos, dims, base)
    v3 = ((1.0 - lam) * v.double() + lam * other.double()).view(T, G, V)
    if one:
        o = oracle.attend(q3, k3, v3, scale, size)
    else:
        see = oracle.visible(T, size)
        o = torch.zeros(T, H, V, dtype=torch.float64)
        for h in range(H):
            g = h // (H // G)
            s = (q3[:, h] @ k3[:, g].t() * scale).masked_fill(~see, float("-inf"))
            o[:, h] = torch.softmax(s, -1) @ v3[:, g]
    return (o.reshape(T, H * V) * torch.sigmoid(gate.double())).float()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("H,G,D,V,dims,size", [(4, 2, 8, 16, 4, 37), (2, 2, 16, 8, 6, 16), (3, 1, 6, 5, 2, 100),
                                               (2, 1, 160, 136, 32, 64), (2, 2, 104, 72, 40, 1000), (3, 3, 8, 8, 2, 1)])
def test_chunked_attention_on_crafted_keys(device, f32, H, G, D, V, dims, size):
    """The attention ops alone: for chosen query positions one key is made to dominate: the first key of the query's
    chunk, the last one before it (not seen), the token itself, keys at page borders, a key hundreds back. One
    prompt, portions cut inside pages and chunks, and token by token over scattered pages whose unused rows hold
    garbage; the FMA and (bf16, GPU, key size a multiple of 8) the MFMA kernels; values blended with another row."""
    from vgate.models.mixers import WindowAttention
    from vgate.ops import seq
    dt = torch.float32 if f32 else torch.bfloat16
    d = torch.device(device)
    g = torch.Generator().manual_seed(19)
    T, scale, base, lam = 310, 0.8 / math.sqrt(D), 50.0, 0.35
    rep = H // G
    q, k, v, other, gate = (torch.randn(T, n, generator=g) for n in (H * D, G * D, G * V, G * V, H * V))
    probe = torch.zeros(D)
    probe[dims:] = 1.0            # unrotated entries keep the probe's direction at every position
    probe *= math.sqrt(6.0 / (probe.norm() ** 2 * scale))
    queries = [309, 300, 290, 255, 200, 160, 131, 64, 48, 37]
    for n, i in enumerate(queries):
        first = i - i % size
        j = (first, first - 1, i, max(first, i // 16 * 16), max(first, i // 16 * 16 - 1))[n % 5]
        if j < 0:
            continue
        h = n % H
        k[j].view(G, D)[h // rep] += probe
        q[i].view(H, D)[h] += probe
    q, k, v, other, gate = (x.to(dt).float() for x in (q, k, v, other, gate))
    args = (H, G, D, V, scale, dims, base)
    want = _chunk_reference(q, k, v, other, lam, gate, *args, size)
    inv_freq = seq.rope_inv_freq(dims, base, d)
    one = torch.zeros(H, device=d)
    for steps in STEPS_310:
        for mfma in ([None, 0, 1] if device == "cuda" and not f32 and D % 8 == 0 else [None]):
            kc = torch.full((20, G, 16, D), 9.0, dtype=dt, device=d)
            vc = torch.full((20, G, 16, V), -9.0, dtype=dt, device=d)
            vt = torch.full((20, G, V, 16), -9.0, dtype=dt, device=d) if mfma is not None else None
            bt = torch.tensor([SCATTERED], dtype=torch.int32, device=d)
            done, outs = 0, []
            for n in steps:
                pos, slots, qs, cl = _step_meta(n, done + n, SCATTERED, d)
                cut = lambda x: x[done: done + n].to(d, dt).contiguous()  # noqa: E731
                qo = torch.zeros(n, H * D, dtype=dt, device=d)
                seq.window_write(cut(q), cut(k), cut(v), None, None, 0.0, False, pos, slots, inv_freq, dims, None, kc, vc, qo, H, G,
                                 vt=vt, v_other=cut(other), lam=lam)
                o = torch.zeros(n, H * V, dtype=dt, device=d)
                seq.window_attn(qo, kc, vc, None, None, bt, cl, qs, o, scale, H, WindowAttention.FULL, 0, one, None, vt=vt,
                                prefill_kernel=mfma or 0, gate=cut(gate), chunk=size)
                outs.append(o.float().cpu())
                done += n
            got = torch.cat(outs)
            assert rel(got, want) < (3e-5 if f32 else 2e-2), (len(steps), mfma)
            for i in queries:   # the crafted positions by themselves
                assert rel(got[i], want[i]) < (1e-4 if f32 else 3e-2), (i, len(steps), mfma)
    # the cases matter: a chunk one longer or shorter, no one in the denominator, unmixed values move the answer
    at = torch.tensor(queries)
    if size < T:
        assert rel(_chunk_reference(q, k, v, other, lam, gate, *args, size + 1)[at], want[at]) > 0.02
    if 1 < size < T:
        assert rel(_chunk_reference(q, k, v, other, lam, gate, *args, size - 1)[at], want[at]) > 0.02
    if size <= 100:
        assert rel(_chunk_reference(q, k, v, other, lam, gate, *args, size, one=False), want) > 0.005
    assert rel(_chunk_reference(q, k, v, other, 0.0, gate, *args, size), want) > 0.02


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("f32", [True, False])
def test_chunked_batch_of_unequal_sequences(device, f32):
    """Decoded tokens of several sequences in one launch (the split of a token's key tiles over workgroups included)
    beside a portion: every sequence as alone, on pages that another sequence used before."""
    from vgate.models.mixers import WindowAttention
    from vgate.ops import seq
    dt = torch.float32 if f32 else torch.bfloat16
    d = torch.device(device)
    g = torch.Generator().manual_seed(29)
    H, G, D, V, size, scale, dims, base = 4, 2, 16, 16, 300, 0.3, 8, 100.0
    lens = [411, 17, 300, 301, 1]
    data = [[torch.randn(n, w, generator=g).to(dt).float() for w in (H * D, G * D, G * V, H * V)] for n in lens]
    want = [_chunk_reference(q, k, v, v, 0.0, gt, H, G, D, V, scale, dims, base, size) for q, k, v, gt in data]
    pages = [(n + 15) // 16 for n in lens]
    perm = torch.randperm(sum(pages), generator=g).tolist()
    tables = [[perm.pop() for _ in range(n)] for n in pages]
    bt = torch.zeros(len(lens), max(pages), dtype=torch.int32)
    for s, t in enumerate(tables):
        bt[s, : len(t)] = torch.tensor(t, dtype=torch.int32)
    bt = bt.to(d)
    P = sum(pages)
    kc = torch.full((P, G, 16, D), 5.0, dtype=dt, device=d)   # what an earlier sequence left
    vc = torch.full((P, G, 16, V), -5.0, dtype=dt, device=d)
    vt = torch.full((P, G, V, 16), -5.0, dtype=dt, device=d) if device == "cuda" and not f32 else None
    inv_freq, one = seq.rope_inv_freq(dims, base, d), torch.zeros(H, device=d)
    done = [0] * len(lens)
    outs: list = [[] for _ in lens]
    plans = ([390, 5, 297, 298, 0], [1, 1, 1, 1, 1], [7, 1, 1, 1, 0], [1, 1, 1, 1, 0], [12, 9, 0, 0, 0])
    for new in plans:
        pos, slots, qs, cl = [], [], [0], []
        for s, n in enumerate(new):
            for j in range(done[s], done[s] + n):
                pos.append(j)
                slots.append(tables[s][j // 16] * 16 + j % 16)
            qs.append(qs[-1] + n)
            cl.append(done[s] + n)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=d)  # noqa: E731
        cat = lambda w: torch.cat([data[s][w][done[s]: done[s] + n] for s, n in enumerate(new)]).to(d, dt).contiguous()  # noqa: E731
        T = qs[-1]
        qo, o = torch.zeros(T, H * D, dtype=dt, device=d), torch.zeros(T, H * V, dtype=dt, device=d)
        seq.window_write(cat(0), cat(1), cat(2), None, None, 0.0, False, i32(pos), i32(slots), inv_freq, dims, None, kc, vc, qo, H, G, vt=vt)
        seq.window_attn(qo, kc, vc, None, None, bt, i32(cl), i32(qs), o, scale, H, WindowAttention.FULL, 0, one, None, vt=vt,
                        gate=cat(3), chunk=size)
        for s, n in enumerate(new):
            outs[s].append(o[qs[s]: qs[s + 1]].float().cpu())
            done[s] += n
    assert done == lens
    for s in range(len(lens)):
        assert rel(torch.cat(outs[s]), want[s]) < (3e-5 if f32 else 2e-2), s


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("T,W", [(5, 42), (3, 1), (4, 768), (2, 4100)])
def test_norms_and_residual_kernel(device, f32, T, W):
    """Layer norms of rows with a large mean; the residual update with its output norm, the next norm and the weighted
    sum of a token's expert rows, in every combination; widths below and beyond what a workgroup keeps in registers."""
    from vgate.ops import seq
    dt = torch.float32 if f32 else torch.bfloat16
    d = torch.device(device)
    g = torch.Generator().manual_seed(31)
    eps, mult, top = 1e-5, 0.7, 3
    x = torch.randn(T, W, generator=g) + 5.0
    y = (torch.randn(T, W, generator=g) * 2.0 - 3.0).to(dt)
    rows = (torch.randn(T * top, W, generator=g) + 2.0).to(dt)
    pos = torch.randperm(T * top, generator=g).to(torch.int32)
    wts = torch.rand(T, top, generator=g)
    pw, w = 1.0 + 0.3 * torch.randn(W, generator=g), 1.0 + 0.3 * torch.randn(W, generator=g)
    out = torch.zeros(2, W, dtype=dt, device=d)
    pick = torch.tensor([T - 1, 0], dtype=torch.int32, device=d)
    seq.norm_rows(x.to(d), w.to(d), eps, out, rows=pick, center=True)
    fine = 2e-5 if f32 else 5e-3

    def near(got, want):
        want = want.double()
        return float((got.double().cpu() - want).abs().max()) <= fine * max(float(want.abs().max()), 1.0)

    assert near(out, oracle.layer_norm(x.double(), eps, w)[[T - 1, 0]])

    def norm(a, ww, center):
        return oracle.layer_norm(a, eps, ww) if center else a / torch.sqrt((a * a).mean(-1, keepdim=True) + eps) * ww.double()

    picked = (rows.double()[pos.long()].view(T, top, W) * wts.double()[:, :, None]).sum(1)
    for center in (True, False):
        for post in (None, pw):
            for gather in (False, True):
                for nxt in (None, w):
                    u = picked if gather else y.double()
                    u = norm(u, post, center) if post is not None else u
                    wx = x.double() + mult * u
                    xd = x.clone().to(d)
                    hd = torch.zeros(T, W, dtype=dt, device=d) if nxt is not None else None
                    src = (rows.to(d), pos.to(d), wts.to(d)) if gather else y.to(d)
                    seq.residual_norm(xd, src, mult, nxt.to(d) if nxt is not None else None, eps, hd,
                                      post_w=post.to(d) if post is not None else None, center=center)
                    assert float((xd.double().cpu() - wx).abs().max()) < 2e-5 * max(1.0, float(wx.abs().max()))
                    if nxt is not None and not (center and W == 1):
                        assert near(hd, norm(wx, nxt, center)), (center, post is not None, gather)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top", [(1, 1), (5, 2), (7, 7), (70, 9), (600, 3)])
def test_router_weighs_the_chosen_alone(device, E, top):
    """The largest logits are chosen and weighted by the softmax over them alone, also where the logits are so far
    apart that a softmax over all experts would vanish for some of the chosen."""
    from vgate.ops import seq
    d = torch.device(device)
    g = torch.Generator().manual_seed(37)
    T = 13
    z = torch.randn(T, E, generator=g) * 3.0
    z[3:6] = z[3:6] * 60.0
    idx = torch.zeros(T, top, dtype=torch.int32, device=d)
    wts = torch.zeros(T, top, device=d)
    seq.moe_route(z.to(d), None, top, 0.0, idx, wts, score=seq.ROUTE_TOP_SOFTMAX)
    want, order = torch.sort(z.double(), -1, descending=True)
    assert torch.equal(idx.cpu().long(), order[:, :top])
    assert float((wts.cpu().double() - torch.softmax(want[:, :top], -1)).abs().max()) < 2e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("act", ["gelu", "relu2"])
def test_activations_without_a_gate(device, f32, act):
    """act(up h) as the epilogue of a plain GEMM, of a GEMM grouped by expert (with gathered rows; few rows and so
    many that the LDS-tiled form runs), and as a row kernel."""
    from vgate.ops import seq
    dt = torch.float32 if f32 else torch.bfloat16
    d = torch.device(device)
    g = torch.Generator().manual_seed(41)
    code = {"gelu": seq.ACT_GELU, "relu2": seq.ACT_RELU2}[act]

    def fn(z):
        return z * 0.5 * (1.0 + torch.erf(z / math.sqrt(2.0))) if act == "gelu" else torch.clamp(z, min=0.0) ** 2

    limit = 1e-5 if f32 else 1e-2
    a, w = (torch.randn(s, generator=g).to(dt) for s in ((9, 21), (14, 21)))
    out = torch.zeros(9, 14, dtype=dt, device=d)
    seq.gemm(a.to(d), w.to(d), out, act=code)
    assert rel(out.float(), fn(a.double() @ w.double().t())) < limit
    for M, E, K, N in ((11, 3, 24, 16), (1500, 4, 64, 520)):
        a, w = torch.randn(M, K, generator=g).to(dt), (torch.randn(E, N, K, generator=g) / math.sqrt(K)).to(dt)
        ends = sorted(torch.randint(0, M + 1, (E - 1,), generator=g).tolist())
        off = [0] + ends + [M]
        rows = torch.randperm(M, generator=g)
        want = torch.cat([fn(a.double()[rows[off[e]: off[e + 1]]] @ w[e].double().t()) for e in range(E)])
        out = torch.zeros(M, N, dtype=dt, device=d)
        i32 = lambda x: torch.as_tensor(x, dtype=torch.int32).to(d)  # noqa: E731
        seq.gemm(a.to(d), w.to(d), out, a_rows=i32(rows), group_off=i32(off), act=code)
        assert rel(out.float(), want) < limit
    if not f32:
        x = (torch.randn(7, 40, generator=g) * 3.0).to(dt)
        y = x.clone().to(d)
        seq.act_rows(y, code)
        assert rel(y.float(), fn(x.double())) < 5e-3


@pytest.mark.parametrize("device", DEVICES)
def test_embedding_rows_are_scaled(device):
    from vgate.ops import seq
    d = torch.device(device)
    g = torch.Generator().manual_seed(43)
    table = torch.randn(9, 13, generator=g).to(torch.bfloat16)
    ids = torch.tensor([3, 0, -2, 8], dtype=torch.int32)     # -2: the previous step's second sample
    prev = torch.tensor([1, 5, 2], dtype=torch.int32)
    out = torch.zeros(4, 13, device=d)
    seq.embed_rows(ids.to(d), table.to(d), out, prev=prev.to(d), scale=0.37)
    assert float((out.cpu() - table[[3, 0, 5, 8]].float() * 0.37).abs().max()) < 1e-6
