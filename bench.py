"""Measures decoding and prefill of the TinyLlama 1.1B shape with random weights on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--batch 8] [--context 2048] [--dtype bfloat16]
                    [--shape tinyllama|llama2_7b|llama3_8b] [--layers N] [--no-points]
    python bench.py --workload serving|mixed [--shape ...] [--token-budget 2048]     (records of their own)
    python bench.py --prefill TOKENS                                                 (a prompt step alone)

A step is one decode step of the whole batch.  The batch's requests are first prefilled so that
after the warm-up and the K timed steps their length is `context`; then W untimed and exactly K
timed steps run, each through the engine's own step function and sampler (greedy), and one JSON
line is printed; that is done `--repeats` times and the median run counts.  `value` is decoded
tokens per second.  The same line carries the prefill of a 2,048-token prompt, the decode step's
share of the HBM roofline, and in `points` (every key a number): decoding at batch 1 and 64, the
workload of a 128-token prompt with 128 generated tokens, the same model in true 32-bit (decoding and
the prompt step), and decoding at the layer sizes of Llama-2-7B and Llama-3-8B with a quarter of
their layers (the counts are named); `*_frac` is the share of the published peak (HBM for decoding,
the matrix cores of the dtype for prompts).

Peaks are the MI355X's published ones: HBM 8 TB/s; dense MFMA 2.5 PFLOP/s for bfloat16, 157.3
TFLOP/s for float32.  `measured_peaks` holds what two microbenchmarks of the kernel library reach
on the machine at hand (a streaming read, chains of bfloat16 matrix instructions), and
`frac_of_measured` the same shares against those.
"""
import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

HBM_PEAK = 8.0e12
MFMA_PEAK = {"bfloat16": 2.5e15, "float32": 157.3e12}

# the TinyLlama 1.1B configuration
TINYLLAMA = dict(model_type="llama", architectures=["LlamaForCausalLM"], hidden_size=2048, intermediate_size=5632,
                 num_hidden_layers=22, num_attention_heads=32, num_key_value_heads=4, max_position_embeddings=2048,
                 vocab_size=32000, rms_norm_eps=1e-5, rope_theta=10000.0, tie_word_embeddings=False, attention_bias=False,
                 hidden_act="silu", bos_token_id=1, eos_token_id=2, torch_dtype="bfloat16")


# the layer sizes of the Llama-2-7B and Llama-3-8B configurations, for `--shape`
OTHER_SHAPES = {
    "llama2_7b": ("Llama-2-7B shape", dict(hidden_size=4096, intermediate_size=11008, num_hidden_layers=32, num_attention_heads=32,
                                           num_key_value_heads=32, max_position_embeddings=4096, vocab_size=32000, rope_theta=10000.0)),
    "llama3_8b": ("Llama-3-8B shape", dict(hidden_size=4096, intermediate_size=14336, num_hidden_layers=32, num_attention_heads=32,
                                           num_key_value_heads=8, max_position_embeddings=8192, vocab_size=128256, rope_theta=500000.0)),
}


def weight_bytes_per_step(cfg, itemsize):
    """Bytes of weights a decode step reads: every matrix once, the norms, the head; of the
    embedding table only the batch's rows (not counted)."""
    h, i, d = cfg["hidden_size"], cfg["intermediate_size"], cfg["hidden_size"] // cfg["num_attention_heads"]
    qd, kvd = cfg["num_attention_heads"] * d, cfg["num_key_value_heads"] * d
    per_layer = (qd + 2 * kvd) * h + h * qd + 2 * i * h + h * i + 2 * h
    return (cfg["num_hidden_layers"] * per_layer + h + cfg["vocab_size"] * h) * itemsize


def kv_bytes_per_token(cfg, itemsize):
    d = cfg["hidden_size"] // cfg["num_attention_heads"]
    return 2 * cfg["num_key_value_heads"] * d * cfg["num_hidden_layers"] * itemsize


def prefill_flops(cfg, tokens):
    h, i, d = cfg["hidden_size"], cfg["intermediate_size"], cfg["hidden_size"] // cfg["num_attention_heads"]
    nq = cfg["num_attention_heads"]
    qd, kvd = nq * d, cfg["num_key_value_heads"] * d
    linear = 2 * tokens * cfg["num_hidden_layers"] * ((qd + 2 * kvd) * h + h * qd + 3 * i * h)
    attention = cfg["num_hidden_layers"] * 4 * nq * d * tokens * (tokens + 1) // 2
    head = 2 * cfg["vocab_size"] * h
    return linear + attention + head


def time_decode(engine, torch, batch, context, steps, warmup, vocab):
    """`batch` requests through the engine's own loop (scheduler, recorded decode steps, sampling
    on the device, tokens read a step behind): prompts first, then warmup + steps decode steps, the
    last token of each request being the `context`-th of its sequence; returns seconds for the
    timed steps."""
    from tlie_amd.engine import Request, SamplingParams, Scheduler
    prompt_len = context - steps - warmup - 1
    generator = torch.Generator().manual_seed(batch)
    # the token budget lets all prompts through in one step, so that every request decodes from the same step on
    scheduler = Scheduler(engine.cache, max_tokens_per_step=batch * prompt_len, max_seqs_per_step=batch,
                          max_positions=engine.spec.max_positions, eos_token_id=engine.spec.eos_token_id)
    requests = [Request(id=("bench", index), prompt=torch.randint(0, vocab, (prompt_len,), generator=generator).tolist(),
                        params=SamplingParams(max_tokens=steps + warmup + 1)) for index in range(batch)]
    for request in requests:
        scheduler.add(request)
    assert engine.run(scheduler, max_steps=1) == 1
    assert all(len(request.generated) == 1 for request in requests)
    assert engine.run(scheduler, max_steps=warmup) == warmup
    torch.cuda.synchronize()
    started = time.perf_counter()
    ran = engine.run(scheduler, max_steps=steps)
    torch.cuda.synchronize()
    elapsed = time.perf_counter() - started
    assert ran == steps and not scheduler.has_work() and all(len(request.generated) == steps + warmup + 1 for request in requests)
    return elapsed


def time_prefill(engine, torch, tokens, vocab, repeats=3):
    from tlie_amd import StepEntry
    generator = torch.Generator().manual_seed(tokens)
    prompt = torch.randint(0, vocab, (tokens,), generator=generator).tolist()
    best = None
    for _ in range(repeats + 1):
        engine.admit("prefill")
        torch.cuda.synchronize()
        started = time.perf_counter()
        logits = engine.step([StepEntry("prefill", prompt, [tokens - 1])])
        logits.argmax(-1).item()
        torch.cuda.synchronize()
        elapsed = time.perf_counter() - started
        engine.finish("prefill")
        best = elapsed if best is None else min(best, elapsed)       # the first run also warms up
    return best


def run_workload(engine, torch, workload, vocab, budget, chunk, slice_steps=8, prompt_cap=None):
    """A whole workload through the scheduler and the engine's loop, timed in slices of a few
    steps.  Returns the record's `value` parts and what the scheduler and the cache counted.
    serving: 64 requests at once, prompts of 128 to 2048 random tokens (or as many as leave the
    model's positions room for the output), 256 tokens decoded each, continuous batching.  mixed: 8 requests of 8192 positions (prompts of 8176 tokens, 16 decoded), cut into portions of `chunk`, beside 56
    streams with prompts of 32 to 128 tokens that decode 256 tokens each."""
    import random
    from tlie_amd.engine import Request, SamplingParams, Scheduler
    rng = random.Random(7)
    generator = torch.Generator().manual_seed(7)
    if workload == "serving":
        longest = min(2048, engine.spec.max_positions - 256)           # (a model of 2048 positions: prompts up to 1792)
        shapes = [(rng.randint(128, longest), 256) for _ in range(64)]
    else:
        shapes = [(rng.randint(32, 128), 256) for _ in range(56)] + [(8192 - 16, 16) for _ in range(8)]   # 8192 positions each
    scheduler = Scheduler(engine.cache, max_tokens_per_step=budget, max_seqs_per_step=len(shapes), chunk_size=chunk,
                          max_positions=engine.spec.max_positions, eos_token_id=engine.spec.eos_token_id,
                          prompt_tokens_beside_decodes=prompt_cap)
    requests = [Request(id=(workload, index), prompt=torch.randint(0, vocab, (length,), generator=generator).tolist(),
                        params=SamplingParams(max_tokens=new)) for index, (length, new) in enumerate(shapes)]
    for request in requests:
        scheduler.add(request)
    pages = engine.cache.num_pages
    slices, peak_pages = [], 0
    torch.cuda.synchronize()
    started = time.perf_counter()
    while scheduler.has_work():
        before = (time.perf_counter(), scheduler.stats["prefill_tokens"])
        ran = engine.run(scheduler, max_steps=slice_steps)
        torch.cuda.synchronize()
        slices.append(((time.perf_counter() - before[0]) / max(ran, 1), scheduler.stats["prefill_tokens"] > before[1]))
        peak_pages = max(peak_pages, pages - min(engine.cache.free_pages()))
    elapsed = time.perf_counter() - started
    assert all(len(request.generated) == new for request, (_, new) in zip(requests, shapes))
    with_prompts = sorted(seconds for seconds, prompts in slices if prompts)
    decode_only = sorted(seconds for seconds, prompts in slices if not prompts)
    middle = lambda values: values[len(values) // 2] * 1e3 if values else None
    prompt_tokens, new_tokens = sum(length for length, _ in shapes), sum(new for _, new in shapes)
    return {"seconds": elapsed, "tokens": prompt_tokens + new_tokens, "generated": new_tokens,
            "steps": scheduler.stats["steps"], "preemptions": scheduler.stats["preemptions"],
            "peak_pages_frac": peak_pages / pages, "ms_step_with_prompts": middle(with_prompts),
            "ms_step_decode_only": middle(decode_only)}


# layer sizes for `--design fadutar`: TinyLlama's and Llama-3-8B's widths, heads and feed-forwards; the latent layers'
# rank and rotated part after the ratios of published latent-attention models, within the 256 value dims the
# plain attention kernel takes; the recurrence as wide as the model
DESIGN_SIZES = {
    "w2048": dict(width=2048, ff=5632, heads=32, kv_heads=4, dim=64, chunk=1024, latent_heads=32, latent_dim=64, latent_rot=32,
                  latent_vdim=64, rank=128, lru_width=2048, lru_blocks=8, taps=4, vocab=32000, groups=2),
    "w4096": dict(width=4096, ff=14336, heads=32, kv_heads=8, dim=128, chunk=1024, latent_heads=32, latent_dim=128, latent_rot=64,
                  latent_vdim=128, rank=192, lru_width=4096, lru_blocks=16, taps=4, vocab=32000, groups=1),
}


def design_configs(sizes):
    """(the Fadutar configuration, the Llama configuration of equal sizes): `groups` times the four kinds of layer
    (chunked attention, attention on that layer's keys and values, latent attention, recurrence), each with a
    feed-forward, beside as many Llama layers of the same width, heads and feed-forward."""
    s = sizes
    mlp = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
    attention = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5,
                 "mask": {"size": s["chunk"]}}
    layers = []
    for group in range(s["groups"]):
        layers += [
            {"type": "attention", "mixer": dict(attention), "mlp": mlp},
            {"type": "attention", "mixer": dict(attention, kv_from=4 * group), "mlp": mlp},
            {"type": "latent_attention", "mixer": {"heads": s["latent_heads"], "dim": s["latent_dim"], "rot_dim": s["latent_rot"],
                                                   "vdim": s["latent_vdim"], "kv_rank": s["rank"],
                                                   "scale": (s["latent_dim"] + s["latent_rot"]) ** -0.5,
                                                   "rot": {"base": 10000.0, "dims": s["latent_rot"]}}, "mlp": mlp},
            {"type": "rglru", "mixer": {"width": s["lru_width"], "blocks": s["lru_blocks"], "conv": s["taps"]}, "mlp": mlp},
        ]
    fadutar = {"architecture": "Fadutar", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["ff"], num_hidden_layers=len(layers),
                 num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], vocab_size=s["vocab"], max_position_embeddings=4096)
    return fadutar, llama


# layer sizes for `--design raketar`: the same widths, feed-forwards and vocabulary; differential attention with half as many
# heads of two maps each (so that its query heads are Llama's) and values twice as wide; memory heads after the ratios
# of published xLSTM models (query/key half as wide as the values); routed feed-forwards whose experts in use plus the
# shared one are as wide as the dense feed-forward; four layers of which the first two run twice (six runs)
RAKETAR_SIZES = {
    "w2048": dict(width=2048, ff=5632, heads=16, kv_heads=2, dim=64, vdim=128, memory_heads=8, memory_dim=128, memory_vdim=256,
                  experts=8, top=2, expert_ff=1408, shared_ff=2816, side=128, vocab=32000, llama_heads=32, llama_kv_heads=4),
    "w4096": dict(width=4096, ff=14336, heads=16, kv_heads=4, dim=128, vdim=256, memory_heads=8, memory_dim=256, memory_vdim=512,
                  experts=8, top=2, expert_ff=3584, shared_ff=7168, side=128, vocab=32000, llama_heads=32, llama_kv_heads=8),
}


def raketar_configs(sizes):
    """(the Raketar configuration, the Llama configuration of equal sizes): differential attention with a dense
    feed-forward, a memory layer with a routed one, differential attention with a routed one, a memory layer with a
    dense one; the first two run twice.  Beside as many Llama layers as that makes runs."""
    s = sizes
    dense = {"kind": "dense", "ff": s["ff"]}
    routed = {"kind": "moe", "expert": {"ff": s["expert_ff"]}, "router": {"experts": s["experts"], "top": s["top"]},
              "shared": {"ff": s["shared_ff"]}}
    attention = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["vdim"], "scale": s["dim"] ** -0.5,
                 "diff": 0.5, "rot": {"base": 10000.0, "dims": s["dim"], "scaling": {"factor": 2.0}}}
    memory = {"heads": s["memory_heads"], "dim": s["memory_dim"], "vdim": s["memory_vdim"], "gate_cap": 15.0}
    layers = [{"type": "attention", "mixer": attention, "mlp": dense}, {"type": "mlstm", "mixer": memory, "mlp": routed},
              {"type": "attention", "mixer": attention, "mlp": routed}, {"type": "mlstm", "mixer": memory, "mlp": dense}]
    raketar = {"architecture": "Raketar", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "residual_mult": 0.5,
               "token_side": {"dim": s["side"]}, "loop": {"start": 0, "stop": 2, "times": 2}, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["ff"], num_hidden_layers=6,
                 num_attention_heads=s["llama_heads"], num_key_value_heads=s["llama_kv_heads"], vocab_size=s["vocab"],
                 max_position_embeddings=4096)
    return raketar, llama


# layer sizes for `--design tugalix`: the same widths and vocabulary; retention and gated linear attention with heads whose
# query/key size is half their value size, after the ratios of published retention and gated-linear-attention models (keys
# half the width, values the width); attention beside token-shift mixing with Llama's heads on the left and heads of 64
# dims on the right, after published RWKV models; a decay rank of 64; four taps of the convolution; a feed-forward of two
# matrices at 1.5 times the gated one's inner size (equal weights) in two layers of four
TUGALIX_SIZES = {
    "w2048": dict(width=2048, ff=8448, llama_ff=5632, heads=32, kv_heads=4, dim=64, ret_heads=8, ret_dim=128, ret_vdim=256,
                  gla_heads=4, gla_dim=256, gla_vdim=512, shift_heads=32, shift_dim=64, rank=64, taps=4, vocab=32000),
    "w4096": dict(width=4096, ff=21504, llama_ff=14336, heads=32, kv_heads=8, dim=128, ret_heads=16, ret_dim=128, ret_vdim=256,
                  gla_heads=8, gla_dim=256, gla_vdim=512, shift_heads=64, shift_dim=64, rank=64, taps=4, vocab=32000),
}


def tugalix_configs(sizes):
    """(the Tugalix configuration, the Llama configuration of equal sizes): retention without a feed-forward, attention
    beside token-shift mixing with one, gated linear attention without, attention beside token-shift mixing with one.
    Beside four Llama layers of the same width and heads (a Llama layer always has its feed-forward)."""
    s = sizes
    dense = {"kind": "dense", "ff": s["ff"]}
    retention = {"heads": s["ret_heads"], "dim": s["ret_dim"], "vdim": s["ret_vdim"],
                 "decay": [1.0 - 2.0 ** (-5 - 3 * head / max(s["ret_heads"] - 1, 1)) for head in range(s["ret_heads"])],
                 "rot": {"base": 10000.0, "dims": s["ret_dim"]}}
    gla = {"heads": s["gla_heads"], "dim": s["gla_dim"], "vdim": s["gla_vdim"], "tau": 16.0, "rank": s["rank"]}
    side = {"left": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5,
                     "rot": {"base": 10000.0, "dims": s["dim"]}},
            "right": {"heads": s["shift_heads"], "dim": s["shift_dim"], "rank": s["rank"]}, "left_scale": 1.0, "right_scale": 1.0}
    layers = [{"type": "retention", "mixer": retention, "mlp": None}, {"type": "parallel", "mixer": side, "mlp": dense},
              {"type": "gla", "mixer": gla, "mlp": None}, {"type": "parallel", "mixer": side, "mlp": dense}]
    tugalix = {"architecture": "Tugalix", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "canon": {"taps": s["taps"]},
               "logit_scale": 1.0, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["llama_ff"], num_hidden_layers=4,
                 num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], vocab_size=s["vocab"], max_position_embeddings=4096)
    return tugalix, llama


# layer sizes for `--design narolorn`: the same widths and vocabulary; attention layers with Llama's heads; a latent vector of 128
# or 256 dims under as many heads; a routed feed-forward whose experts in use plus the shared one are as wide as the dense
# feed-forward; four streams of the residual; four layers of which the first two run twice (six runs)
NAROLORN_SIZES = {
    "w2048": dict(width=2048, ff=5632, vocab=32000, streams=4, heads=32, kv_heads=4, dim=64, softcap=50.0, chunk=1024, window=1024,
                  latent_heads=32, latent_dim=64, latent_vdim=64, rank=128, experts=8, top=2, expert_ff=1408, shared_ff=2816),
    "w4096": dict(width=4096, ff=14336, vocab=32000, streams=4, heads=32, kv_heads=8, dim=128, softcap=50.0, chunk=1024, window=1024,
                  latent_heads=32, latent_dim=128, latent_vdim=128, rank=256, experts=8, top=2, expert_ff=3584, shared_ff=7168),
}


def narolorn_configs(sizes):
    """(the Narolorn configuration, the Llama configuration of equal sizes): windowed latent attention, chunked attention
    whose values are its keys, attention with capped scores and a query temperature, latent attention again, each with a
    routed feed-forward; the first two run twice.  Beside as many Llama layers as that makes runs."""
    s = sizes
    routed = {"kind": "moe", "expert": {"ff": s["expert_ff"], "limit": 7.0}, "router": {"experts": s["experts"], "top": s["top"]},
              "shared": {"ff": s["shared_ff"], "limit": 7.0}}
    scale = s["dim"] ** -0.5
    latent = {"heads": s["latent_heads"], "dim": s["latent_dim"], "vdim": s["latent_vdim"], "kv_rank": s["rank"],
              "scale": s["latent_dim"] ** -0.5, "mask": {"size": s["window"]}}
    chunked = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": scale,
               "mask": {"size": s["chunk"]}, "rot": {"base": 10000.0, "dims": s["dim"]}}
    capped = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": scale, "softcap": s["softcap"],
              "q_temp": {"coef": 0.1, "every": 512}}
    layers = [{"type": "latent_attention", "mixer": latent, "mlp": routed}, {"type": "attention_2", "mixer": chunked, "mlp": routed},
              {"type": "attention", "mixer": capped, "mlp": routed}, {"type": "latent_attention", "mixer": latent, "mlp": routed}]
    narolorn = {"architecture": "Narolorn", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "streams": s["streams"],
                "logit_softcap": 30.0, "loop": {"start": 0, "stop": 2, "times": 2}, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["ff"], num_hidden_layers=6,
                 num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], vocab_size=s["vocab"], max_position_embeddings=4096)
    return narolorn, llama


# layer sizes for `--design paluzen`: the same widths and vocabulary; attention with Llama's heads over a window of 1024 beside
# heads of 64 dims as many as the width has; lightning attention with heads of 128 x 128 over the width; experts without a
# gate of which four in use have as many weights as Llama's feed-forward (two matrices of 1.5 times its inner size together),
# 14 of them beside 2 identities in 4 groups of which 3 stay; a dense feed-forward of the same weights; four layers of which
# the first two run twice (six runs)
PALUZEN_SIZES = {
    "w2048": dict(width=2048, ff=8448, llama_ff=5632, vocab=32000, heads=32, kv_heads=4, dim=64, window=1024, shift_heads=32, shift_dim=64,
                  light_heads=16, light_dim=128, light_vdim=128, experts=14, identity=2, groups=4, keep=3, top=4, expert_ff=2112, rank=16),
    "w4096": dict(width=4096, ff=21504, llama_ff=14336, vocab=32000, heads=32, kv_heads=8, dim=128, window=1024, shift_heads=64, shift_dim=64,
                  light_heads=32, light_dim=128, light_vdim=128, experts=14, identity=2, groups=4, keep=3, top=4, expert_ff=5376, rank=16),
}


def paluzen_configs(sizes):
    """(the Paluzen configuration, the Llama configuration of equal sizes): attention beside token-shift mixing with a dense
    feed-forward, lightning attention with a routed one, the two mixers again with routed ones; the first two run twice,
    each pass after its product with the embedding's output.  Beside as many Llama layers as that makes runs."""
    s = sizes
    dense = {"kind": "dense", "ff": s["ff"]}
    routed = {"kind": "moe", "expert": {"ff": s["expert_ff"]},
              "router": {"experts": s["experts"], "top": s["top"], "identity": s["identity"], "groups": {"count": s["groups"], "keep": s["keep"]}}}
    side = {"left": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5,
                     "mask": {"size": s["window"]}, "rot": {"base": 10000.0, "dims": s["dim"] // 2}},
            "right": {"heads": s["shift_heads"], "dim": s["shift_dim"]}, "left_scale": 1.0, "right_scale": 1.0}
    light = {"heads": s["light_heads"], "dim": s["light_dim"], "vdim": s["light_vdim"],
             "decay": [1.0 - 2.0 ** (-5 - 3 * head / max(s["light_heads"] - 1, 1)) for head in range(s["light_heads"])]}
    layers = [{"type": "parallel", "mixer": side, "mlp": dense}, {"type": "lightning", "mixer": light, "mlp": routed},
              {"type": "parallel", "mixer": side, "mlp": routed}, {"type": "lightning", "mixer": light, "mlp": routed}]
    paluzen = {"architecture": "Paluzen", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5}, "logit_softcap": 30.0,
               "loop": {"start": 0, "stop": 2, "times": 2}, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["llama_ff"], num_hidden_layers=6,
                 num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], vocab_size=s["vocab"], max_position_embeddings=4096)
    return paluzen, llama


# layer sizes for `--design barilix`: the same widths, feed-forwards and vocabulary; attention with Llama's heads over a window of
# 1024 beside a state-space side of twice the width in heads of 64 (state 128, as published models of the kind have it);
# delta-rule heads of 128 x 128 over the width, a query/key head for two; eight experts of a quarter of the feed-forward of
# which a token uses two, beside a shared one of half of it; four layers
BARILIX_SIZES = {
    "w2048": dict(width=2048, ff=5632, vocab=32000, heads=32, kv_heads=4, dim=64, window=1024, taps=4, space_heads=64, space_dim=64, space_state=128,
                  space_groups=1, delta_heads=16, delta_kv_heads=8, delta_dim=128, experts=8, top=2, expert_ff=1408, shared_ff=2816),
    "w4096": dict(width=4096, ff=14336, vocab=32000, heads=32, kv_heads=8, dim=128, window=1024, taps=4, space_heads=128, space_dim=64, space_state=128,
                  space_groups=8, delta_heads=32, delta_kv_heads=16, delta_dim=128, experts=8, top=2, expert_ff=3584, shared_ff=7168),
}


def barilix_configs(sizes):
    """(the Barilix configuration, the Llama configuration of equal sizes): attention beside a state-space mixer with a dense
    feed-forward, the delta rule with experts named by a table, and both with the other's feed-forward; beside four Llama layers."""
    s = sizes
    dense = {"kind": "dense", "ff": s["ff"]}
    routed = {"kind": "moe", "expert": {"ff": s["expert_ff"]}, "router": {"experts": s["experts"], "top": s["top"]}, "shared": {"ff": s["shared_ff"]}}
    side = {"left": {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "conv": s["taps"], "scale": s["dim"] ** -0.5,
                     "mask": {"size": s["window"]}, "rot": {"base": 500000.0, "dims": s["dim"],
                                                            "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}},
            "right": {"heads": s["space_heads"], "vdim": s["space_dim"], "state": s["space_state"], "groups": s["space_groups"],
                      "norm_groups": s["space_groups"], "conv": s["taps"]}}
    delta = {"heads": s["delta_heads"], "kv_heads": s["delta_kv_heads"], "dim": s["delta_dim"], "vdim": s["delta_dim"], "conv": s["taps"]}
    layers = [{"type": "parallel", "mixer": side, "mlp": dense}, {"type": "delta", "mixer": delta, "mlp": routed},
              {"type": "parallel", "mixer": side, "mlp": routed}, {"type": "delta", "mixer": delta, "mlp": dense}]
    barilix = {"architecture": "Barilix", "vocab": s["vocab"], "width": s["width"], "norm": {"eps": 1e-5},
               "embedding": {"scale": s["width"] ** 0.5}, "layers": layers}
    llama = dict(TINYLLAMA, hidden_size=s["width"], intermediate_size=s["ff"], num_hidden_layers=len(layers),
                 num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], vocab_size=s["vocab"], max_position_embeddings=4096)
    return barilix, llama


def bench_design(args, torch) -> int:
    """`--design fadutar|raketar|tugalix|narolorn|paluzen|barilix`: one JSON line.  Per size: tokens a second of a prompt step of 2048 tokens and of decode steps
    at the record's batch and context, for that decoder and for the Llama decoder of equal sizes (random
    weights, bfloat16, through the engine's own loop), and every kernel the design adds alone, beside the like kernel."""
    from tlie_amd import Engine, ops
    from tlie_amd.kernel_bench import (bench_barilix_kernels, bench_design_kernels, bench_narolorn_kernels, bench_paluzen_kernels,
                                       bench_raketar_kernels, bench_tugalix_kernels)
    peaks = ops.measured_peaks("cuda:0")
    record = {"metric": f"{args.design}: prefill and decode tok/s beside the Llama decoder of equal sizes", "unit": "tokens/s",
              "n_gpus": 1, "dtype": "bf16", "data": "synthetic: uniform random token ids, random weights",
              "batch": args.batch, "context": args.context, "measured_peaks": peaks, "sizes": {}}
    steps, warmup = min(args.steps, 48), 4
    all_sizes, configs, kernels = {"fadutar": (DESIGN_SIZES, design_configs, bench_design_kernels),
                                   "raketar": (RAKETAR_SIZES, raketar_configs, bench_raketar_kernels),
                                   "tugalix": (TUGALIX_SIZES, tugalix_configs, bench_tugalix_kernels),
                                   "narolorn": (NAROLORN_SIZES, narolorn_configs, bench_narolorn_kernels),
                                   "paluzen": (PALUZEN_SIZES, paluzen_configs, bench_paluzen_kernels),
                                   "barilix": (BARILIX_SIZES, barilix_configs, bench_barilix_kernels)}[args.design]
    for name, sizes in all_sizes.items():
        entry = {"layers": {"fadutar": 4 * sizes.get("groups", 0), "raketar": 6, "tugalix": 4, "narolorn": 6, "paluzen": 6, "barilix": 4}[args.design], "sizes": sizes}
        for model, config in zip((args.design, "llama"), configs(sizes)):
            engine = Engine(None, dtype="bfloat16", config=config, random_seed=0, max_tokens=args.batch * args.context + 4096,
                            page_size=16, max_requests=args.batch + 1)
            seconds = time_prefill(engine, torch, 2048, sizes["vocab"])
            entry[f"{model}_prefill_2048_tok_s"] = 2048 / seconds
            entry[f"{model}_prefill_2048_ms"] = seconds * 1e3
            seconds = sorted(time_decode(engine, torch, args.batch, args.context, steps, warmup, sizes["vocab"]) for _ in range(3))[1]
            entry[f"{model}_decode_tok_s"] = args.batch * steps / seconds
            entry[f"{model}_decode_ms_step"] = seconds / steps * 1e3
            del engine
            torch.cuda.empty_cache()
        if not args.no_points:
            entry["kernels"] = kernels(sizes, batch=args.batch, context=args.context, prompt=2048,
                                       hbm_gbs=peaks["stream_read_gbs"], mfma_tflops=peaks["mfma_bf16_tflops"])
        record["sizes"][name] = entry
    record["library_fallbacks"] = ops.library_fallbacks()
    print(json.dumps(record))
    return 0


def main() -> int:
    parser = argparse.ArgumentParser()
    parser.add_argument("--gpus", type=int, default=1)
    parser.add_argument("--steps", type=int, default=128)
    parser.add_argument("--warmup", type=int, default=8)
    parser.add_argument("--batch", type=int, default=8)
    parser.add_argument("--context", type=int, default=2048)
    parser.add_argument("--repeats", type=int, default=3,
                        help="the timed steps are run so many times, each after prompts and warm-up of its own; the median is reported")
    parser.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    parser.add_argument("--layers", type=int, default=0, help="run fewer layers than the configuration has (named in the record)")
    parser.add_argument("--no-points", action="store_true", help="skip batch 1 and 64 and the prefill")
    parser.add_argument("--prefill", type=int, default=0, metavar="TOKENS",
                        help="only a prompt step of TOKENS tokens, ten times (for profiles): prints its record alone")
    parser.add_argument("--workload", default="decode", choices=["decode", "serving", "mixed"],
                        help="serving: 64 requests with prompts of 128 to 2048 tokens and 256 decoded tokens each, batched "
                             "continuously; mixed: 8 prompts of 8192 tokens in portions beside 56 short decode streams "
                             "(needs a shape with 8192 positions); each prints a record of its own")
    parser.add_argument("--token-budget", type=int, default=2048, help="tokens a step of a workload may hold")
    parser.add_argument("--prompt-cap", type=int, default=0,
                        help="workloads: the most prompt tokens in a step that also holds decoding requests (0: what the budget leaves)")
    parser.add_argument("--kernels", nargs="?", const="", default=None, metavar="NAME",
                        help="time the kernels of a decode step (--batch, --context) and of a prompt step one by one at the "
                             "shape's layer sizes, each inside a replayed recording that walks through copies of its weights; "
                             "NAME keeps the kernels whose name holds it; prints one JSON line per kernel")
    parser.add_argument("--design", default=None, choices=["fadutar", "raketar", "tugalix", "narolorn", "paluzen", "barilix"],
                        help="prefill and decode throughput of that decoder design at layer sizes of real models, beside the Llama "
                             "decoder at equal sizes, and its own kernels alone beside the like kernels (one JSON line of its own)")
    parser.add_argument("--shape", default="tinyllama", choices=["tinyllama", *OTHER_SHAPES],
                        help="layer sizes of another model of the same architecture (the default is the record's)")
    args = parser.parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {args.gpus} is not supported (this engine runs on a single MI355X)")
        return 2
    import torch
    from tlie_amd import Engine
    if args.design:
        return bench_design(args, torch)
    cfg, model_name = dict(TINYLLAMA), "TinyLlama 1.1B shape"
    if args.shape != "tinyllama":
        model_name = OTHER_SHAPES[args.shape][0]
        cfg.update(OTHER_SHAPES[args.shape][1])
    full_layers = cfg["num_hidden_layers"]
    if args.layers:
        cfg["num_hidden_layers"] = args.layers
    if args.context > cfg["max_position_embeddings"] or args.steps + args.warmup >= args.context:
        print("context must fit the model's positions and exceed steps + warmup")
        return 2
    itemsize = 2 if args.dtype == "bfloat16" else 4
    vocab = cfg["vocab_size"]
    if args.kernels is not None:
        from tlie_amd.kernel_bench import bench_kernels
        for row in bench_kernels(cfg, batch=args.batch, context=args.context, prompt=args.prefill or 2048, only=args.kernels or None):
            print(json.dumps(row), flush=True)
        return 0
    if args.workload != "decode":
        if args.workload == "mixed" and cfg["max_position_embeddings"] < 8192:
            print("the mixed workload has prompts of 8192 tokens: take --shape llama3_8b")
            return 2
        live = 64 * (2048 + 256) if args.workload == "serving" else 8 * (8192 + 64) + 56 * (128 + 256 + 64)
        engine = Engine(None, dtype=args.dtype, config=cfg, random_seed=0, max_tokens=live, page_size=16, max_requests=65)
        chunk = None if args.workload == "serving" else 512
        cap = args.prompt_cap or None
        run_workload(engine, torch, args.workload, vocab, args.token_budget, chunk, prompt_cap=cap)   # warms up (recordings, plans)
        got = run_workload(engine, torch, args.workload, vocab, args.token_budget, chunk, prompt_cap=cap)
        print(json.dumps({"metric": f"total tok/s, {args.workload} workload ({model_name})", "value": got["tokens"] / got["seconds"],
                          "unit": "tokens/s", "generated_per_s": got["generated"] / got["seconds"], "seconds": got["seconds"],
                          "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "token_budget": args.token_budget,
                          "prompt_tokens_beside_decodes": args.prompt_cap or None,
                          "layers": cfg["num_hidden_layers"], "layers_of_model": full_layers,
                          **{key: got[key] for key in ("steps", "preemptions", "peak_pages_frac", "ms_step_with_prompts",
                                                       "ms_step_decode_only")}}))
        return 0
    if args.prefill:
        engine = Engine(None, dtype=args.dtype, config=cfg, random_seed=0, max_tokens=args.prefill + 2048, page_size=16, max_requests=2)
        seconds = time_prefill(engine, torch, args.prefill, vocab, repeats=10)
        print(json.dumps({"metric": f"prefill tok/s at {args.prefill} tokens ({model_name})", "value": args.prefill / seconds,
                          "unit": "tokens/s", "tokens": args.prefill, "ms": seconds * 1e3,
                          "frac": prefill_flops(cfg, args.prefill) / seconds / MFMA_PEAK[args.dtype]}))
        return 0
    most = max(args.batch, 1 if args.no_points else 64)
    started_all = time.perf_counter()
    engine = Engine(None, dtype=args.dtype, config=cfg, random_seed=0, max_tokens=most * args.context + 2048,
                    page_size=16, max_requests=most + 1)

    def median_decode(engine, batch, context, steps, warmup, vocab, repeats):
        """Seconds for `steps` timed decode steps: the median of `repeats` runs, each with its own
        prompts and `warmup` untimed steps before the timed ones."""
        runs = sorted(time_decode(engine, torch, batch, context, steps, warmup, vocab) for _ in range(repeats))
        return runs[len(runs) // 2]

    def step_bytes(cfg, itemsize, batch, context, steps):
        return weight_bytes_per_step(cfg, itemsize) + batch * (context - steps / 2) * kv_bytes_per_token(cfg, itemsize)

    elapsed = median_decode(engine, args.batch, args.context, args.steps, args.warmup, vocab, args.repeats)
    ms_per_step = elapsed / args.steps * 1e3
    value = args.batch * args.steps / elapsed
    achieved = step_bytes(cfg, itemsize, args.batch, args.context, args.steps) / (elapsed / args.steps)
    record = {
        "metric": f"decode tok/s at batch {args.batch}, context {args.context} ({model_name})", "value": value, "unit": "tokens/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "ms_per_step": ms_per_step, "higher_is_better": True,
        "scaling": "weak", "vs_baseline": None, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
        "data": "synthetic: uniform random token ids, random weights N(0, 0.02)",
        "repeats": args.repeats,            # the timed steps were run so many times, each after its own warm-up; the median counts
        "config": {"model": model_name, "layers": cfg["num_hidden_layers"], "layers_of_model": full_layers,
                   "hidden": cfg["hidden_size"], "heads": cfg["num_attention_heads"], "kv_heads": cfg["num_key_value_heads"],
                   "head_dim": cfg["hidden_size"] // cfg["num_attention_heads"], "ffn": cfg["intermediate_size"],
                   "vocab": vocab, "global_batch": args.batch, "seq_len": args.context, "page_size": 16,
                   "parallelism": "single GPU"},
        "roofline": {"bound": "hbm", "achieved": achieved / 1e9, "peak": HBM_PEAK / 1e9, "unit": "GB/s",
                     "frac": achieved / HBM_PEAK},
    }
    if not args.no_points:
        from tlie_amd import ops
        peaks = ops.measured_peaks(engine.device)
        record["measured_peaks"] = {"stream_read_gbs": peaks["stream_read_gbs"], "mfma_bf16_tflops": peaks["mfma_bf16_tflops"]}
        record["roofline"]["frac_of_measured"] = achieved / (peaks["stream_read_gbs"] * 1e9)
        prefill_tokens = 2048
        seconds = time_prefill(engine, torch, prefill_tokens, vocab)
        flops = prefill_flops(cfg, prefill_tokens)
        record["prefill"] = {"value": prefill_tokens / seconds, "tokens": prefill_tokens, "ms": seconds * 1e3,
                             "frac": flops / seconds / MFMA_PEAK[args.dtype]}
        if args.dtype == "bfloat16":
            record["prefill"]["frac_of_measured"] = flops / seconds / (peaks["mfma_bf16_tflops"] * 1e12)
        points = {}
        for batch in (1, 64):
            steps = min(args.steps, 64)
            seconds = median_decode(engine, batch, args.context, steps, 4, vocab, args.repeats)
            points[f"decode_b{batch}"] = batch * steps / seconds
            points[f"decode_b{batch}_frac"] = step_bytes(cfg, itemsize, batch, args.context, steps) / (seconds / steps) / HBM_PEAK
        # a short prompt: its step is replayed from a recording (the long one's is launched kernel by kernel)
        points["prefill_256"] = 256 / time_prefill(engine, torch, 256, vocab)
        # the workload of a prompt of 128 tokens and 128 generated ones, at the record's batch and at 1 and 64
        warm = 8
        timed = 128 - warm - 1
        for batch in sorted({args.batch, 1, 64}):
            seconds = median_decode(engine, batch, 256, timed, warm, vocab, args.repeats)
            points[f"decode_b{batch}_prompt128"] = batch * timed / seconds
            points[f"decode_b{batch}_prompt128_frac"] = step_bytes(cfg, itemsize, batch, 256, timed) / (seconds / timed) / HBM_PEAK
        del engine
        torch.cuda.empty_cache()
        if args.dtype == "bfloat16" and args.shape == "tinyllama":
            # the same model in true 32-bit (the check path): decoding at the record's batch and the prompt step
            wide = Engine(None, dtype="float32", config=cfg, random_seed=0, max_tokens=args.batch * args.context + 4096,
                          page_size=16, max_requests=args.batch + 1)
            steps = 24
            seconds = median_decode(wide, args.batch, args.context, steps, 2, vocab, args.repeats)
            points[f"fp32_decode_b{args.batch}"] = args.batch * steps / seconds
            points[f"fp32_decode_b{args.batch}_frac"] = step_bytes(cfg, 4, args.batch, args.context, steps) / (seconds / steps) / HBM_PEAK
            seconds = time_prefill(wide, torch, prefill_tokens, vocab, repeats=2)
            points["fp32_prefill_2048"] = prefill_tokens / seconds
            points["fp32_prefill_2048_frac"] = flops / seconds / MFMA_PEAK["float32"]
            del wide
            torch.cuda.empty_cache()
            # the layer sizes of the two larger models of the same architecture, a quarter of their layers
            # (named beside the number), decoding at the record's batch at 2048 positions
            for shape, (name, sizes) in OTHER_SHAPES.items():
                larger = dict(TINYLLAMA)
                larger.update(sizes)
                layers_of_model = larger["num_hidden_layers"]
                larger["num_hidden_layers"] = layers_of_model // 4
                other = Engine(None, dtype="bfloat16", config=larger, random_seed=0, max_tokens=args.batch * 2048 + 2048,
                               page_size=16, max_requests=args.batch + 1)
                steps = 32
                seconds = median_decode(other, args.batch, 2048, steps, 4, larger["vocab_size"], args.repeats)
                key = f"{shape}_decode_b{args.batch}"
                points[key] = args.batch * steps / seconds
                points[key + "_ms"] = seconds / steps * 1e3
                points[key + "_frac"] = step_bytes(larger, 2, args.batch, 2048, steps) / (seconds / steps) / HBM_PEAK
                points[key + "_layers"] = larger["num_hidden_layers"]
                points[key + "_layers_of_model"] = layers_of_model
                del other
                torch.cuda.empty_cache()
                # and that model's whole workload through the scheduler (the same number of layers): 64
                # requests served at once, or 8 long prompts in portions beside 56 short decode streams;
                # the second run is timed, the first makes the recordings
                workload, chunk = ("serving", None) if larger["max_position_embeddings"] < 8192 else ("mixed", 512)
                live = 64 * (2048 + 256) if workload == "serving" else 8 * (8192 + 64) + 56 * (128 + 256 + 64)
                other = Engine(None, dtype="bfloat16", config=larger, random_seed=0, max_tokens=live, page_size=16, max_requests=65)
                run_workload(other, torch, workload, larger["vocab_size"], 2048, chunk)
                got = run_workload(other, torch, workload, larger["vocab_size"], 2048, chunk)
                key = f"{shape}_{workload}"
                points[key + "_tok_s"] = got["tokens"] / got["seconds"]
                points[key + "_generated_tok_s"] = got["generated"] / got["seconds"]
                points[key + "_ms_step_with_prompts"] = got["ms_step_with_prompts"]
                points[key + "_ms_step_decode_only"] = got["ms_step_decode_only"]
                points[key + "_preemptions"] = got["preemptions"]
                if workload == "mixed":
                    # the other end of the trade: prompts get at most 256 tokens in a step that also decodes, so
                    # the 56 decoding streams wait less for each of their tokens and the long prompts take longer
                    run_workload(other, torch, workload, larger["vocab_size"], 2048, chunk, prompt_cap=256)
                    got = run_workload(other, torch, workload, larger["vocab_size"], 2048, chunk, prompt_cap=256)
                    points[key + "_cap256_tok_s"] = got["tokens"] / got["seconds"]
                    points[key + "_cap256_generated_tok_s"] = got["generated"] / got["seconds"]
                    points[key + "_cap256_ms_step_with_prompts"] = got["ms_step_with_prompts"]
                    # and decoding at the model's longest context, 8192 positions, at the record's batch
                    steps = 24
                    seconds = median_decode(other, args.batch, 8192, steps, 4, larger["vocab_size"], args.repeats)
                    points[f"{shape}_decode_b{args.batch}_ctx8192"] = args.batch * steps / seconds
                    points[f"{shape}_decode_b{args.batch}_ctx8192_frac"] = step_bytes(larger, 2, args.batch, 8192, steps) / (seconds / steps) / HBM_PEAK
                del other
                torch.cuda.empty_cache()
        record["points"] = points
        record["bench_seconds"] = time.perf_counter() - started_all
    from tlie_amd import ops as kernel_faces
    # products of many rows that fell from the vendor's library to the plain 32-bit kernel (each many
    # times slower): a record measured with any would not be this engine's speed
    record["library_fallbacks"] = kernel_faces.library_fallbacks()
    assert record["library_fallbacks"] == 0, f"{record['library_fallbacks']} matrix products took the plain kernel instead of the library's"
    print(json.dumps(record))
    return 0


if __name__ == "__main__":
    sys.exit(main())
