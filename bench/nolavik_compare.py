"""Prefill and decode throughput of the Nolavik design beside the closest uniform family (Llama: sequential pre-norm
blocks, RMS norm, rotary grouped-query attention, gated feed-forward) at equal size, random weights, through the serving
engine (scheduler, paged cache, state slots, decode graphs, sampler). Run as ``python bench.py --nolavik [SIZE,...]``.

Nolavik: four layers - gated delta rule, attention beside a selective scan, latent attention, gated delta rule - each with
experts and a gated shared expert; the first two are a repeated stretch of one pass (its vector is added, nothing runs
twice). "Equal size": same width, vocabulary and number of layer runs, the attention's heads, key/value heads and head size;
the dense family's gated feed-forward is as wide as what a Nolavik token touches (top x expert ff + shared ff).
"""
from __future__ import annotations

import torch

from timisun_compare import measure

SIZES = {
    # width; attention heads / key heads / head size; scan channels x state, step rank; delta heads / key heads x key size x
    # value size; latent heads = attention heads, rotated part, query rank, latent rank; experts / top / expert ff / shared ff
    "w1024": dict(width=1024, heads=8, kv=2, dim=128, inner=2048, state=16, dtr=64, dheads=8, dkv=4, ddim=128, dvdim=128,
                  rot=64, qrank=384, krank=192, experts=16, top=2, eff=512, sff=512, vocab=32000),
    "w2048": dict(width=2048, heads=16, kv=4, dim=128, inner=4096, state=16, dtr=128, dheads=16, dkv=8, ddim=128, dvdim=128,
                  rot=64, qrank=768, krank=192, experts=32, top=4, eff=768, sff=768, vocab=32000),
    "w4096": dict(width=4096, heads=32, kv=8, dim=128, inner=8192, state=16, dtr=256, dheads=32, dkv=16, ddim=128, dvdim=128,
                  rot=64, qrank=1536, krank=192, experts=32, top=4, eff=1536, sff=1536, vocab=32000),
}
LAYERS = 4


def nolavik_dict(s):
    moe = dict(kind="moe", router=dict(experts=s["experts"], top=s["top"]), expert=dict(ff=s["eff"]), shared=dict(ff=s["sff"]))
    delta = dict(type="delta", mlp=moe,
                 mixer=dict(heads=s["dheads"], kv_heads=s["dkv"], dim=s["ddim"], vdim=s["dvdim"], conv=4))
    left = dict(heads=s["heads"], kv_heads=s["kv"], dim=s["dim"], vdim=s["dim"], scale=s["dim"] ** -0.5,
                rot=dict(base=500000.0, dims=s["dim"], scaling=dict(factor=8.0, low=1.0, high=4.0, original=8192)))
    par = dict(type="parallel", mlp=moe,
               mixer=dict(left=left, right=dict(inner=s["inner"], state=s["state"], dt_rank=s["dtr"], conv=4), left_scale=0.7,
                          right_scale=0.6))
    lat = dict(type="latent_attention", mlp=moe,
               mixer=dict(heads=s["heads"], dim=s["dim"], rot_dim=s["rot"], vdim=s["dim"], q_rank=s["qrank"], kv_rank=s["krank"],
                          scale=(s["dim"] + s["rot"]) ** -0.5, rot=dict(base=10000.0, dims=s["rot"])))
    return dict(architecture="Nolavik", vocab=s["vocab"], width=s["width"], norm=dict(eps=1e-6),
                loop=dict(start=0, stop=2, times=1), layers=[delta, par, lat, delta])


def dense_ff(s):
    return (s["top"] * s["eff"] + s["sff"]) // 64 * 64


def build(kind, s, dev):
    from llmss_amd.models.config import ModelConfig, get_preset
    from llmss_amd.models.layered import create_model
    from llmss_amd.models.weights import random_nolavik_weights, random_weights

    if kind == "nolavik":
        cfg = ModelConfig.from_hf_dict(nolavik_dict(s))
        return create_model(cfg, random_nolavik_weights(cfg, device=dev, dtype=torch.bfloat16, seed=1))
    cfg = get_preset("llama2-7b", hidden_size=s["width"], num_layers=LAYERS, num_heads=s["heads"],
                     num_kv_heads=s["kv"], head_dim=s["dim"], intermediate_size=dense_ff(s), vocab_size=s["vocab"],
                     max_position_embeddings=8192, rotary_dim=s["dim"])
    return create_model(cfg, random_weights(cfg, device=dev, dtype=torch.bfloat16, seed=1))


def run(sizes, batch, prompt_len, gen_len, rounds, progress, kinds=("nolavik", "dense")):
    dev = torch.device("cuda", torch.cuda.current_device())
    rows = []
    for name in sizes:
        s = SIZES[name]
        row = dict(size=name, shape=s, batch=batch, prompt_len=prompt_len, gen_len=gen_len)
        for kind in kinds:
            progress(f"{name} {kind}: building")
            model = build(kind, s, dev)
            row[kind] = measure(model, batch, prompt_len, gen_len, rounds, progress)
            row[kind]["params_M"] = round(model.cfg.num_params() / 1e6, 1)
            del model
            torch.cuda.empty_cache()
        if "nolavik" in row and "dense" in row:
            row["prefill_ratio"] = round(row["nolavik"]["prefill_tok_s"] / row["dense"]["prefill_tok_s"], 3)
            row["decode_ratio"] = round(row["nolavik"]["decode_tok_s"] / row["dense"]["decode_tok_s"], 3)
        rows.append(row)
    return dict(metric="nolavik_vs_dense_tokens_per_sec", unit="tokens/s", dtype="bf16", data="synthetic",
                sizes=rows)
