// The cache object behind cr_kv: per-sequence bookkeeping (tokens cached, ids generated) that every language model shares, and the model's own cached state --
// K / V rows of InternLM2's 8 KV heads, or, for a described decoder (lm.hpp), one latent row per token and layer pass.
#pragma once
#include <vector>

#include "ctx.hpp"

struct cr_kv {
    cr_ctx* ctx;
    int n_seqs, max_tokens, gen_cap, layers;
    bf16* k;             // [layers][n_seqs][8][max_tokens][128]
    bf16* v;
    // described decoders: what layer pass r keeps starts at lat + lat_off[r] bytes: latent rows [n_seqs][max_tokens][padded kv_rank] in the model's element type, or keys and values
    // [2][n_seqs][kv_heads][ring][padded head] (ring = the rows a chunk needs); retention's fp32 states [n_seqs][heads][..] at lat + state_off[r]
    char* lat;
    std::vector<size_t> lat_off, state_off;
    int32_t* d_len;      // [n_seqs] tokens cached
    int32_t* d_ngen;     // [n_seqs] ids generated
    int64_t* d_gen;      // [n_seqs][gen_cap]
    int32_t* d_seqs;     // [n_seqs] staging for the seqs[] of one decode call
    std::vector<int32_t> seqs_on_device;   // what d_seqs holds (decode skips the host-to-device copy of an unchanged list: a pageable copy
                                           // makes the host wait for the stream, which stops it from feeding a second stream)
    std::vector<int> len, ngen;
    // batched decode as a hipGraph (CR_DECODE_GRAPH=1): a step is ~290 short launches whose parameters only change with
    // the row count and the number of attention splits (positions, ids and cache lengths live in device memory), so the
    // launch sequence is captured once per (rows, splits, penalty) and replayed.  OFF by default: on ROCm 7.2 / MI355X the
    // replay measured 0.3 % slower than plain launches at 64 pages per step (6.86 vs 6.88 pages/s) and 5 % slower for a
    // single page (0.711 vs 0.678 s) -- the ~3 us gaps between dependent kernels are not launch overhead the graph removes
    struct DecodeGraph { int n, nsplit; float penalty; char* ws; uint64_t weight_gen; hipGraphExec_t exec; int warm; };
    std::vector<DecodeGraph> graphs;
};

// repetition penalty + argmax + append, one row per sequence seqs[row] (llm.hip); len_add: tokens the step added to the cache length
int launch_pick(float* logits, int64_t ld, int vocab, float penalty, int n, const int32_t* seqs, cr_kv* kv, int len_add, hipStream_t st);
