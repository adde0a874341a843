// Described decoders: a language model whose layers are listed at run time (cr_lm_configure) instead of being compiled in.  Every size and constant comes from the
// description; the mechanisms below (latent attention, attention over grouped heads with chunks and capped scores, retention, clamped gated experts behind a grouped router,
// dense feed-forwards, a residual stream in fp32 with or without norms behind a sublayer, layer spans that run several times, token inputs per layer) are each a kernel
// family of their own with those constants as parameters.
#pragma once
#include <memory>
#include <string>
#include <vector>

#include "attention.hpp"
#include "common.hpp"
#include "ctx.hpp"

inline int lm_pad64(int n) { return (n + 63) / 64 * 64; }

// a per-head size padded to the next power of two from 64 on: a head's rows never straddle a wave's 512 columns in the row kernels
inline int lm_pad_head(int n) { int p = 64; while (p < n) p *= 2; return p; }
constexpr int LM_MAX_HEAD = 512;

// Rows of the fused input projection of a layer with attention over heads and / or retention: one region per projection, widest heads first (a head starts at a multiple of its
// padded size).
enum LmRegionKind { LM_Q, LM_K, LM_V, LM_RQ, LM_RK, LM_RV, LM_RG };
struct LmRegion { int kind, off, heads, P; };      // columns [off, off + heads * P)
constexpr int LM_REGIONS = 7;

// One layer: the description, the padded sizes (every contraction length is a multiple of 64 with zero weights behind the real ones) and the derived tensors.
struct LmLayer {
    cr_lm_layer s;
    int Qp, Rp, Ap, Gp;        // padded q_rank, kv_rank (the cache row), per-head query / key / value size, width of the output projection's input
    int off_c, off_g, Na;      // columns of the latent and of the output gate in the fused down projection [dq | dkv | g], and its width
    int ffp, Ep;
    // attention over heads / retention: padded per-head sizes of retention (Ap is attention's), regions, where retention's columns start in the output projection's input,
    // which of the model's distinct chunk sizes this layer has
    int Kp, Vp, n_regions, off_r, chunk_ix;
    LmRegion regions[LM_REGIONS];
    std::vector<double> decay;
    // element type of the model (bf16 or float)
    void *wa, *wuq, *wkv, *wukT, *wo, *router, *wgu, *wdn;      // (wgu, wdn: fragment-ordered blocks for bf16, rows for float; dense feed-forward: up and down in rows)
    void *sgate, *sproj;
    bf16 *wa_dl, *wuq_dl, *wo_dl, *wgu_dl, *wdn_dl, *sgate_dl, *sproj_dl;      // bf16: decode-layout copies for the weight-streaming kernels (gemm_skinny.hip), may be null
    // fp32: gains (one plus the stored weight for the norms about zero), router correction
    float *n1, *n1b, *n2, *n2b, *nq, *nc, *corr, *ns;
    float *fq_a, *fq_r;        // rotation frequencies of attention and of retention
    float *pw;                 // retention: decay^0 .. decay^RET_CHUNK of every head

    const LmRegion* region(int kind) const {
        for (int i = 0; i < n_regions; i++) if (regions[i].kind == kind) return regions + i;
        return nullptr;
    }
    bool latent() const { return s.mixer == CR_MIX_LATENT; }
    bool heads() const { return (s.mixer & CR_MIX_HEADS) != 0; }
    bool retention() const { return (s.mixer & CR_MIX_RETENTION) != 0; }
};

struct Lm {
    cr_lm_desc d;
    std::vector<LmLayer> layers;
    std::vector<int> passes;   // layer index of every layer pass (the looped span unrolled)
    std::vector<char> starts;  // per pass: a pass of the looped span begins here and the model mixes the embedding in first (loop_in)
    std::vector<int> chunks;   // distinct chunk sizes of attention over heads (INT32_MAX: no chunks)
    int Wp = 0, Vp = 0, Sp = 0;      // padded width, vocabulary, side input
    bool f32 = false;
    void *embed = nullptr, *head = nullptr, *side = nullptr, *loop_in = nullptr;
    bf16 *head_dl = nullptr, *loop_dl = nullptr;
    float *fin = nullptr, *freq = nullptr;
    float gain_base() const { return d.norm_plain ? 0.f : 1.f; }
    size_t esz() const { return f32 ? 4 : 2; }
};

// ---- matrix products (lm_gemm.hip): C = epi(A . W^T), K % 64 == 0, optionally batched over heads or grouped over experts ----
enum LmEpi {
    LM_STORE = 0,      // element type
    LM_RAW32 = 1,      // fp32, the accumulator itself; softcap > 0: softcap * tanh(acc / softcap)
    LM_GLU = 2,        // rows of W interleaved [8 gate | 8 up]: g = min(gate, limit), u = clamp(up, -limit, limit); g * sigmoid(1.702 g) * (u + 1)
    LM_GATE = 3,       // acc * sigmoid(gate[m][n])
    LM_RELU2 = 4,      // max(acc, 0)^2
    LM_SIDE = 5,       // gelu_tanh(acc) * gate[tok[m]][n]
};
struct LmGemmParams {
    const void* A; int64_t lda;
    const void* W; int64_t ldw;
    void* C; int64_t ldc;
    int M, N, K;
    int batch; int64_t a_bs, w_bs, c_bs, g_bs;      // heads: blockIdx.z, strides in elements
    const int4* tiles; const int32_t* n_tiles; int max_tiles;      // experts: {expert, first sorted position, rows, -}; W of an expert at + expert * w_bs
    const int32_t* perm; int gather_div, scatter;   // row of A = perm[pos] / gather_div (0: pos); row of C = perm[pos] when scatter
    float softcap, limit;
    const void* gate; int64_t ldg;
    const int32_t* tok;
};
int launch_lm_gemm(bool f32, int epi, const LmGemmParams& p, hipStream_t st);
constexpr int LM_TILE_M = 64;

// ---- rows (lm_rows.hip): one workgroup per token ----
struct LmRowIndex {            // where a row's token sits: prefill gives arrays, decode reads the cache's own lengths
    const int32_t *row_seq, *row_pos;      // prefill
    const int32_t *seqs, *lens;            // decode: seq = seqs[row], pos = lens[seq]
};
// where a row of the residual goes for its next reader, in the element type: rms(x) * gain, or with a null gain x itself
struct LmSink { void* h; int64_t ldh; const float* gain; };
// x = embed[token] + sinusoid(pos), then the sink.  token = tokens[row], or the last generated id of the row's sequence; also written to tok[row], and the row as it is to
// x0 (rows ldx0 apart) when given
int launch_lm_embed(bool f32, const Lm& lm, int M, const int64_t* tokens, const LmRowIndex& ix, const int64_t* gen, const int32_t* ngen, int gen_cap,
                    float* x, const LmSink& to, int32_t* tok, void* x0, int64_t ldx0, hipStream_t st);
// what a sublayer left for a row: one row of Y in the element type (fp32 rows: slices = 1); with `slices` the sum of fp32 K-slices Y [slices][M][ldy]; with `top` the weighted
// sum of the row's expert rows
struct LmPostIn { const void* Y; int64_t ldy; int slices; const float* wt; int top; };
// x += gain_b ? rms(y) * gain_b : y (x = y with `replace`), then the sink (h may be null)
int launch_lm_post(bool f32, const Lm& lm, int M, const LmPostIn& in, float* x, const float* gain_b, bool replace, const LmSink& to, hipStream_t st);
// h[i] = rms(x[rows[i]]) * gain
int launch_lm_pick_rows(bool f32, const Lm& lm, int n, const float* x, const int32_t* rows, void* h, const float* gain, hipStream_t st);
// the down projection (rows `a`, or fp32 K-slices `part` [slices][M][Na]: then the gate's columns are also written to `a`) -> its two latents: cq = rms(a[0 .. q_rank)) * nq; c = rms(a[off_c .. + kv_rank)) * nc -> the cache row and (prefill) a dense copy
int launch_lm_latents(bool f32, const Lm& lm, const LmLayer& L, int M, void* a, const float* part, int slices, void* cq, void* c_dense, void* cache, int max_tokens, const LmRowIndex& ix, void* ao, hipStream_t st);

// ---- routing (moe.hip) ----
// z [slices][M][ldz] fp32 (summed in slice order) -> idx [M][top], wt [M][top]
int launch_lm_route(const LmLayer& L, int M, const float* z, int64_t ldz, int slices, int32_t* idx, float* wt, hipStream_t st);
// assignments sorted by expert: perm[pos] = row * top + slot, tiles of at most tile_m positions
int launch_lm_plan(const LmLayer& L, int M, int tile_m, const int32_t* idx, int32_t* perm, int4* tiles, int32_t* n_tiles, hipStream_t st);
inline int lm_max_tiles(int rows, int experts, int tile_m) { return rows / tile_m + (experts < rows ? experts : rows); }

// router product + routing in one kernel (bf16): z = h . router^T accumulated in fp32 and kept on the chip
bool lm_router_supported(const LmLayer& L);
int launch_lm_router(const Lm& lm, const LmLayer& L, int M, const void* h, int32_t* idx, float* wt, float* part, hipStream_t st);
constexpr int LM_ROUTER_SLICES = 16;          // few rows: K-slices of the router product in `part` [slices][M][Ep], summed by the routing kernel

// ---- expert products in bf16 (moe_gemm.hip) ----
constexpr int MOE_TILE_M = 128, MOE_STREAM_ROWS = 64;
struct MoeGemmParams {
    const bf16* A; int64_t lda;
    const bf16* W; int64_t w_es;                    // fragment-ordered blocks, elements per expert
    bf16* C; int64_t ldc;
    int N, K;
    const int4* tiles; const int32_t* n_tiles; int max_tiles; const int32_t* perm; int scatter;       // tiled form (lm_plan_kernel with MOE_TILE_M)
    bool grouped256;                                // tiled form: tiles of 256 positions through gemm256.hip
    int gather_div;                                 // row of A: tiled: perm[pos] / gather_div (0: pos); stream: assignment / gather_div (0: assignment)
    const int32_t* idx; int M, top, experts;        // stream form: routing table [M][top]
    float limit;
};
bool moe_grouped256(int M, int top, int experts, int N, int K);
int launch_moe_tiled(bool glu_epi, const MoeGemmParams& p, hipStream_t st);
int launch_moe_stream(bool glu_epi, const MoeGemmParams& p, hipStream_t st);

// ---- latent attention (attention_latent.hip) ----
struct LatentAttnParams {
    const void* Q;             // [M][heads][Rp]: the queries carried into the latent space
    const void* C;             // this pass's cache [n_seqs][max_tokens][Rp]
    void* O;                   // [M][heads][Rp]
    int M, H, Rp, max_tokens;
    float scale;
    LmRowIndex ix;
};
int launch_latent_attn_plain(bool f32, const LatentAttnParams& p, hipStream_t st);
// bf16 decode: splits of LATENT_SPLIT keys on the matrix cores, then one kernel per head that merges them, carries the result back by W_uv and applies the output gate
constexpr int LATENT_TILE = 32;
struct LatentDecodeParams {
    LatentAttnParams a;        // a.O unused
    int nsplit, split;         // splits of the longest row, keys per split (a multiple of LATENT_TILE)
    float *part_o, *part_ml;   // [M][H][nsplit][Rp], [M][H][nsplit][2]
    const bf16* wuv;           // head h at + h * uv_hs: [vdim][Rp]
    int64_t uv_hs; int vdim;
    const bf16* gate; int64_t ldg;
    bf16* out; int64_t ldo;    // [M][heads * vdim]
};
bool latent_decode_supported(int Rp);
inline size_t latent_part_floats(int M, int H, int nsplit, int Rp) { return (size_t)M * H * nsplit * (Rp + 2); }
int latent_split_keys(int heads, int64_t keys);      // keys per split of a batch that holds `keys` cached tokens in all
int launch_latent_decode(const LatentDecodeParams& p, hipStream_t st);
// few rows: q (fp32 K-slices [slices][M][heads * Ap]) carried into the latent space, out [M][heads][Rp]
int launch_latent_absorb(const LmLayer& L, int M, const float* part, int slices, void* out, hipStream_t st);

// ---- attention over heads and retention: the fused projection's rows (lm_heads.hip) ----
// key rows of a prompt: kv [Mk][2 * kv_heads * Ap] (keys, then values); cache: K and V [n_seqs][kv_heads][ring][Ap] each, position p in row p % chunk
struct LmHeadsIn {
    const void* a; int64_t lda;            // projection rows, or
    const float* part; int slices;         //   fp32 K-slices [slices][M][Na] of it (decode): retention's v and g are then written to `a` too
    LmRowIndex ix;
    void *q, *kv, *cache_k, *cache_v;      // attention; kv null in decode
    int ring, chunk;
    const int32_t *row_key, *row_slot;     // prompts: a row's key row, its cache row (sequence * ring + place) or -1
    float *rq, *rk;                        // retention, one of the two forms: fp32 [M][heads * Kp], or
    bf16 *rq2, *rk2;                       //   two bf16 terms [2][M][heads * Kp]
    void* ao;                              // output projection's input: its padding columns are zeroed
};
int launch_lm_heads(bool f32, const Lm& lm, const LmLayer& L, int M, const LmHeadsIn& in, hipStream_t st);
// cached key and value rows of the chunk a portion goes on in, into the prompt's key rows: (key row, cache row) pairs
int launch_lm_prefix(bool f32, const LmLayer& L, int n, const int32_t* key_rows, const int32_t* cache_rows, void* kv, const void* cache_k, const void* cache_v, int ring, hipStream_t st);
// softmax attention for any size and type: one workgroup per query row and head, keys from `first` on
struct HeadsAttnParams {
    const void *Q, *K, *V; void* O;        // Q [M][heads * Ap], O rows ldo apart
    int64_t k_rs, k_hs, ldo;               // elements between key rows and between key heads
    int M, H, G, Ap, vdim, chunk, ring;
    float scale, softcap, out_scale;
    const int32_t* row_key;                // prompts: key row of the query itself; null: the cache
    LmRowIndex ix;
};
int launch_heads_attn_plain(bool f32, const HeadsAttnParams& p, hipStream_t st);

// ---- retention (retention.hip) ----
// state of a (sequence, head): fp32 [Vp / 16][Kp / 16][64][4]: 16 value columns a block, lane = (dk / (Kp / 16)) * 4 + column quad, element dk % (Kp / 16) outermost (ret_state_at)
constexpr int RET_CHUNK = 256;
struct RetParams {
    const float *rq, *rk; const bf16 *rq2, *rk2;      // LmHeadsIn's
    const void *v, *g; int64_t lda;                   // columns of the projection rows
    void* ao; int64_t ldo;                            // out: head h at column h * vdim
    float* state;                                     // this pass's states [n_seqs][heads][Vp * Kp]
    float* raw;                                       // prompts, recurrent form: [M][heads * Vp]
    bf16* snap;                                       // prompts, matrix form: what every chunk adds, then the state ahead of it [chunks][heads][Vp * Kp * 4 bytes]
    const float* pw;                                  // [heads][RET_CHUNK + 1]
    int M, H, Kp, Vp, vdim;
    float eps, out_scale;
    LmRowIndex ix;
    const int32_t* seg; const int32_t* snap0; int n_segs, longest;      // prompts: {first row, rows, first position, sequence} per segment, its first chunk
    const int32_t* chunks; int n_chunks;              // prompts, matrix form: {first row, rows} of every chunk of RET_CHUNK rows
};
bool ret_matrix_supported(int Kp, int Vp);
inline int ret_chunks(int rows) { return (rows + RET_CHUNK - 1) / RET_CHUNK; }
// merge: decode splits that the attention beside it left (AttnParams::no_merge), of heads of merge_dim columns
int launch_ret_decode(bool f32, const RetParams& p, const AttnParams* merge, int merge_dim, hipStream_t st);
int launch_ret_recurrent(bool f32, const RetParams& p, hipStream_t st);
int launch_ret_matrix(const RetParams& p, hipStream_t st);
// decode of <= 64 rows: z[m][n] = gelu_tanh(sum of K-slices) * side[tok[m]][n]
int launch_lm_side_act(const Lm& lm, int M, const float* part, int slices, const void* side, int64_t lds, const int32_t* tok, void* z, hipStream_t st);
// ... and y [M][Wp] = z . W^T in the same launch (few rows)
bool lm_side_proj_supported(const Lm& lm, int M);
int launch_lm_side_proj(const Lm& lm, int M, const float* part, int slices, const void* side, int64_t lds, const int32_t* tok, const void* W, void* y, hipStream_t st);

int lm_finalize(cr_ctx* c, hipStream_t st);
struct cr_kv;
int lm_kv_alloc(const Lm& lm, cr_kv* kv);
int lm_decode_step(cr_ctx* c, cr_kv* kv, int n, const int64_t* force_tokens, float penalty, float* logits, hipStream_t st);
