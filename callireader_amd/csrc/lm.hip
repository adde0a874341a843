// Described decoders: configuration, derived weights, the layer loop, and the step the shared entry points (llm.hip: prefill, decode) run.
//
// Per layer pass (x = fp32 residual, h / a / q / ... in the model's element type):
//   [x += rms(y) * g, h = rms(x) * g']  ->  a = h . [dq | dkv | g]^T  ->  cq, c (-> cache)  ->  q = cq . W_uq^T
//   -> latent attention, gated -> y = ao . W_o^T -> [x += rms(y) * g, h = rms(x) * g'] -> routing -> expert products -> the next pass's first bracket sums the experts.
// Attention takes one of two forms of the same sum.  EXPANDED (bf16 prompts): k and v of every key are formed by one product and the flash kernel runs over them.
// ABSORBED (decode, fp32, sizes the flash kernel has no instance for): q is carried into the latent space per head and the cached rows serve as key and value of every head.
//
// Layers with attention over heads and / or retention have one fused projection too ([q | k | v | rq | rk | rv | rg], widest heads first) and one output projection whose input is
// the concatenation of both mixers' results, already scaled: side by side costs no launch of its own.  A chunked layer's cache is a ring of one chunk; a prompt's key rows are laid
// out portion by portion with the cached start of the chunk in front (KeyPlan), so that a chunk is a plain causal segment to the attention kernels.
#include <math.h>
#include <string.h>

#include <algorithm>

#include <stdlib.h>

#include "attention.hpp"
#include "decode.hpp"
#include "kv.hpp"
#include "lm.hpp"

bool gemm_stream_supported(int epi, const GemmParams& p, int splits);      // gemm_stream.hip

namespace {

// Re-laid-out, padded, converted copies of checkpoint tensors (load time): src row r goes to row d = r, or to row 16 (r / 8) + r % 8 + row_off when interleaved in eights;
// element c of it to dst[d * rs + c * cs], or to its place in the 1-KiB fragment blocks of moe_gemm.hip when frag_k (= K / 32) is given.
// With `group` columns come in groups of that many, `group_to` apart in the copy.
struct Place { int64_t rs, cs; int interleave8, row_off, frag_k, group, group_to; };
template <typename T>
__global__ __launch_bounds__(256) void lm_place_kernel(const bf16* __restrict__ src, int64_t lds, int cols, T* __restrict__ dst, const Place w) {
    const int r = blockIdx.x;
    const int64_t d = w.interleave8 ? (int64_t)(r / 8) * 16 + (r % 8) + w.row_off : r;
    for (int c = threadIdx.x; c < cols; c += 256) {
        const int64_t at = w.frag_k ? ((d / 16) * w.frag_k + c / 32) * 512 + (c % 32) / 8 * 128 + (d % 16) * 8 + c % 8 : w.group ? d * w.rs + c / w.group * w.group_to + c % w.group : d * w.rs + c * w.cs;
        dst[at] = (T)bf2f(src[r * lds + c]);
    }
}
__global__ __launch_bounds__(256) void lm_gain_kernel(const bf16* __restrict__ src, int n, float base, float* __restrict__ dst) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i < n) dst[i] = base + bf2f(src[i]);
}

struct Deriver {
    cr_ctx* c; Lm& lm; hipStream_t st;
    std::vector<std::string> used;        // checkpoint tensors that went into a derived one

    bool has(const std::string& n) const { return c->w.count(n) != 0; }
    const DevTensor* src(const std::string& n, int64_t rows, int64_t cols) {
        const DevTensor* t = WT(c, n);
        if (!t) return nullptr;
        const bool ok = cols ? t->shape.size() == 2 && t->shape[0] == rows && t->shape[1] == cols : t->numel() == rows;
        if (!ok || t->dtype != CR_BF16) { cr_fail(CR_ERR_ARG, "%s: expected bf16 [%lld%s%lld]", n.c_str(), (long long)rows, cols ? ", " : "", (long long)cols); return nullptr; }
        used.push_back(n);
        return t;
    }
    void* make(const std::string& n, size_t elems, size_t es, int dtype) {
        auto old = c->w.find(n);
        if (old != c->w.end()) { hipFree(old->second.ptr); c->w.erase(old); }
        DevTensor t;
        t.dtype = dtype; t.shape = {(int64_t)elems}; t.bytes = elems * es;
        if (hipMalloc(&t.ptr, std::max<size_t>(t.bytes, 256)) != hipSuccess) { cr_fail(CR_ERR_NOMEM, "%s: %zu bytes", n.c_str(), t.bytes); return nullptr; }
        if (hipMemsetAsync(t.ptr, 0, t.bytes, st) != hipSuccess) { cr_fail(CR_ERR_HIP, "%s", n.c_str()); return nullptr; }
        c->w[n] = t;
        return t.ptr;
    }
    void* mat(const std::string& n, size_t elems) { return make(n, elems, lm.esz(), lm.f32 ? CR_F32 : CR_BF16); }
    // rows [r0, r0 + rows) of checkpoint tensor t into dst + off (elements)
    int place(const DevTensor* t, int64_t r0, int rows, void* dst, size_t off, const Place& w) {
        const int cols = (int)t->shape[1];
        const bf16* s = (const bf16*)t->ptr + r0 * cols;
        if (lm.f32) hipLaunchKernelGGL(lm_place_kernel<float>, dim3(rows), dim3(256), 0, st, s, (int64_t)cols, cols, (float*)dst + off, w);
        else hipLaunchKernelGGL(lm_place_kernel<bf16>, dim3(rows), dim3(256), 0, st, s, (int64_t)cols, cols, (bf16*)dst + off, w);
        return hipGetLastError() == hipSuccess ? CR_OK : cr_fail(CR_ERR_HIP, "lm_place");
    }
    int place(const DevTensor* t, int64_t r0, int rows, void* dst, size_t off, int64_t rs, int64_t cs = 1) { return place(t, r0, rows, dst, off, Place{rs, cs, 0, 0, 0, 0, 0}); }
    // decode-layout copy of a dense bf16 weight [N][K]; none (null) where the weight-streaming kernels do not take the shape, memory is short or CR_DECODE_LAYOUT=0
    bf16* swizzled(const std::string& n, const void* w, int N, int K) {
        const char* e = getenv("CR_DECODE_LAYOUT");
        if (lm.f32 || K % 128 || (e && atoi(e) == 0)) return nullptr;
        bf16* d = (bf16*)make(n, decode_swizzled_bytes(N, K) / 2, 2, CR_BF16);
        if (!d) { (void)hipGetLastError(); return nullptr; }
        return decode_swizzle_weight(DEC_WO, (const bf16*)w, K, N, K, d, st) == CR_OK ? d : nullptr;
    }
    float* gain(const std::string& name, const std::string& n, int len, int padded, float base) {
        const DevTensor* t = src(n, len, 0);
        if (!t) return nullptr;
        float* d = (float*)make(name, padded, 4, CR_F32);
        if (d) hipLaunchKernelGGL(lm_gain_kernel, dim3((len + 255) / 256), dim3(256), 0, st, (const bf16*)t->ptr, len, base, d);
        return d;
    }
    float* table(const std::string& n, const std::vector<float>& v) {
        float* d = (float*)make(n, v.size(), 4, CR_F32);
        if (d && (hipMemcpyAsync(d, v.data(), v.size() * 4, hipMemcpyHostToDevice, st) != hipSuccess || hipStreamSynchronize(st) != hipSuccess)) { cr_fail(CR_ERR_HIP, "%s", n.c_str()); return nullptr; }
        return d;
    }
};

int derive_latent(Deriver& dv, const std::string& p, const std::string& o, LmLayer& L) {
    const Lm& lm = dv.lm;
    const cr_lm_layer& s = L.s;
    const int W = lm.d.width, Wp = lm.Wp, H = s.heads;
    L.nq = dv.gain(o + "nq", p + "mix.dq.norm", s.q_rank, L.Qp, 0.f); L.nc = dv.gain(o + "nc", p + "mix.dkv.norm", s.kv_rank, L.Rp, 0.f);
    if (!L.nq || !L.nc) return CR_ERR_STATE;
    const DevTensor *dq = dv.src(p + "mix.dq", s.q_rank, W), *dkv = dv.src(p + "mix.dkv", s.kv_rank, W), *g = dv.src(p + "mix.g", (int64_t)H * s.vdim, W);
    const DevTensor *uq = dv.src(p + "mix.uq", (int64_t)H * s.dim, s.q_rank), *uk = dv.src(p + "mix.uk", (int64_t)H * s.dim, s.kv_rank),
                    *uv = dv.src(p + "mix.uv", (int64_t)H * s.vdim, s.kv_rank), *wo = dv.src(p + "mix.o", W, (int64_t)H * s.vdim);
    if (!dq || !dkv || !g || !uq || !uk || !uv || !wo) return CR_ERR_STATE;
    L.wa = dv.mat(o + "a", (size_t)L.Na * Wp); L.wuq = dv.mat(o + "uq", (size_t)H * L.Ap * L.Qp); L.wkv = dv.mat(o + "kv", (size_t)2 * H * L.Ap * L.Rp);
    L.wukT = dv.mat(o + "ukT", (size_t)H * L.Rp * L.Ap); L.wo = dv.mat(o + "o", (size_t)Wp * L.Gp);
    if (!L.wa || !L.wuq || !L.wkv || !L.wukT || !L.wo) return CR_ERR_NOMEM;
    CR_TRY(dv.place(dq, 0, s.q_rank, L.wa, 0, Wp));
    CR_TRY(dv.place(dkv, 0, s.kv_rank, L.wa, (size_t)L.off_c * Wp, Wp));
    CR_TRY(dv.place(g, 0, H * s.vdim, L.wa, (size_t)L.off_g * Wp, Wp));
    CR_TRY(dv.place(wo, 0, W, L.wo, 0, L.Gp));
    for (int h = 0; h < H; h++) {
        CR_TRY(dv.place(uq, (int64_t)h * s.dim, s.dim, L.wuq, (size_t)h * L.Ap * L.Qp, L.Qp));
        CR_TRY(dv.place(uk, (int64_t)h * s.dim, s.dim, L.wkv, (size_t)h * L.Ap * L.Rp, L.Rp));
        CR_TRY(dv.place(uv, (int64_t)h * s.vdim, s.vdim, L.wkv, (size_t)(H + h) * L.Ap * L.Rp, L.Rp));
        CR_TRY(dv.place(uk, (int64_t)h * s.dim, s.dim, L.wukT, (size_t)h * L.Rp * L.Ap, 1, L.Ap));         // transposed: row = latent column
    }
    L.wa_dl = dv.swizzled(o + "a.dl", L.wa, L.Na, Wp); L.wuq_dl = dv.swizzled(o + "uq.dl", L.wuq, H * L.Ap, L.Qp); L.wo_dl = dv.swizzled(o + "o.dl", L.wo, Wp, L.Gp);
    return CR_OK;
}

// attention over heads and / or retention: the fused projection's regions, the joint output projection, gains, rotation frequencies, powers of the decays
int derive_heads(Deriver& dv, const std::string& p, const std::string& o, LmLayer& L) {
    const Lm& lm = dv.lm;
    const int W = lm.d.width, Wp = lm.Wp;
    const cr_lm_heads& a = L.s.attn;
    const cr_lm_retention& r = L.s.ret;
    L.wa = dv.mat(o + "a", (size_t)L.Na * Wp); L.wo = dv.mat(o + "o", (size_t)Wp * L.Gp);
    if (!L.wa || !L.wo) return CR_ERR_NOMEM;
    auto rotations = [&](const std::string& n, double base, int dims) {
        std::vector<float> f(dims / 2);
        for (int i = 0; i < dims / 2; i++) f[i] = (float)pow(base, -2.0 * i / dims);
        return dv.table(n, f);
    };
    auto rows = [&](int kind, const std::string& name, int size) -> int {
        const LmRegion* g = L.region(kind);
        const DevTensor* t = dv.src(name, (int64_t)g->heads * size, W);
        if (!t) return CR_ERR_STATE;
        for (int h = 0; h < g->heads; h++) CR_TRY(dv.place(t, (int64_t)h * size, size, L.wa, ((size_t)g->off + (size_t)h * g->P) * Wp, Wp));
        return CR_OK;
    };
    if (L.heads()) {
        const std::string q = p + "mix." + std::string(a.name, strnlen(a.name, sizeof a.name));
        CR_TRY(rows(LM_Q, q + "q", a.dim));
        CR_TRY(rows(LM_K, q + "k", a.dim));
        CR_TRY(rows(LM_V, q + "v", a.vdim));
        const DevTensor* wo = dv.src(q + "o", W, (int64_t)a.heads * a.vdim);
        if (!wo) return CR_ERR_STATE;
        CR_TRY(dv.place(wo, 0, W, L.wo, 0, L.Gp));
        if (a.qk_norm && (!(L.nq = dv.gain(o + "nq", q + "q.norm", a.dim, L.Ap, 0.f)) || !(L.nc = dv.gain(o + "nk", q + "k.norm", a.dim, L.Ap, 0.f)))) return CR_ERR_STATE;
        if (a.rot_dims && !(L.fq_a = rotations(o + "fa", a.rot_base, a.rot_dims))) return CR_ERR_NOMEM;
    }
    if (L.retention()) {
        const std::string q = p + "mix." + std::string(r.name, strnlen(r.name, sizeof r.name));
        CR_TRY(rows(LM_RQ, q + "q", r.dim));
        CR_TRY(rows(LM_RK, q + "k", r.dim));
        CR_TRY(rows(LM_RV, q + "v", r.vdim));
        CR_TRY(rows(LM_RG, q + "g", r.vdim));
        const DevTensor* wo = dv.src(q + "o", W, (int64_t)r.heads * r.vdim);
        if (!wo) return CR_ERR_STATE;
        CR_TRY(dv.place(wo, 0, W, L.wo, L.off_r, L.Gp));
        if (r.rot_dims && !(L.fq_r = rotations(o + "fr", r.rot_base, r.rot_dims))) return CR_ERR_NOMEM;
        std::vector<float> pw((size_t)r.heads * (RET_CHUNK + 1));
        for (int h = 0; h < r.heads; h++)
            for (int i = 0; i <= RET_CHUNK; i++) pw[(size_t)h * (RET_CHUNK + 1) + i] = i ? (float)pow(L.decay[h], (double)i) : 1.f;
        if (!(L.pw = dv.table(o + "pw", pw))) return CR_ERR_NOMEM;
    }
    L.wa_dl = dv.swizzled(o + "a.dl", L.wa, L.Na, Wp); L.wo_dl = dv.swizzled(o + "o.dl", L.wo, Wp, L.Gp);
    return CR_OK;
}

int derive_layer(Deriver& dv, int i, LmLayer& L) {
    const Lm& lm = dv.lm;
    const cr_lm_layer& s = L.s;
    const std::string p = "l" + std::to_string(i) + ".", o = "derived.lm." + std::to_string(i) + ".";
    const int W = lm.d.width, Wp = lm.Wp;
    const float base = lm.gain_base();
    const bool post = !lm.d.no_post_norm;
    L.n1 = dv.gain(o + "n1", p + "norm1", W, Wp, base);
    if (!L.n1 || (post && !(L.n1b = dv.gain(o + "n1b", p + "norm1b", W, Wp, base)))) return CR_ERR_STATE;
    CR_TRY(L.latent() ? derive_latent(dv, p, o, L) : derive_heads(dv, p, o, L));
    if (lm.d.side_dim > 0) {
        const DevTensor *g = dv.src(p + "side.gate", lm.d.side_dim, W), *u = dv.src(p + "side.proj", W, lm.d.side_dim);
        L.ns = dv.gain(o + "ns", p + "side.norm", W, Wp, 0.f);
        if (!g || !u || !L.ns) return CR_ERR_STATE;
        L.sgate = dv.mat(o + "sg", (size_t)lm.Sp * Wp); L.sproj = dv.mat(o + "sp", (size_t)Wp * lm.Sp);
        if (!L.sgate || !L.sproj) return CR_ERR_NOMEM;
        CR_TRY(dv.place(g, 0, lm.d.side_dim, L.sgate, 0, Wp));
        CR_TRY(dv.place(u, 0, W, L.sproj, 0, lm.Sp));
        L.sgate_dl = dv.swizzled(o + "sg.dl", L.sgate, lm.Sp, Wp); L.sproj_dl = dv.swizzled(o + "sp.dl", L.sproj, Wp, lm.Sp);
    }
    if (s.ff == CR_FF_NONE) return CR_OK;
    L.n2 = dv.gain(o + "n2", p + "norm2", W, Wp, base);
    if (!L.n2 || (post && !(L.n2b = dv.gain(o + "n2b", p + "norm2b", W, Wp, base)))) return CR_ERR_STATE;
    if (s.ff == CR_FF_DENSE) {
        const DevTensor *up = dv.src(p + "mlp.up", s.expert_ff, W), *dn = dv.src(p + "mlp.down", W, s.expert_ff);
        if (!up || !dn) return CR_ERR_STATE;
        L.wgu = dv.mat(o + "up", (size_t)L.ffp * Wp); L.wdn = dv.mat(o + "dn", (size_t)Wp * L.ffp);
        if (!L.wgu || !L.wdn) return CR_ERR_NOMEM;
        CR_TRY(dv.place(up, 0, s.expert_ff, L.wgu, 0, Wp));
        CR_TRY(dv.place(dn, 0, W, L.wdn, 0, L.ffp));
        L.wgu_dl = dv.swizzled(o + "up.dl", L.wgu, L.ffp, Wp); L.wdn_dl = dv.swizzled(o + "dn.dl", L.wdn, Wp, L.ffp);
        return CR_OK;
    }
    L.corr = dv.gain(o + "corr", p + "mlp.correction", s.experts, L.Ep, 0.f);
    const DevTensor* rt = dv.src(p + "mlp.router", s.experts, W);
    if (!L.corr || !rt) return CR_ERR_STATE;
    L.router = dv.mat(o + "router", (size_t)L.Ep * Wp); L.wgu = dv.mat(o + "gu", (size_t)s.experts * 2 * L.ffp * Wp); L.wdn = dv.mat(o + "dn", (size_t)s.experts * Wp * L.ffp);
    if (!L.router || !L.wgu || !L.wdn) return CR_ERR_NOMEM;
    CR_TRY(dv.place(rt, 0, s.experts, L.router, 0, Wp));
    for (int e = 0; e < s.experts; e++) {
        const std::string q = p + "mlp.e" + std::to_string(e) + ".";
        const DevTensor *ga = dv.src(q + "gate", s.expert_ff, W), *up = dv.src(q + "up", s.expert_ff, W), *dn = dv.src(q + "down", W, s.expert_ff);
        if (!ga || !up || !dn) return CR_ERR_STATE;
        CR_TRY(dv.place(ga, 0, s.expert_ff, L.wgu, (size_t)e * 2 * L.ffp * Wp, Place{Wp, 1, 1, 0, lm.f32 ? 0 : Wp / 32, 0, 0}));
        CR_TRY(dv.place(up, 0, s.expert_ff, L.wgu, (size_t)e * 2 * L.ffp * Wp, Place{Wp, 1, 1, 8, lm.f32 ? 0 : Wp / 32, 0, 0}));
        CR_TRY(dv.place(dn, 0, W, L.wdn, (size_t)e * Wp * L.ffp, Place{L.ffp, 1, 0, 0, lm.f32 ? 0 : L.ffp / 32, 0, 0}));
    }
    return CR_OK;
}

// Where a prompt's keys sit for layers of one chunk size: per sequence its cached rows of the chunk the portion goes on in, then the portion; pieces are the chunks (causal segments
// {first row, rows, place of the first row in its chunk, key row of the chunk's start}).  Device pointers into the step's one upload.
struct KeyPlan {
    int ring, n_pieces, longest, n_pre; size_t Mk;
    const int32_t *row_key, *row_slot, *pieces, *pre_key, *pre_slot;
};
// attention splits of a decode step for layers of one chunk size
constexpr int HEADS_SPLIT = 64 * ATTN_SPLIT_TILES;

struct Step {
    int M; bool decode;
    const int64_t* tokens;          // device; null: the sequences' last generated ids
    LmRowIndex ix;
    struct Seg { int row0, S, pos0, seq, key0; };
    std::vector<Seg> segs;          // prefill
    const int32_t* d_seg;           // prefill: {first row, rows, first position, first key row} per segment
    bool fresh;                     // prefill: every sequence starts empty (key rows = token rows)
    int Mk;                         // key rows
    int nsplit, split;              // decode, latent attention: splits of the longest sequence, keys per split
    std::vector<KeyPlan> plans;     // prefill, one per distinct chunk size
    std::vector<int> hsplit;        // decode: attention splits per distinct chunk size
    const int32_t *d_rseg, *d_snap0, *d_chunks;      // prefill: {first row, rows, first position, sequence} per segment, its first retention chunk; {first row, rows} per chunk
    int snaps, longest;
};

// one activations carve-up for a step; the same function sizes the workspace and lays it out
struct Buffers {
    float* x; void *h, *a, *cq, *q, *c, *kv, *qp, *ol, *ao, *y, *act, *ye, *cat, *z2; float *z, *wt, *part, *sl, *rq, *rk, *raw; bf16 *rq2, *rk2, *snap;
    int32_t *idx, *perm, *n_tiles, *tok; int4* tiles;
};
bool expanded(const Lm& lm, const LmLayer& L, bool decode) { return !lm.f32 && !decode && L.s.scale > 0.f && (L.Ap == 64 || L.Ap == 128 || L.Ap == 256); }
bool split_decode(const Lm& lm, const LmLayer& L, bool decode) { return !lm.f32 && decode && latent_decode_supported(L.Rp); }
bool flash_heads(const Lm& lm, const LmLayer& L) { return !lm.f32 && L.s.attn.scale > 0.f && L.Ap <= 256; }
bool matrix_retention(const Lm& lm, const LmLayer& L, bool decode) { return !lm.f32 && !decode && ret_matrix_supported(L.Kp, L.Vp); }
// decode: query heads of one key head handled by one workgroup of the split kernel (at most 32 rows)
int heads_per_split(const cr_lm_heads& a) {
    int n = a.heads / a.kv_heads, d = std::min(n, 32);
    while (n % d) d--;
    return d;
}

// decode of <= 64 rows: fp32 K-slices of A . W^T (gemm_skinny.hip) for a consumer that adds them; 0 when the shape has no such form.  Wide products of more than a few rows are one
// slice through the kernel that splits N over its waves (gemm_stream.hip).
GemmParams slice_params(const void* A, int64_t lda, const void* W, const bf16* dl, float* C, int M, int N, int K) {
    GemmParams p{};
    p.A = (const bf16*)A; p.lda = lda; p.W = dl ? dl : (const bf16*)W; p.ldw = K; p.wsw = dl ? 1 : 0; p.C = C; p.ldc = N; p.M = M; p.N = N; p.K = K;
    return p;
}
bool one_slice(int M, int N, int K) { return gemm_stream_supported(EPI_F32, slice_params(nullptr, K, nullptr, nullptr, nullptr, M, N, K), 1); }
int slices_of(const Lm& lm, int M, int N, int K, bool decode) { return lm.f32 || !decode || M > 64 ? 0 : one_slice(M, N, K) ? 1 : gemm_partial_splits(N, K); }
int sliced(cr_ctx* c, const void* A, int64_t lda, const void* W, const bf16* dl, float* C, int M, int N, int K, hipStream_t st) {
    GemmParams p = slice_params(A, lda, W, dl, C, M, N, K);
    if (!one_slice(M, N, K)) return ctx_gemm(c, EPI_PARTIAL, p, st);
    p.raw32 = 1;
    return ctx_gemm(c, EPI_F32, p, st);
}

// K-slices of the token side's gate in the 128-row kernel: four where K allows (depends on K alone)
int side_slices(int K) { return K % 256 == 0 ? 4 : K % 128 == 0 ? 2 : 1; }

Buffers carve(const Lm& lm, Arena& ar, const Step& sp) {
    const size_t es = lm.esz();
    const int M = sp.M, Wp = lm.Wp;
    const bool decode = sp.decode, sliced = decode && !lm.f32 && M <= 64;
    size_t Na = 0, Qp = 0, Rp = 0, Gp = 0, qn = 0, kvn = 0, hr = 0, Ep = 0, top = 0, act = 0, tiles = 0, part = 0, sl = 0, kvh = 0, r32 = 0, r16 = 0, raw = 0, snap = 0;
    auto slices = [&](int N, int K) { if (sliced) sl = std::max(sl, (size_t)M * std::max(1, gemm_partial_splits(N, K)) * N); };
    for (const LmLayer& L : lm.layers) {
        Na = std::max<size_t>(Na, L.Na); Gp = std::max<size_t>(Gp, L.Gp);
        slices(L.Na, Wp); slices(Wp, L.Gp);
        if (L.latent()) {
            Qp = std::max<size_t>(Qp, L.Qp); Rp = std::max<size_t>(Rp, L.Rp);
            qn = std::max<size_t>(qn, (size_t)L.s.heads * L.Ap);
            if (expanded(lm, L, decode)) kvn = std::max<size_t>(kvn, (size_t)2 * L.s.heads * L.Ap);
            else hr = std::max<size_t>(hr, (size_t)L.s.heads * L.Rp);
            if (split_decode(lm, L, decode)) part = std::max(part, latent_part_floats(M, L.s.heads, sp.nsplit, L.Rp));
            slices(L.s.heads * L.Ap, L.Qp);
        }
        if (L.heads()) {
            const cr_lm_heads& a = L.s.attn;
            qn = std::max<size_t>(qn, (size_t)a.heads * L.Ap);
            if (!decode) kvh = std::max<size_t>(kvh, sp.plans[L.chunk_ix].Mk * 2 * a.kv_heads * L.Ap);
            else if (flash_heads(lm, L)) part = std::max(part, (size_t)M * a.heads * sp.hsplit[L.chunk_ix] * (L.Ap + 2));
        }
        if (L.retention()) {
            const size_t n = (size_t)M * L.s.ret.heads * L.Kp;
            if (matrix_retention(lm, L, decode)) { r16 = std::max(r16, 2 * n); snap = std::max(snap, (size_t)sp.snaps * L.s.ret.heads * 2 * L.Vp * L.Kp); }
            else r32 = std::max(r32, n);
            if (!decode && !matrix_retention(lm, L, decode)) raw = std::max(raw, (size_t)M * L.s.ret.heads * L.Vp);
        }
        if (L.s.ff == CR_FF_DENSE) { act = std::max<size_t>(act, L.ffp); slices(Wp, L.ffp); }
        if (L.s.ff != CR_FF_MOE) continue;
        Ep = std::max<size_t>(Ep, L.Ep); top = std::max<size_t>(top, L.s.top); act = std::max<size_t>(act, (size_t)L.s.top * L.ffp);
        tiles = std::max<size_t>(tiles, lm_max_tiles(M * L.s.top, L.s.experts, LM_TILE_M));
    }
    if (lm.Sp) {
        slices(lm.Sp, Wp); slices(Wp, lm.Sp);
        if (!lm.f32 && !slices_of(lm, M, lm.Sp, Wp, decode)) sl = std::max(sl, (size_t)M * side_slices(Wp) * lm.Sp);
    }
    if (lm.d.loop_in) slices(Wp, 2 * Wp);
    auto T = [&](size_t n) { return (void*)ar.take<char>(n * es); };
    Buffers b{};
    b.x = ar.take<float>((size_t)M * Wp); b.h = T((size_t)M * Wp); b.a = T((size_t)M * Na); b.cq = T((size_t)M * Qp); b.q = T((size_t)M * qn);
    b.c = T((size_t)M * Rp); b.kv = T(std::max((size_t)sp.Mk * kvn, kvh)); b.qp = T((size_t)M * hr); b.ol = T((size_t)M * hr); b.ao = T((size_t)M * Gp); b.y = T((size_t)M * Wp);
    b.act = T((size_t)M * act); b.ye = T((size_t)M * top * Wp);
    b.part = ar.take<float>(part); b.sl = ar.take<float>(sl);
    b.z = ar.take<float>((size_t)M * Ep * (M <= 128 ? LM_ROUTER_SLICES : 1)); b.wt = ar.take<float>((size_t)M * top);
    b.idx = ar.take<int32_t>((size_t)M * top); b.perm = ar.take<int32_t>((size_t)M * top); b.n_tiles = ar.take<int32_t>(1); b.tiles = ar.take<int4>(tiles);
    b.rq = ar.take<float>(r32); b.rk = ar.take<float>(r32); b.rq2 = ar.take<bf16>(r16); b.rk2 = ar.take<bf16>(r16); b.raw = ar.take<float>(raw); b.snap = ar.take<bf16>(snap);
    b.tok = ar.take<int32_t>(M); b.z2 = T((size_t)M * lm.Sp); b.cat = T(lm.d.loop_in ? (size_t)M * 2 * Wp : 0);
    return b;
}
size_t carve_bytes(const Lm& lm, const Step& sp) {
    Arena ar(nullptr);
    carve(lm, ar, sp);
    return ar.off + 512;
}

// C[M, N] = A . W^T in the model's element type: the engine's dense kernels for bf16, the fp32 tile kernel otherwise
int dense(cr_ctx* c, const Lm& lm, const void* A, int64_t lda, const void* W, void* C, int64_t ldc, int M, int N, int K, hipStream_t st, bool prompt, const bf16* dl = nullptr,
          bool relu2 = false) {
    if (lm.f32) {
        LmGemmParams p{};
        p.A = A; p.lda = lda; p.W = W; p.ldw = K; p.C = C; p.ldc = ldc; p.M = M; p.N = N; p.K = K;
        return launch_lm_gemm(true, relu2 ? LM_RELU2 : LM_STORE, p, st);
    }
    GemmParams p{};
    p.A = (const bf16*)A; p.lda = lda; p.W = (const bf16*)W; p.ldw = K; p.C = C; p.ldc = ldc; p.M = M; p.N = N; p.K = K;
    if (prompt && M <= 64) p.kernel = 128;           // a prompt row's sum does not depend on how many rows it is prefilled with
    if (!prompt && M <= 64 && dl) { p.W = dl; p.wsw = 1; }
    return ctx_gemm(c, relu2 ? EPI_RELU2 : EPI_STORE, p, st);
}
// the same product left in fp32 (router scores, logits, the looped span's entry)
int raw32(cr_ctx* c, const Lm& lm, const void* A, const void* W, float* C, int64_t ldc, int M, int N, int K, float softcap, hipStream_t st, const bf16* dl = nullptr) {
    if (!lm.f32) {
        GemmParams p{};
        p.A = (const bf16*)A; p.lda = K; p.W = (const bf16*)W; p.ldw = K; p.C = C; p.ldc = ldc; p.M = M; p.N = N; p.K = K; p.raw32 = 1; p.softcap = softcap;
        if (M <= 64 && dl) { p.W = dl; p.wsw = 1; }
        return ctx_gemm(c, EPI_F32, p, st);
    }
    LmGemmParams p{};
    p.A = A; p.lda = K; p.W = W; p.ldw = K; p.C = C; p.ldc = ldc; p.M = M; p.N = N; p.K = K; p.softcap = softcap;
    return launch_lm_gemm(lm.f32, LM_RAW32, p, st);
}

// h -> ao, latent attention
int latent_mixer(cr_ctx* c, cr_kv* kv, const Step& sp, Buffers& b, const LmLayer& L, size_t r, hipStream_t st) {
    const Lm& lm = *c->lm;
    const cr_lm_layer& s = L.s;
    const int M = sp.M, Wp = lm.Wp, H = s.heads;
    const size_t es = lm.esz();
    char* cache = kv->lat + kv->lat_off[r];
    const int s_a = slices_of(lm, M, L.Na, Wp, sp.decode);
    if (s_a) CR_TRY(sliced(c, b.h, Wp, L.wa, L.wa_dl, b.sl, M, L.Na, Wp, st));
    else CR_TRY(dense(c, lm, b.h, Wp, L.wa, b.a, L.Na, M, L.Na, Wp, st, !sp.decode, L.wa_dl));
    CR_TRY(launch_lm_latents(lm.f32, lm, L, M, b.a, s_a ? b.sl : nullptr, s_a, b.cq, sp.decode ? nullptr : b.c, cache, kv->max_tokens, sp.ix, b.ao, st));
    const int s_q = L.Ap <= 512 ? slices_of(lm, M, H * L.Ap, L.Qp, sp.decode) : 0;
    if (s_q) CR_TRY(sliced(c, b.cq, L.Qp, L.wuq, L.wuq_dl, b.sl, M, H * L.Ap, L.Qp, st));
    else CR_TRY(dense(c, lm, b.cq, L.Qp, L.wuq, b.q, (int64_t)H * L.Ap, M, H * L.Ap, L.Qp, st, !sp.decode, L.wuq_dl));
    const void* gate = (const char*)b.a + (size_t)L.off_g * es;
    if (expanded(lm, L, sp.decode)) {
        const int64_t ldk = (int64_t)2 * H * L.Ap;
        if (sp.fresh) CR_TRY(dense(c, lm, b.c, L.Rp, L.wkv, b.kv, ldk, M, 2 * H * L.Ap, L.Rp, st, true));
        else
            for (const Step::Seg& sg : sp.segs)
                CR_TRY(dense(c, lm, cache + (size_t)sg.seq * kv->max_tokens * L.Rp * es, L.Rp, L.wkv, (bf16*)b.kv + (size_t)sg.key0 * ldk, ldk, sg.pos0 + sg.S, 2 * H * L.Ap, L.Rp, st, true));
        AttnParams ap{};
        ap.Q = (const bf16*)b.q; ap.K = (const bf16*)b.kv; ap.V = (const bf16*)b.kv + (size_t)H * L.Ap; ap.O = (bf16*)b.ao;
        ap.q_rs = (int64_t)H * L.Ap; ap.q_hs = L.Ap; ap.k_bs = ap.v_bs = ap.k_rs = ap.v_rs = ldk; ap.k_hs = ap.v_hs = L.Ap; ap.o_rs = L.Gp; ap.o_hs = s.vdim;
        ap.B = (int)sp.segs.size(); ap.H = H; ap.kv_group = 1; ap.seg = sp.d_seg; ap.q_prescale = 1.f; ap.s_div = 1.f;
        ap.wide = 1; ap.s_mul = s.scale; ap.vdim = s.vdim; ap.gate = (const bf16*)gate; ap.g_rs = L.Na;
        for (const Step::Seg& sg : sp.segs) ap.Sq = std::max(ap.Sq, sg.S);
        if (launch_flash_attn(ap, L.Ap, true, st) != CR_OK) return cr_fail(CR_ERR_HIP, "latent attention (expanded): launch failed");
    } else {
        LmGemmParams g{};
        g.A = b.q; g.lda = (int64_t)H * L.Ap; g.W = L.wukT; g.ldw = L.Ap; g.C = b.qp; g.ldc = (int64_t)H * L.Rp; g.M = M; g.N = L.Rp; g.K = L.Ap;
        g.batch = H; g.a_bs = L.Ap; g.w_bs = (int64_t)L.Rp * L.Ap; g.c_bs = L.Rp;
        if (s_q) CR_TRY(launch_latent_absorb(L, M, b.sl, s_q, b.qp, st));
        else CR_TRY(launch_lm_gemm(lm.f32, LM_STORE, g, st));
        LatentAttnParams ap{};
        ap.Q = b.qp; ap.C = cache; ap.O = b.ol; ap.M = M; ap.H = H; ap.Rp = L.Rp; ap.max_tokens = kv->max_tokens; ap.scale = s.scale; ap.ix = sp.ix;
        if (split_decode(lm, L, sp.decode)) {
            LatentDecodeParams dp{};
            dp.a = ap; dp.nsplit = sp.nsplit; dp.split = sp.split; dp.part_o = b.part; dp.part_ml = b.part + (size_t)M * H * sp.nsplit * L.Rp; dp.wuv = (const bf16*)L.wkv + (size_t)H * L.Ap * L.Rp;
            dp.uv_hs = (int64_t)L.Ap * L.Rp; dp.vdim = s.vdim; dp.gate = (const bf16*)gate; dp.ldg = L.Na; dp.out = (bf16*)b.ao; dp.ldo = L.Gp;
            CR_TRY(launch_latent_decode(dp, st));
        } else {
        CR_TRY(launch_latent_attn_plain(lm.f32, ap, st));
        g = LmGemmParams{};
        g.A = b.ol; g.lda = (int64_t)H * L.Rp; g.W = (const char*)L.wkv + (size_t)H * L.Ap * L.Rp * es; g.ldw = L.Rp; g.C = b.ao; g.ldc = L.Gp; g.M = M; g.N = s.vdim; g.K = L.Rp;
        g.batch = H; g.a_bs = L.Rp; g.w_bs = (int64_t)L.Ap * L.Rp; g.c_bs = s.vdim; g.gate = gate; g.ldg = L.Na; g.g_bs = s.vdim;
        CR_TRY(launch_lm_gemm(lm.f32, LM_GATE, g, st));
        }
    }
    return CR_OK;
}

// h -> ao, attention over heads and / or retention
int heads_mixer(cr_ctx* c, cr_kv* kv, const Step& sp, Buffers& b, const LmLayer& L, size_t r, hipStream_t st) {
    const Lm& lm = *c->lm;
    const cr_lm_heads& a = L.s.attn;
    const cr_lm_retention& rt = L.s.ret;
    const int M = sp.M, Wp = lm.Wp;
    const size_t es = lm.esz();
    const int s_a = slices_of(lm, M, L.Na, Wp, sp.decode);
    if (s_a) CR_TRY(sliced(c, b.h, Wp, L.wa, L.wa_dl, b.sl, M, L.Na, Wp, st));
    else CR_TRY(dense(c, lm, b.h, Wp, L.wa, b.a, L.Na, M, L.Na, Wp, st, !sp.decode, L.wa_dl));
    const KeyPlan* kp = L.heads() && !sp.decode ? &sp.plans[L.chunk_ix] : nullptr;
    const int ring = L.heads() ? std::min(lm.chunks[L.chunk_ix], kv->max_tokens) : 1, chunk = L.heads() ? lm.chunks[L.chunk_ix] : 1;
    char *ck = kv->lat + kv->lat_off[r], *cv = ck + (size_t)kv->n_seqs * a.kv_heads * ring * L.Ap * es;
    if (kp) CR_TRY(launch_lm_prefix(lm.f32, L, kp->n_pre, kp->pre_key, kp->pre_slot, b.kv, ck, cv, ring, st));
    const bool matrix = L.retention() && matrix_retention(lm, L, sp.decode);
    LmHeadsIn in{};
    in.a = b.a; in.lda = L.Na; in.part = s_a ? b.sl : nullptr; in.slices = s_a; in.ix = sp.ix; in.q = b.q; in.kv = kp ? b.kv : nullptr; in.cache_k = ck; in.cache_v = cv;
    in.ring = ring; in.chunk = chunk; in.row_key = kp ? kp->row_key : nullptr; in.row_slot = kp ? kp->row_slot : nullptr; in.ao = b.ao;
    if (matrix) { in.rq2 = b.rq2; in.rk2 = b.rk2; } else { in.rq = b.rq; in.rk = b.rk; }
    CR_TRY(launch_lm_heads(lm.f32, lm, L, M, in, st));
    AttnParams ap{};
    bool merge = false;
    if (L.heads()) {
        const int64_t qld = (int64_t)a.heads * L.Ap, ldk = (int64_t)2 * a.kv_heads * L.Ap;
        if (flash_heads(lm, L)) {
            ap.Q = (const bf16*)b.q; ap.O = (bf16*)b.ao; ap.q_prescale = 1.f; ap.s_div = 1.f; ap.wide = 1; ap.s_mul = a.scale; ap.softcap = a.softcap; ap.out_mul = a.out_scale; ap.vdim = a.vdim;
            if (sp.decode) {
                const int rows = heads_per_split(a), nsplit = sp.hsplit[L.chunk_ix];
                ap.K = (const bf16*)ck; ap.V = (const bf16*)cv; ap.H = a.heads / rows; ap.kv_group = a.heads / a.kv_heads / rows; ap.B = M; ap.Sq = rows;
                ap.q_bs = qld; ap.q_rs = L.Ap; ap.q_hs = (int64_t)rows * L.Ap; ap.k_rs = ap.v_rs = L.Ap; ap.k_hs = ap.v_hs = (int64_t)ring * L.Ap; ap.k_bs = ap.v_bs = a.kv_heads * ap.k_hs;
                ap.o_bs = L.Gp; ap.o_rs = a.vdim; ap.o_hs = (int64_t)rows * a.vdim; ap.seq_map = sp.ix.seqs; ap.sk_arr = sp.ix.lens; ap.sk_add = 1; ap.sk_mod = chunk;
                ap.nsplit = nsplit; ap.part_o = b.part; ap.part_ml = b.part + (size_t)M * a.heads * nsplit * L.Ap;
                ap.no_merge = merge = L.retention();          // retention's launch takes the merge along
                if (launch_flash_attn_split(ap, L.Ap, st) != CR_OK) return cr_fail(CR_ERR_HIP, "attention over heads (decode): launch failed");
            } else {
                ap.K = (const bf16*)b.kv; ap.V = (const bf16*)b.kv + (size_t)a.kv_heads * L.Ap;
                ap.q_rs = qld; ap.q_hs = L.Ap; ap.k_bs = ap.v_bs = ap.k_rs = ap.v_rs = ldk; ap.k_hs = ap.v_hs = L.Ap; ap.o_rs = L.Gp; ap.o_hs = a.vdim;
                ap.H = a.heads; ap.kv_group = a.heads / a.kv_heads; ap.Sq = kp->longest;
                for (int i = 0; i < kp->n_pieces; i += 32768) {
                    ap.seg = kp->pieces + 4 * (size_t)i; ap.B = std::min(32768, kp->n_pieces - i);
                    if (launch_flash_attn(ap, L.Ap, true, st) != CR_OK) return cr_fail(CR_ERR_HIP, "attention over heads: launch failed");
                }
            }
        } else {
            HeadsAttnParams hp{};
            hp.Q = b.q; hp.O = b.ao; hp.ldo = L.Gp; hp.M = M; hp.H = a.heads; hp.G = a.kv_heads; hp.Ap = L.Ap; hp.vdim = a.vdim; hp.chunk = chunk; hp.ring = ring;
            hp.scale = a.scale; hp.softcap = a.softcap; hp.out_scale = a.out_scale; hp.ix = sp.ix;
            if (sp.decode) { hp.K = ck; hp.V = cv; hp.k_rs = L.Ap; }
            else { hp.K = b.kv; hp.V = (char*)b.kv + (size_t)a.kv_heads * L.Ap * es; hp.k_rs = ldk; hp.k_hs = L.Ap; hp.row_key = kp->row_key; }
            CR_TRY(launch_heads_attn_plain(lm.f32, hp, st));
        }
    }
    if (!L.retention()) return CR_OK;
    RetParams rp{};
    rp.rq = b.rq; rp.rk = b.rk; rp.rq2 = b.rq2; rp.rk2 = b.rk2; rp.lda = L.Na; rp.v = (char*)b.a + (size_t)L.region(LM_RV)->off * es; rp.g = (char*)b.a + (size_t)L.region(LM_RG)->off * es;
    rp.ao = (char*)b.ao + (size_t)L.off_r * es; rp.ldo = L.Gp; rp.state = (float*)(kv->lat + kv->state_off[r]); rp.raw = b.raw; rp.snap = b.snap; rp.pw = L.pw;
    rp.M = M; rp.H = rt.heads; rp.Kp = L.Kp; rp.Vp = L.Vp; rp.vdim = rt.vdim; rp.eps = lm.d.eps; rp.out_scale = rt.out_scale; rp.ix = sp.ix;
    rp.seg = sp.d_rseg; rp.snap0 = sp.d_snap0; rp.n_segs = (int)sp.segs.size(); rp.longest = sp.longest; rp.chunks = sp.d_chunks; rp.n_chunks = sp.snaps;
    return sp.decode ? launch_ret_decode(lm.f32, rp, merge ? &ap : nullptr, L.Ap, st) : matrix ? launch_ret_matrix(rp, st) : launch_ret_recurrent(lm.f32, rp, st);
}

// h -> ye, wt: the rows of every chosen expert and their weights
int expert_mixture(cr_ctx* c, const Step& sp, Buffers& b, const LmLayer& L, hipStream_t st) {
    const Lm& lm = *c->lm;
    const cr_lm_layer& s = L.s;
    const int M = sp.M, Wp = lm.Wp;
    if (!lm.f32 && lm_router_supported(L)) CR_TRY(launch_lm_router(lm, L, M, b.h, b.idx, b.wt, b.z, st));
    else {
        CR_TRY(raw32(c, lm, b.h, L.router, b.z, L.Ep, M, s.experts, Wp, 0.f, st));
        CR_TRY(launch_lm_route(L, M, b.z, L.Ep, 1, b.idx, b.wt, st));
    }
    if (!lm.f32) {
        MoeGemmParams mp{};
        const bool stream = sp.decode && M <= MOE_STREAM_ROWS;
        mp.A = (const bf16*)b.h; mp.lda = Wp; mp.W = (const bf16*)L.wgu; mp.w_es = (int64_t)2 * L.ffp * Wp; mp.C = (bf16*)b.act; mp.ldc = L.ffp; mp.N = 2 * L.ffp; mp.K = Wp;
        mp.gather_div = s.top; mp.limit = s.limit; mp.idx = b.idx; mp.M = M; mp.top = s.top; mp.experts = s.experts;
        if (!stream) {
            mp.grouped256 = moe_grouped256(M, s.top, s.experts, 2 * L.ffp, Wp) && moe_grouped256(M, s.top, s.experts, Wp, L.ffp);
            const int tile_m = mp.grouped256 ? 256 : MOE_TILE_M;
            CR_TRY(launch_lm_plan(L, M, tile_m, b.idx, b.perm, b.tiles, b.n_tiles, st));
            mp.tiles = b.tiles; mp.n_tiles = b.n_tiles; mp.max_tiles = lm_max_tiles(M * s.top, s.experts, tile_m); mp.perm = b.perm;
        }
        CR_TRY(stream ? launch_moe_stream(true, mp, st) : launch_moe_tiled(true, mp, st));
        mp.A = (const bf16*)b.act; mp.lda = L.ffp; mp.W = (const bf16*)L.wdn; mp.w_es = (int64_t)Wp * L.ffp; mp.C = (bf16*)b.ye; mp.ldc = Wp; mp.N = Wp; mp.K = L.ffp;
        mp.gather_div = 0; mp.scatter = 1;
        CR_TRY(stream ? launch_moe_stream(false, mp, st) : launch_moe_tiled(false, mp, st));
        return CR_OK;
    }
    CR_TRY(launch_lm_plan(L, M, LM_TILE_M, b.idx, b.perm, b.tiles, b.n_tiles, st));
    LmGemmParams g{};
    g.A = b.h; g.lda = Wp; g.W = L.wgu; g.ldw = Wp; g.w_bs = (int64_t)2 * L.ffp * Wp; g.C = b.act; g.ldc = L.ffp; g.N = 2 * L.ffp; g.K = Wp;
    g.tiles = b.tiles; g.n_tiles = b.n_tiles; g.max_tiles = lm_max_tiles(M * s.top, s.experts, LM_TILE_M); g.perm = b.perm; g.gather_div = s.top; g.limit = s.limit;
    CR_TRY(launch_lm_gemm(lm.f32, LM_GLU, g, st));
    g.A = b.act; g.lda = L.ffp; g.W = L.wdn; g.ldw = L.ffp; g.w_bs = (int64_t)Wp * L.ffp; g.C = b.ye; g.ldc = Wp; g.N = Wp; g.K = L.ffp; g.gather_div = 0; g.scatter = 1;
    CR_TRY(launch_lm_gemm(lm.f32, LM_STORE, g, st));
    return CR_OK;
}

// last: where the final norm of every row goes (decode); null: the residual stays in b.x, rows are picked from it afterwards
int run_passes(cr_ctx* c, cr_kv* kv, const Step& sp, Buffers& b, void* last, hipStream_t st) {
    const Lm& lm = *c->lm;
    const int M = sp.M, Wp = lm.Wp;
    const size_t es = lm.esz();
    auto probe = [&](int slot) -> int {
        if (!c->probe_dst || sp.decode || c->probe_row0 + c->probe_rows > M) return CR_OK;
        CR_HIP(hipMemcpy2DAsync((float*)c->probe_dst + (size_t)slot * c->probe_rows * lm.d.width, (size_t)lm.d.width * 4, b.x + (size_t)c->probe_row0 * Wp, (size_t)Wp * 4,
                                (size_t)lm.d.width * 4, c->probe_rows, hipMemcpyDeviceToDevice, st));
        return CR_OK;
    };
    // what reads the residual ahead of pass r: its first norm, or the product that mixes the embedding in
    auto entry = [&](size_t r) -> LmSink {
        if (r >= lm.passes.size()) return {last, Wp, lm.fin};
        if (lm.starts[r]) return {b.cat, 2 * Wp, nullptr};
        return {b.h, Wp, lm.layers[lm.passes[r]].n1};
    };
    // y = A . W^T for launch_lm_post: fp32 K-slices where the step streams its weights, element type otherwise
    auto project = [&](const void* A, const void* W, const bf16* dl, int K, LmPostIn& out) -> int {
        const int n = slices_of(lm, M, Wp, K, sp.decode);
        out = LmPostIn{n ? (const void*)b.sl : b.y, Wp, n, nullptr, 0};
        return n ? sliced(c, A, K, W, dl, b.sl, M, Wp, K, st) : dense(c, lm, A, K, W, b.y, Wp, M, Wp, K, st, !sp.decode, dl);
    };
    CR_TRY(launch_lm_embed(lm.f32, lm, M, sp.tokens, sp.ix, kv->d_gen, kv->d_ngen, kv->gen_cap, b.x, entry(0), b.tok, lm.d.loop_in ? (char*)b.cat + (size_t)Wp * es : nullptr, 2 * Wp, st));
    CR_TRY(probe(0));
    for (size_t r = 0; r < lm.passes.size(); r++) {
        const LmLayer& L = lm.layers[lm.passes[r]];
        LmPostIn y;
        if (lm.starts[r]) {
            const LmSink to{b.h, Wp, L.n1};
            const int n = slices_of(lm, M, Wp, 2 * Wp, sp.decode);
            if (n) {
                CR_TRY(sliced(c, b.cat, 2 * Wp, lm.loop_in, lm.loop_dl, b.sl, M, Wp, 2 * Wp, st));
                CR_TRY(launch_lm_post(lm.f32, lm, M, LmPostIn{b.sl, Wp, n, nullptr, 0}, b.x, nullptr, true, to, st));
            } else {
                CR_TRY(raw32(c, lm, b.cat, lm.loop_in, b.x, Wp, M, Wp, 2 * Wp, 0.f, st, sp.decode ? lm.loop_dl : nullptr));
                CR_TRY(launch_lm_pick_rows(lm.f32, lm, M, b.x, nullptr, b.h, L.n1, st));
            }
        }
        CR_TRY(L.latent() ? latent_mixer(c, kv, sp, b, L, r, st) : heads_mixer(c, kv, sp, b, L, r, st));
        CR_TRY(project(b.ao, L.wo, L.wo_dl, L.Gp, y));
        const LmSink next = entry(r + 1), end = lm.Sp ? LmSink{b.h, Wp, nullptr} : next;
        CR_TRY(launch_lm_post(lm.f32, lm, M, y, b.x, L.n1b, false, L.s.ff == CR_FF_NONE ? end : LmSink{b.h, Wp, L.n2}, st));
        if (L.s.ff == CR_FF_DENSE) {
            CR_TRY(dense(c, lm, b.h, Wp, L.wgu, b.act, L.ffp, M, L.ffp, Wp, st, !sp.decode, L.wgu_dl, true));
            CR_TRY(project(b.act, L.wdn, L.wdn_dl, L.ffp, y));
            CR_TRY(launch_lm_post(lm.f32, lm, M, y, b.x, L.n2b, false, end, st));
        } else if (L.s.ff == CR_FF_MOE) {
            CR_TRY(expert_mixture(c, sp, b, L, st));
            CR_TRY(launch_lm_post(lm.f32, lm, M, LmPostIn{b.ye, Wp, 0, b.wt, L.s.top}, b.x, L.n2b, false, end, st));
        }
        if (lm.Sp) {
            const char* side = (const char*)lm.side + (size_t)lm.passes[r] * lm.Sp * es;
            const int64_t lds = (int64_t)lm.layers.size() * lm.Sp;
            bool projected = false;
            if (lm.f32) {
                LmGemmParams g{};
                g.A = b.h; g.lda = Wp; g.W = L.sgate; g.ldw = Wp; g.C = b.z2; g.ldc = lm.Sp; g.M = M; g.N = lm.Sp; g.K = Wp; g.gate = side; g.ldg = lds; g.tok = b.tok;
                CR_TRY(launch_lm_gemm(true, LM_SIDE, g, st));
            } else {
                // few columns: K-slices keep the chip busy, and the kernel that adds them applies the activation and the token's row
                int n = slices_of(lm, M, lm.Sp, Wp, sp.decode);
                if (n) CR_TRY(sliced(c, b.h, Wp, L.sgate, L.sgate_dl, b.sl, M, lm.Sp, Wp, st));
                else {
                    GemmParams g = slice_params(b.h, Wp, L.sgate, nullptr, b.sl, M, lm.Sp, Wp);
                    g.kernel = 128; g.group = n = side_slices(Wp);
                    CR_TRY(ctx_gemm(c, EPI_PARTIAL, g, st));
                }
                projected = sp.decode && lm_side_proj_supported(lm, M);
                if (projected) CR_TRY(launch_lm_side_proj(lm, M, b.sl, n, side, lds, b.tok, L.sproj, b.y, st));
                else CR_TRY(launch_lm_side_act(lm, M, b.sl, n, side, lds, b.tok, b.z2, st));
            }
            if (projected) y = LmPostIn{b.y, Wp, 0, nullptr, 0};
            else CR_TRY(project(b.z2, L.sproj, L.sproj_dl, lm.Sp, y));
            CR_TRY(launch_lm_post(lm.f32, lm, M, y, b.x, L.ns, false, next, st));
        }
        CR_TRY(probe((int)r + 1));
    }
    return CR_OK;
}

// final norm of n rows of x (device indices), then the logits, in pieces that fit `hl`
int lm_head(cr_ctx* c, const Lm& lm, const float* x, const int32_t* rows, int n, void* hl, int piece, float* out, hipStream_t st) {
    for (int i = 0; i < n; i += piece) {
        const int m = std::min(piece, n - i);
        CR_TRY(launch_lm_pick_rows(lm.f32, lm, m, x, rows + i, hl, lm.fin, st));
        CR_TRY(raw32(c, lm, hl, lm.head, out + (size_t)i * lm.d.vocab, lm.d.vocab, m, lm.d.vocab, lm.Wp, lm.d.softcap, st));
    }
    return CR_OK;
}

}  // namespace

int lm_finalize(cr_ctx* c, hipStream_t st) {
    // derived once; the checkpoint's tensors are released (they are all there again when a model is loaded anew)
    if (!c->w.count("embed")) return c->lm->embed ? CR_OK : cr_fail(CR_ERR_STATE, "described decoder: weight 'embed' was never loaded");
    auto lm = std::make_shared<Lm>(*c->lm);
    Deriver dv{c, *lm, st, {}};
    const bool tied = lm->d.tied_head != 0;
    const DevTensor *e = dv.src("embed", lm->d.vocab, lm->d.width), *h = tied ? e : dv.src("head", lm->d.vocab, lm->d.width);
    lm->fin = dv.gain("derived.lm.final", "final.norm", lm->d.width, lm->Wp, lm->gain_base());
    if (!e || !h || !lm->fin) return CR_ERR_STATE;
    lm->embed = dv.mat("derived.lm.embed", (size_t)lm->d.vocab * lm->Wp);
    lm->head = tied ? lm->embed : dv.mat("derived.lm.head", (size_t)lm->d.vocab * lm->Wp);
    if (!lm->embed || !lm->head) return CR_ERR_NOMEM;
    CR_TRY(dv.place(e, 0, lm->d.vocab, lm->embed, 0, lm->Wp));
    if (!tied) CR_TRY(dv.place(h, 0, lm->d.vocab, lm->head, 0, lm->Wp));
    if (lm->Sp) {                                             // a layer's part of a token's row, padded
        const int n = (int)lm->layers.size(), D = lm->d.side_dim;
        const DevTensor* t = dv.src("side.embed", lm->d.vocab, (int64_t)n * D);
        if (!t || !(lm->side = dv.mat("derived.lm.side", (size_t)lm->d.vocab * n * lm->Sp))) return CR_ERR_STATE;
        CR_TRY(dv.place(t, 0, lm->d.vocab, lm->side, 0, Place{(int64_t)n * lm->Sp, 1, 0, 0, 0, D, lm->Sp}));
    }
    if (lm->d.loop_in) {
        const DevTensor* t = dv.src("loop.in", lm->d.width, (int64_t)2 * lm->d.width);
        if (!t || !(lm->loop_in = dv.mat("derived.lm.loop", (size_t)lm->Wp * 2 * lm->Wp))) return CR_ERR_STATE;
        CR_TRY(dv.place(t, 0, lm->d.width, lm->loop_in, 0, Place{(int64_t)2 * lm->Wp, 1, 0, 0, 0, lm->d.width, lm->Wp}));
        lm->loop_dl = dv.swizzled("derived.lm.loop.dl", lm->loop_in, lm->Wp, 2 * lm->Wp);
    }
    lm->head_dl = dv.swizzled("derived.lm.head.dl", lm->head, lm->d.vocab, lm->Wp);
    if (lm->d.pos == CR_POS_SINUSOID) {
        const int n = (lm->Wp + 1) / 2;
        std::vector<float> f(n, 0.f);
        for (int i = 0; i < n; i++) f[i] = (float)pow((double)lm->d.pos_base, -2.0 * i / lm->d.width);
        lm->freq = (float*)dv.make("derived.lm.freq", n, 4, CR_F32);
        if (!lm->freq) return CR_ERR_NOMEM;
        CR_HIP(hipMemcpyAsync(lm->freq, f.data(), (size_t)n * 4, hipMemcpyHostToDevice, st));
        CR_HIP(hipStreamSynchronize(st));
    }
    for (size_t i = 0; i < lm->layers.size(); i++) CR_TRY(derive_layer(dv, (int)i, lm->layers[i]));
    CR_HIP(hipStreamSynchronize(st));
    for (const std::string& n : dv.used) {
        auto it = c->w.find(n);
        if (it == c->w.end()) continue;
        hipFree(it->second.ptr);
        c->w.erase(it);
    }
    c->lm = lm;
    return CR_OK;
}

int lm_kv_alloc(const Lm& lm, cr_kv* kv) {
    size_t off = 0;
    auto take = [&](size_t bytes) { const size_t at = off; off += (bytes + 255) & ~(size_t)255; return at; };
    for (int l : lm.passes) {
        const LmLayer& L = lm.layers[l];
        const size_t n = kv->n_seqs;
        kv->lat_off.push_back(L.latent() ? take(n * kv->max_tokens * L.Rp * lm.esz())
                              : take(L.heads() ? 2 * n * L.s.attn.kv_heads * std::min(lm.chunks[L.chunk_ix], kv->max_tokens) * L.Ap * lm.esz() : 0));
        kv->state_off.push_back(take(L.retention() ? n * L.s.ret.heads * L.Vp * L.Kp * 4 : 0));
    }
    if (hipMalloc((void**)&kv->lat, off) != hipSuccess) return cr_fail(CR_ERR_NOMEM, "cr_kv_alloc: %zu bytes of cache", off);
    // rows past a sequence's length are read (with weight zero) by tiles that end behind it: they must be numbers.  (States need no clearing: position 0 starts from zero.)
    CR_HIP(hipMemset(kv->lat, 0, off));
    return CR_OK;
}

// one greedy step for n sequences whose ids are staged in kv->d_seqs (llm.hip: cr_llm_decode validates, advances the lengths)
int lm_decode_step(cr_ctx* c, cr_kv* kv, int n, const int64_t* force_tokens, float penalty, float* logits, hipStream_t st) {
    const Lm& lm = *c->lm;
    int longest = 0, heads = 1;
    int64_t keys = 0;
    for (int32_t s : kv->seqs_on_device) { longest = std::max(longest, kv->len[s] + 1); keys += kv->len[s] + 1; }
    for (const LmLayer& L : lm.layers) if (L.latent()) heads = std::max(heads, (int)L.s.heads);
    Step sp{};
    sp.M = n; sp.decode = true; sp.tokens = force_tokens; sp.ix.seqs = kv->d_seqs; sp.ix.lens = kv->d_len;
    sp.split = latent_split_keys(heads, keys); sp.nsplit = (longest + sp.split - 1) / sp.split;
    for (int chunk : lm.chunks) {
        int most = 0;
        for (int32_t s : kv->seqs_on_device) most = std::max(most, kv->len[s] % chunk + 1);
        sp.hsplit.push_back((most + HEADS_SPLIT - 1) / HEADS_SPLIT);
    }
    const size_t cb = carve_bytes(lm, sp);
    CR_TRY(ws_ensure(c, cb + (size_t)n * lm.Wp * lm.esz() + (size_t)n * lm.d.vocab * 4 + 1024));
    Arena ar(c->ws);
    Buffers b = carve(lm, ar, sp);
    void* hl = ar.take<char>((size_t)n * lm.Wp * lm.esz());
    float* lg = ar.take<float>((size_t)n * lm.d.vocab);
    CR_TRY(run_passes(c, kv, sp, b, hl, st));
    CR_TRY(raw32(c, lm, hl, lm.head, lg, lm.d.vocab, n, lm.d.vocab, lm.Wp, lm.d.softcap, st, lm.head_dl));
    if (logits) CR_HIP(hipMemcpyAsync(logits, lg, (size_t)n * lm.d.vocab * 4, hipMemcpyDeviceToDevice, st));
    return launch_pick(lg, lm.d.vocab, lm.d.vocab, penalty, n, kv->d_seqs, kv, 1, st);
}

namespace {

int size_latent(int i, LmLayer& L) {
    const cr_lm_layer& s = L.s;
    if (s.heads <= 0 || s.dim <= 0 || s.vdim <= 0 || s.q_rank <= 0 || s.kv_rank <= 0 || s.kv_rank > 2048)
        return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: heads %d, dim %d, vdim %d, q_rank %d, kv_rank %d (at most 2048)", i, s.heads, s.dim, s.vdim, s.q_rank, s.kv_rank);
    const int m = std::max(s.dim, s.vdim);
    L.Ap = m <= 64 ? 64 : m <= 128 ? 128 : m <= 256 ? 256 : lm_pad64(m);
    L.Rp = s.kv_rank <= 64 ? 64 : s.kv_rank <= 128 ? 128 : s.kv_rank <= 256 ? 256 : s.kv_rank <= 512 ? 512 : lm_pad64(s.kv_rank);
    L.Qp = lm_pad64(s.q_rank); L.Gp = lm_pad64(s.heads * s.vdim);
    L.off_c = L.Qp; L.off_g = L.Qp + L.Rp; L.Na = L.Qp + L.Rp + L.Gp;
    return CR_OK;
}

int size_heads(int i, Lm& lm, LmLayer& L) {
    const cr_lm_heads& a = L.s.attn;
    const cr_lm_retention& r = L.s.ret;
    if ((L.s.mixer & ~(CR_MIX_HEADS | CR_MIX_RETENTION)) || !L.s.mixer) return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: mixer %d", i, L.s.mixer);
    auto bad_rot = [](int dims, int dim, double base) { return dims < 0 || dims % 2 || dims > dim || (dims && !(base > 0.0)); };
    std::vector<LmRegion> reg;
    if (L.heads()) {
        if (a.heads <= 0 || a.kv_heads <= 0 || a.heads % a.kv_heads || a.dim <= 0 || a.vdim <= 0 || std::max(a.dim, a.vdim) > LM_MAX_HEAD || a.chunk < 0 || bad_rot(a.rot_dims, a.dim, a.rot_base))
            return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: heads %d / %d, dim %d, vdim %d (at most %d), chunk %d, rotated %d", i, a.heads, a.kv_heads, a.dim, a.vdim, LM_MAX_HEAD, a.chunk, a.rot_dims);
        L.Ap = lm_pad_head(std::max(a.dim, a.vdim));
        reg.push_back({LM_Q, 0, a.heads, L.Ap}); reg.push_back({LM_K, 0, a.kv_heads, L.Ap}); reg.push_back({LM_V, 0, a.kv_heads, L.Ap});
        L.off_r = lm_pad64(a.heads * a.vdim);
        const int chunk = a.chunk > 0 ? a.chunk : INT32_MAX;
        L.chunk_ix = (int)(std::find(lm.chunks.begin(), lm.chunks.end(), chunk) - lm.chunks.begin());
        if (L.chunk_ix == (int)lm.chunks.size()) lm.chunks.push_back(chunk);
    }
    L.Gp = L.off_r;
    if (L.retention()) {
        if (r.heads <= 0 || r.dim <= 0 || r.vdim <= 0 || std::max(r.dim, r.vdim) > LM_MAX_HEAD || !r.decay || bad_rot(r.rot_dims, r.dim, r.rot_base))
            return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: retention heads %d, dim %d, vdim %d (at most %d), rotated %d", i, r.heads, r.dim, r.vdim, LM_MAX_HEAD, r.rot_dims);
        L.Kp = lm_pad_head(r.dim); L.Vp = lm_pad_head(r.vdim);
        reg.push_back({LM_RQ, 0, r.heads, L.Kp}); reg.push_back({LM_RK, 0, r.heads, L.Kp}); reg.push_back({LM_RV, 0, r.heads, L.Vp}); reg.push_back({LM_RG, 0, r.heads, L.Vp});
        L.Gp += lm_pad64(r.heads * r.vdim);
        L.decay.assign(r.decay, r.decay + r.heads);
        L.s.ret.decay = nullptr;                              // (the caller's array)
    }
    std::stable_sort(reg.begin(), reg.end(), [](const LmRegion& x, const LmRegion& y) { return x.P > y.P; });
    L.n_regions = (int)reg.size();
    for (int k = 0; k < L.n_regions; k++) { reg[k].off = L.Na; L.Na += reg[k].heads * reg[k].P; L.regions[k] = reg[k]; }
    return CR_OK;
}

// the key plan of one chunk size, appended to the upload `hv` (offsets until the upload has an address)
struct KeyPlanAt { KeyPlan k; size_t row_key, row_slot, pieces, pre_key, pre_slot; };
KeyPlanAt plan_keys(const Step& sp, int chunk, int max_tokens, std::vector<int32_t>& hv) {
    KeyPlanAt o{};
    o.k.ring = std::min(chunk, max_tokens);
    std::vector<int32_t> key, slot, pieces, pk, ps;
    int base = 0;
    for (const Step::Seg& g : sp.segs) {
        const int pre = g.pos0 % chunk, last_chunk = (g.pos0 + g.S - 1) / chunk;
        for (int i = 0; i < pre; i++) { pk.push_back(base + i); ps.push_back(g.seq * o.k.ring + i); }
        for (int t = 0; t < g.S; t++) {
            const int pos = g.pos0 + t;
            key.push_back(base + pre + t);
            slot.push_back(pos / chunk == last_chunk ? g.seq * o.k.ring + pos % chunk : -1);
        }
        for (int t = 0; t < g.S;) {
            const int at = (g.pos0 + t) % chunk, n = std::min(g.S - t, chunk - at);
            for (int32_t v : {g.row0 + t, n, at, base + pre + t - at}) pieces.push_back(v);
            o.k.longest = std::max(o.k.longest, n);
            t += n;
        }
        base += pre + g.S;
    }
    o.k.Mk = base; o.k.n_pieces = (int)pieces.size() / 4; o.k.n_pre = (int)pk.size();
    auto put = [&](const std::vector<int32_t>& v) { const size_t at = hv.size(); hv.insert(hv.end(), v.begin(), v.end()); return at; };
    o.row_key = put(key); o.row_slot = put(slot); o.pieces = put(pieces); o.pre_key = put(pk); o.pre_slot = put(ps);
    return o;
}

}  // namespace

extern "C" {

int cr_lm_configure(cr_ctx* c, const cr_lm_desc* d, const cr_lm_layer* layers) {
    if (!c || !d || !layers || d->layers <= 0 || d->width <= 0 || d->vocab <= 0) return cr_fail(CR_ERR_ARG, "cr_lm_configure: bad argument");
    if (d->dtype != CR_BF16 && d->dtype != CR_F32) return cr_fail(CR_ERR_ARG, "cr_lm_configure: dtype %d", d->dtype);
    if (d->width > 16384) return cr_fail(CR_ERR_ARG, "cr_lm_configure: width %d (at most 16384)", d->width);
    if (c->borrowed) return cr_fail(CR_ERR_STATE, "cr_lm_configure: this context borrows its weights");
    auto lm = std::make_shared<Lm>();
    lm->d = *d; lm->f32 = d->dtype == CR_F32; lm->Wp = lm_pad64(d->width); lm->Vp = lm_pad64(d->vocab); lm->Sp = d->side_dim > 0 ? lm_pad64(d->side_dim) : 0;
    if (d->loop_times <= 0) lm->d.loop_in = 0;
    for (int i = 0; i < d->layers; i++) {
        LmLayer L{};
        L.s = layers[i];
        const cr_lm_layer& s = L.s;
        CR_TRY(s.mixer == CR_MIX_LATENT ? size_latent(i, L) : size_heads(i, *lm, L));
        if (s.ff == CR_FF_MOE) {
            if (s.experts <= 0 || s.experts > 1024 || s.top <= 0 || s.expert_ff <= 0 || s.groups <= 0 || s.experts % s.groups || s.keep <= 0 || s.keep > s.groups ||
                s.top > s.keep * (s.experts / s.groups))
                return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: %d experts (at most 1024), top %d, %d groups, keep %d", i, s.experts, s.top, s.groups, s.keep);
            L.ffp = lm_pad64(s.expert_ff); L.Ep = lm_pad64(s.experts);
        } else if (s.ff == CR_FF_DENSE) {
            if (s.expert_ff <= 0 || s.act != CR_ACT_RELU2) return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: feed-forward width %d, activation %d", i, s.expert_ff, s.act);
            L.ffp = lm_pad64(s.expert_ff);
        } else if (s.ff != CR_FF_NONE) return cr_fail(CR_ERR_ARG, "cr_lm_configure: layer %d: feed-forward %d", i, s.ff);
        lm->layers.push_back(L);
    }
    if (d->loop_times > 0 && (d->loop_start < 0 || d->loop_stop > d->layers || d->loop_start >= d->loop_stop))
        return cr_fail(CR_ERR_ARG, "cr_lm_configure: loop %d .. %d x %d of %d layers", d->loop_start, d->loop_stop, d->loop_times, d->layers);
    const int a = d->loop_times > 0 ? d->loop_start : d->layers, z = d->loop_times > 0 ? d->loop_stop : d->layers;
    for (int i = 0; i < a; i++) lm->passes.push_back(i);
    for (int t = 0; t < (d->loop_times > 0 ? d->loop_times : 0); t++)
        for (int i = a; i < z; i++) lm->passes.push_back(i);
    for (int i = z; i < d->layers; i++) lm->passes.push_back(i);
    lm->starts.assign(lm->passes.size(), 0);
    if (lm->d.loop_in)
        for (int t = 0; t < d->loop_times; t++) lm->starts[a + t * (z - a)] = 1;
    c->lm = lm;
    c->d.vocab = d->vocab;
    c->finalized = false;
    cr_bump_gen(c);
    return CR_OK;
}

int cr_lm_passes(const cr_ctx* c) { return c && c->lm ? (int)c->lm->passes.size() : 0; }

int cr_llm_prefill_tokens(cr_ctx* c, cr_kv* kv, const int32_t* seqs, int n, const int64_t* tokens, const int32_t* lens, float penalty, float* last_logits, const int32_t* want, int n_want,
                          float* want_logits, void* stream) {
    if (!c || !kv || !seqs || !lens || !tokens || n <= 0 || n > kv->n_seqs || n_want < 0 || (n_want && (!want || !want_logits))) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: bad argument");
    if (!c->lm) return cr_fail(CR_ERR_STATE, "cr_llm_prefill_tokens: the context has no described decoder (cr_lm_configure)");
    if (!c->finalized) return cr_fail(CR_ERR_STATE, "cr_llm_prefill_tokens: call cr_finalize first");
    CR_TRY(ctx_share_ok(c, "cr_llm_prefill_tokens"));
    const Lm& lm = *c->lm;
    Step sp{};
    sp.fresh = true;
    for (int i = 0; i < n; i++) {
        const int s = seqs[i];
        if (s < 0 || s >= kv->n_seqs || lens[i] <= 0) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: bad sequence %d / length %d", s, lens[i]);
        for (int j = 0; j < i; j++) if (seqs[j] == s) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: sequence %d listed twice", s);
        if (kv->len[s] + lens[i] > kv->max_tokens) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: %d + %d tokens exceed the cache (%d)", kv->len[s], lens[i], kv->max_tokens);
        sp.segs.push_back({sp.M, lens[i], kv->len[s], s, sp.Mk});
        sp.fresh = sp.fresh && kv->len[s] == 0;
        sp.M += lens[i]; sp.Mk += kv->len[s] + lens[i];
    }
    const int M = sp.M;
    for (int i = 0; i < M; i++) if (tokens[i] < 0 || tokens[i] >= lm.d.vocab) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: token id %lld outside the vocabulary", (long long)tokens[i]);
    for (int i = 0; i < n_want; i++) if (want[i] < 0 || want[i] >= M) return cr_fail(CR_ERR_ARG, "cr_llm_prefill_tokens: row %d of %d asked for", want[i], M);
    CR_HIP(hipSetDevice(c->device));
    hipStream_t st = (hipStream_t)stream;
    const int V = lm.d.vocab, piece = std::max(n, std::min(std::max(n_want, 1), 4096));
    // one host-to-device copy: tokens, then per row sequence and position, per segment its bounds (two orders), the last rows, first retention chunks, the rows asked for, the chunks, key plans
    const size_t fixed = (size_t)M * 4 + (size_t)n * 10 + n_want;
    std::vector<int32_t> hv(fixed);
    memcpy(hv.data(), tokens, (size_t)M * 8);
    int32_t *h_seq = hv.data() + 2 * (size_t)M, *h_pos = h_seq + M, *h_seg = h_pos + M, *h_rseg = h_seg + 4 * n, *h_last = h_rseg + 4 * n, *h_snap = h_last + n, *h_want = h_snap + n;
    for (int i = 0; i < n; i++) {
        const Step::Seg& sg = sp.segs[i];
        for (int r = 0; r < sg.S; r++) { h_seq[sg.row0 + r] = sg.seq; h_pos[sg.row0 + r] = sg.pos0 + r; }
        const int32_t b0[4] = {sg.row0, sg.S, sg.pos0, sg.key0}, b1[4] = {sg.row0, sg.S, sg.pos0, sg.seq};
        memcpy(h_seg + 4 * i, b0, 16);
        memcpy(h_rseg + 4 * i, b1, 16);
        h_last[i] = sg.row0 + sg.S - 1;
        h_snap[i] = sp.snaps;
        sp.snaps += ret_chunks(sg.S);
        sp.longest = std::max(sp.longest, sg.S);
    }
    if (n_want) memcpy(h_want, want, (size_t)n_want * 4);
    const size_t at_chunks = hv.size();
    for (const Step::Seg& sg : sp.segs)
        for (int t = 0; t < sg.S; t += RET_CHUNK) { hv.push_back(sg.row0 + t); hv.push_back(std::min(RET_CHUNK, sg.S - t)); }
    std::vector<KeyPlanAt> at;
    for (int chunk : lm.chunks) { at.push_back(plan_keys(sp, chunk, kv->max_tokens, hv)); sp.plans.push_back(at.back().k); }
    CR_TRY(ws_ensure(c, carve_bytes(lm, sp) + (size_t)piece * lm.Wp * lm.esz() + (size_t)n * V * 4 + hv.size() * 4 + 8192));
    Arena ar(c->ws);
    Buffers b = carve(lm, ar, sp);
    void* hl = ar.take<char>((size_t)piece * lm.Wp * lm.esz());
    float* lg = ar.take<float>((size_t)n * V);
    int32_t* dv = ar.take<int32_t>(hv.size());
    CR_HIP(hipMemcpyAsync(dv, hv.data(), hv.size() * 4, hipMemcpyHostToDevice, st));       // pageable source: staged before return
    CR_HIP(hipMemcpyAsync(kv->d_seqs, seqs, (size_t)n * 4, hipMemcpyHostToDevice, st));
    kv->seqs_on_device.assign(seqs, seqs + n);
    sp.tokens = (const int64_t*)dv;
    sp.ix.row_seq = dv + 2 * (size_t)M; sp.ix.row_pos = sp.ix.row_seq + M; sp.d_seg = sp.ix.row_pos + M; sp.d_rseg = sp.d_seg + 4 * n;
    const int32_t *d_last = sp.d_rseg + 4 * n, *d_want = d_last + 2 * n;
    sp.d_snap0 = d_last + n; sp.d_chunks = dv + at_chunks;
    for (size_t i = 0; i < at.size(); i++) {
        KeyPlan& k = sp.plans[i];
        k.row_key = dv + at[i].row_key; k.row_slot = dv + at[i].row_slot; k.pieces = dv + at[i].pieces; k.pre_key = dv + at[i].pre_key; k.pre_slot = dv + at[i].pre_slot;
    }
    CR_TRY(run_passes(c, kv, sp, b, nullptr, st));
    if (n_want) CR_TRY(lm_head(c, lm, b.x, d_want, n_want, hl, piece, want_logits, st));
    CR_TRY(lm_head(c, lm, b.x, d_last, n, hl, piece, lg, st));
    if (last_logits) CR_HIP(hipMemcpyAsync(last_logits, lg, (size_t)n * V * 4, hipMemcpyDeviceToDevice, st));
    CR_TRY(launch_pick(lg, V, V, penalty, n, kv->d_seqs, kv, 0, st));
    for (const Step::Seg& sg : sp.segs) {
        kv->len[sg.seq] += sg.S;
        if (kv->ngen[sg.seq] < kv->gen_cap) kv->ngen[sg.seq] += 1;
    }
    CR_HIP(hipMemcpyAsync(kv->d_len, kv->len.data(), (size_t)kv->n_seqs * 4, hipMemcpyHostToDevice, st));
    return CR_OK;
}

}  // extern "C"
