// Attention over grouped heads and retention, the parts around their cores: one kernel turns a row of the fused input projection into normed, rotated queries and keys, cache rows
// and retention operands; a copy kernel fetches the cached start of a chunk; an attention kernel for any size and type (the matrix-core forms are in attention.hip).
//
// Row kernel: a wave holds 512 columns, eight per lane.  A head's padded size is a power of two (64 .. 512) and regions are laid out widest first, so a head is a run of lanes of
// one wave: its norm is a lane reduction, its rotation partner (half a rotation away, at any distance) comes through 2 KiB of the wave's own LDS.  Angles are fp32 and are
// computed once per row.
#include "lm.hpp"

namespace {

template <typename T> __device__ __forceinline__ void ld8(const T* p, float (&v)[8]);
template <> __device__ __forceinline__ void ld8<bf16>(const bf16* p, float (&v)[8]) {
    const bf16x8 x = *(const bf16x8*)p;
#pragma unroll
    for (int e = 0; e < 8; e++) v[e] = (float)x[e];
}
template <> __device__ __forceinline__ void ld8<float>(const float* p, float (&v)[8]) {
    const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
    for (int e = 0; e < 4; e++) { v[e] = a[e]; v[4 + e] = b[e]; }
}
__device__ __forceinline__ void st8(bf16* p, const float (&v)[8]) {
    bf16x8 x;
#pragma unroll
    for (int e = 0; e < 8; e++) x[e] = (bf16)v[e];
    *(bf16x8*)p = x;
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
    *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]};
    *(f32x4*)(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}

struct HeadsArgs {
    LmHeadsIn in;
    int M, Na, n_regions;
    LmRegion reg[LM_REGIONS];
    float eps, k_scale;
    int dim, G, Ap, half_a, half_r;              // half a rotation's entries, 0 = no rotation
    const float *nq, *nk, *fq_a, *fq_r;          // nq null: no query / key norm
    int pad0, pad1, pad2, pad3, ldo;             // columns [pad0, pad1) and [pad2, pad3) of `ao` are padding
    int64_t rplane;                              // elements of one term of rq2 / rk2
};

template <typename T>
__global__ __launch_bounds__(256) void lm_heads_kernel(const HeadsArgs p) {
    __shared__ float cs[2][2][LM_MAX_HEAD / 2];              // [attention, retention][cos, sin][pair]
    __shared__ __attribute__((aligned(16))) float sx[4][512];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int64_t row = blockIdx.x;
    const int seq = p.in.ix.row_seq ? p.in.ix.row_seq[row] : p.in.ix.seqs[row];
    const int pos = p.in.ix.row_pos ? p.in.ix.row_pos[row] : p.in.ix.lens[seq];
    for (int i = tid; i < p.half_a + p.half_r; i += 256) {
        const bool r = i >= p.half_a;
        const int j = r ? i - p.half_a : i;
        float s, c;
        sincosf((float)pos * (r ? p.fq_r[j] : p.fq_a[j]), &s, &c);
        cs[r][0][j] = c; cs[r][1][j] = s;
    }
    if (blockIdx.y == 0) {
        T* ao = (T*)p.in.ao + row * p.ldo;
        for (int i = p.pad0 + tid; i < p.pad1; i += 256) ao[i] = (T)0.f;
        for (int i = p.pad2 + tid; i < p.pad3; i += 256) ao[i] = (T)0.f;
    }
    __syncthreads();
    const int64_t slot = p.in.row_slot ? p.in.row_slot[row] : (int64_t)seq * p.in.ring + pos % p.in.chunk;      // cache row, < 0: not kept
    const int64_t crow = slot >= 0 && p.in.ring > 0 ? slot / p.in.ring * p.G * p.in.ring + slot % p.in.ring : 0;
    for (int t = blockIdx.y * 4 + wave; t * 512 < p.Na; t += gridDim.y * 4) {
        const int col = t * 512 + lane * 8;
        LmRegion rg{-1, 0, 0, 64};
#pragma unroll
        for (int i = 0; i < LM_REGIONS; i++)
            if (i < p.n_regions && col >= p.reg[i].off && col < p.reg[i].off + p.reg[i].heads * p.reg[i].P) rg = p.reg[i];
        const int at = col - rg.off, e0 = at & (rg.P - 1), head = at / rg.P;
        const bool raw = rg.kind == LM_RV || rg.kind == LM_RG;
        float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (rg.kind >= 0) {
            if (p.in.part) {
                for (int k = 0; k < p.in.slices; k++) {
                    float w[8];
                    ld8<float>(p.in.part + ((int64_t)k * p.M + row) * p.Na + col, w);
#pragma unroll
                    for (int e = 0; e < 8; e++) v[e] += w[e];
                }
            } else if (!raw) ld8<T>((const T*)p.in.a + row * p.in.lda + col, v);
        }
        // the norm of a query or key head
        const float* gain = rg.kind == LM_Q ? p.nq : rg.kind == LM_K ? p.nk : nullptr;
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; e++) ss += v[e] * v[e];
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const float other = __shfl_xor(ss, o, 64);
            ss += o < rg.P / 8 ? other : 0.f;
        }
        if (gain) {
            const float rs = 1.0f / sqrtf(ss / (float)p.dim + p.eps);
            float g[8];
            ld8<float>(gain + e0, g);
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] *= rs * g[e];
        }
        // the rotation: partners through LDS
        st8(&sx[wave][lane * 8], v);
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
        const bool rq = rg.kind == LM_RQ || rg.kind == LM_RK;
        const int half = rg.kind == LM_Q || rg.kind == LM_K ? p.half_a : rq ? p.half_r : 0;
        if (e0 < 2 * half) {
            const float *c = cs[rq][0], *s = cs[rq][1];
            if (half % 8 == 0) {
                const bool first = e0 < half;
                const int i = first ? e0 : e0 - half;
                float u[8], cc[8], sn[8];
                ld8<float>(&sx[wave][lane * 8 + (first ? half : -half)], u);
                ld8<float>(c + i, cc);
                ld8<float>(s + i, sn);
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = first ? v[e] * cc[e] - u[e] * sn[e] : v[e] * cc[e] + u[e] * sn[e];
            } else {
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const int q = e0 + e;
                    if (q < half) v[e] = v[e] * c[q] - sx[wave][lane * 8 + e + half] * s[q];
                    else if (q < 2 * half) v[e] = v[e] * c[q - half] + sx[wave][lane * 8 + e - half] * s[q - half];
                }
            }
        }
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();                        // (the next round overwrites sx)
        if (rg.kind == LM_Q) st8((T*)p.in.q + row * ((int64_t)rg.heads * rg.P) + at, v);
        else if (rg.kind == LM_K || rg.kind == LM_V) {
            if (p.in.kv) st8((T*)p.in.kv + ((int64_t)p.in.row_key[row] * 2 + (rg.kind == LM_V)) * p.G * p.Ap + at, v);
            if (slot >= 0) st8((T*)(rg.kind == LM_K ? p.in.cache_k : p.in.cache_v) + (crow + (int64_t)head * p.in.ring) * p.Ap + e0, v);
        } else if (rq) {
            if (rg.kind == LM_RK) {
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] *= p.k_scale;
            }
            const int64_t o = row * ((int64_t)rg.heads * rg.P) + at;
            if (p.in.rq2) {
                bf16* d = (rg.kind == LM_RQ ? p.in.rq2 : p.in.rk2) + o;
                float lo[8];
#pragma unroll
                for (int e = 0; e < 8; e++) lo[e] = v[e] - rbf(v[e]);
                st8(d, v);
                st8(d + p.rplane, lo);
            } else st8((rg.kind == LM_RQ ? p.in.rq : p.in.rk) + o, v);
        } else if (raw && p.in.part) st8((T*)const_cast<void*>(p.in.a) + row * p.in.lda + col, v);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void lm_prefix_kernel(const int32_t* __restrict__ key_rows, const int32_t* __restrict__ cache_rows, T* __restrict__ kv, const T* __restrict__ ck,
                                                        const T* __restrict__ cv, int G, int Ap, int ring) {
    const int64_t k = key_rows[blockIdx.x], slot = cache_rows[blockIdx.x];
    const int64_t crow = slot / ring * G * ring + slot % ring;
    for (int i = threadIdx.x * 8; i < G * Ap; i += 2048) {
        const int64_t src = (crow + (int64_t)(i / Ap) * ring) * Ap + i % Ap;
        float a[8], b[8];
        ld8<T>(ck + src, a);
        ld8<T>(cv + src, b);
        st8(kv + k * 2 * G * Ap + i, a);
        st8(kv + (k * 2 + 1) * G * Ap + i, b);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void heads_attn_plain_kernel(const HeadsAttnParams p) {
    __shared__ float q[LM_MAX_HEAD], w[256], red[8];
    const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    const int g = head / (p.H / p.G);
    const int seq = p.ix.row_seq ? p.ix.row_seq[row] : p.ix.seqs[row];
    const int n = (p.ix.row_pos ? p.ix.row_pos[row] : p.ix.lens[seq]) % p.chunk + 1;
    const int64_t base = p.row_key ? (int64_t)(p.row_key[row] - n + 1) * p.k_rs + g * p.k_hs : ((int64_t)seq * p.G + g) * p.ring * p.Ap;
    const T *Q = (const T*)p.Q + ((int64_t)row * p.H + head) * p.Ap, *K = (const T*)p.K + base, *V = (const T*)p.V + base;
    for (int i = tid; i < p.Ap; i += 256) q[i] = (float)Q[i];
    float acc[LM_MAX_HEAD / 256] = {0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;
    for (int k0 = 0; k0 < n; k0 += 256) {
        __syncthreads();
        const int key = k0 + tid;
        float s = -INFINITY;
        if (key < n) {
            const T* c = K + (int64_t)key * p.k_rs;
            float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
            for (int i = 0; i < p.Ap; i += 4) { d0 += q[i] * (float)c[i]; d1 += q[i + 1] * (float)c[i + 1]; d2 += q[i + 2] * (float)c[i + 2]; d3 += q[i + 3] * (float)c[i + 3]; }
            s = ((d0 + d1) + (d2 + d3)) * p.scale;
            if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
        }
        const float mx = wave_max(s);
        if ((tid & 63) == 0) red[tid >> 6] = mx;
        __syncthreads();
        const float m_new = fmaxf(m_run, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float e = key < n ? expf(s - m_new) : 0.f;
        w[tid] = e;
        const float sum = wave_sum(e);
        if ((tid & 63) == 0) red[4 + (tid >> 6)] = sum;
        __syncthreads();
        const float alpha = expf(m_run - m_new);
        l_run = l_run * alpha + (red[4] + red[5] + red[6] + red[7]);
        m_run = m_new;
        const int nk = min(256, n - k0);
#pragma unroll
        for (int j = 0; j < LM_MAX_HEAD / 256; j++) {
            const int i = tid + 256 * j;
            if (i >= p.vdim) break;
            float a = acc[j] * alpha;
            const T* c = V + (int64_t)k0 * p.k_rs + i;
            for (int k = 0; k < nk; k++) a += w[k] * (float)c[(int64_t)k * p.k_rs];
            acc[j] = a;
        }
    }
    T* O = (T*)p.O + (int64_t)row * p.ldo + (int64_t)head * p.vdim;
#pragma unroll
    for (int j = 0; j < LM_MAX_HEAD / 256; j++) {
        const int i = tid + 256 * j;
        if (i < p.vdim) O[i] = (T)(acc[j] * (p.out_scale / l_run));
    }
}

}  // namespace

int launch_lm_heads(bool f32, const Lm& lm, const LmLayer& L, int M, const LmHeadsIn& in, hipStream_t st) {
    const cr_lm_heads& a = L.s.attn;
    const cr_lm_retention& r = L.s.ret;
    HeadsArgs p{};
    p.in = in; p.M = M; p.Na = L.Na; p.n_regions = L.n_regions;
    for (int i = 0; i < L.n_regions; i++) p.reg[i] = L.regions[i];
    p.eps = lm.d.eps; p.k_scale = r.k_scale; p.G = a.kv_heads; p.Ap = L.Ap; p.dim = a.dim;
    p.half_a = L.heads() ? a.rot_dims / 2 : 0; p.half_r = L.retention() ? r.rot_dims / 2 : 0;
    p.nq = L.nq; p.nk = L.nc; p.fq_a = L.fq_a; p.fq_r = L.fq_r;
    p.pad0 = L.heads() ? a.heads * a.vdim : 0; p.pad1 = L.off_r; p.pad2 = L.off_r + (L.retention() ? r.heads * r.vdim : 0); p.pad3 = L.Gp; p.ldo = L.Gp;
    p.rplane = (int64_t)M * r.heads * L.Kp;
    if (!L.heads()) { p.in.ring = p.in.chunk = 1; }
    const int tasks = (L.Na + 511) / 512, y = M <= 512 ? (tasks + 3) / 4 : 1;
    if (f32) hipLaunchKernelGGL(lm_heads_kernel<float>, dim3((unsigned)M, y), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(lm_heads_kernel<bf16>, dim3((unsigned)M, y), dim3(256), 0, st, p);
    CR_HIP(hipGetLastError());
    return CR_OK;
}

int launch_lm_prefix(bool f32, const LmLayer& L, int n, const int32_t* key_rows, const int32_t* cache_rows, void* kv, const void* cache_k, const void* cache_v, int ring, hipStream_t st) {
    if (n <= 0) return CR_OK;
    const int G = L.s.attn.kv_heads;
    if (f32) hipLaunchKernelGGL(lm_prefix_kernel<float>, dim3((unsigned)n), dim3(256), 0, st, key_rows, cache_rows, (float*)kv, (const float*)cache_k, (const float*)cache_v, G, L.Ap, ring);
    else hipLaunchKernelGGL(lm_prefix_kernel<bf16>, dim3((unsigned)n), dim3(256), 0, st, key_rows, cache_rows, (bf16*)kv, (const bf16*)cache_k, (const bf16*)cache_v, G, L.Ap, ring);
    CR_HIP(hipGetLastError());
    return CR_OK;
}

int launch_heads_attn_plain(bool f32, const HeadsAttnParams& p, hipStream_t st) {
    if (p.M <= 0 || p.H <= 0 || p.G <= 0 || p.H % p.G || p.Ap <= 0 || p.Ap > LM_MAX_HEAD || p.vdim > p.Ap || p.chunk <= 0)
        return cr_fail(CR_ERR_ARG, "attention over heads: rows %d, heads %d / %d, size %d / %d", p.M, p.H, p.G, p.Ap, p.vdim);
    if (f32) hipLaunchKernelGGL(heads_attn_plain_kernel<float>, dim3(p.M, p.H), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(heads_attn_plain_kernel<bf16>, dim3(p.M, p.H), dim3(256), 0, st, p);
    CR_HIP(hipGetLastError());
    return CR_OK;
}
