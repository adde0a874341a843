// Row kernels of described decoders (lm.hpp): one workgroup per token, fp32 arithmetic throughout, the residual stream stored in fp32.  All are bound by their
// bytes; rows are padded to multiples of 64 with zeros (gains of the padding are zero), so every access is a vector of four and no tail needs a branch.
// Few rows (decode) get wide workgroups -- a thread holds four elements and every load is in flight at once; many rows get 256 threads.
#include "lm.hpp"

namespace {

template <typename T> struct Vec4;
template <> struct Vec4<float> { typedef f32x4 type; };
template <> struct Vec4<bf16> { typedef bf16x4 type; };

template <typename T> __device__ __forceinline__ f32x4 ld4(const T* p) {
    const typename Vec4<T>::type v = *(const typename Vec4<T>::type*)p;
    return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
template <typename T> __device__ __forceinline__ void st4(T* p, f32x4 v) {
    *(typename Vec4<T>::type*)p = typename Vec4<T>::type{(T)v[0], (T)v[1], (T)v[2], (T)v[3]};
}

// sum over the TPB threads; `red` holds a float per wave, two barriers
template <int TPB>
__device__ __forceinline__ float block_sum(float v, float* red, int tid) {
    v = wave_sum_s(v);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = v;
    __syncthreads();
    float s = red[0];
#pragma unroll
    for (int w = 1; w < TPB / 64; w++) s += red[w];
    return s;
}
__device__ __forceinline__ float sumsq4(f32x4 v) { return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3]; }

// h = x / sqrt(mean(x^2) + eps) * gain for a row held as NV vectors of four per thread (elements 4 tid + 4 TPB j)
template <typename T, int TPB, int NV>
__device__ __forceinline__ void norm_store(const f32x4 (&x)[NV], int Wp, int W, float eps, const float* gain, T* h, float* red, int tid) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; j++) ss += sumsq4(x[j]);
    const float rs = 1.0f / sqrtf(block_sum<TPB>(ss, red, tid) / (float)W + eps);
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        if (i < Wp) st4(h + i, x[j] * rs * *(const f32x4*)(gain + i));
    }
}

// the row for its next reader: rms(x) * gain, or x itself
template <typename T, int TPB, int NV>
__device__ __forceinline__ void sink_store(const f32x4 (&x)[NV], int Wp, int W, float eps, const LmSink& to, int64_t row, float* red, int tid) {
    if (!to.h) return;
    T* h = (T*)to.h + row * to.ldh;
    if (to.gain) { norm_store<T, TPB, NV>(x, Wp, W, eps, to.gain, h, red, tid); return; }
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        if (i < Wp) st4(h + i, x[j]);
    }
}

__device__ __forceinline__ int row_seq(const LmRowIndex& ix, int row) { return ix.row_seq ? ix.row_seq[row] : ix.seqs[row]; }
__device__ __forceinline__ int row_pos(const LmRowIndex& ix, int row) { return ix.row_pos ? ix.row_pos[row] : ix.lens[ix.seqs[row]]; }

template <typename T, int TPB, int NV>
__global__ __launch_bounds__(TPB) void lm_embed_kernel(const T* __restrict__ table, const float* __restrict__ freq, int Wp, int W, int vocab, float eps, const int64_t* __restrict__ tokens,
                                                       const LmRowIndex ix, const int64_t* __restrict__ gen, const int32_t* __restrict__ ngen, int gen_cap,
                                                       float* __restrict__ xo, const LmSink to, int32_t* __restrict__ tok, T* __restrict__ x0, int64_t ldx0) {
    __shared__ float red[TPB / 64];
    const int row = blockIdx.x, tid = threadIdx.x;
    const int seq = row_seq(ix, row);
    const float pos = (float)row_pos(ix, row);
    const int64_t t = tokens ? tokens[row] : gen[(int64_t)seq * gen_cap + ngen[seq] - 1];
    const int64_t id = t < 0 ? 0 : (t >= vocab ? vocab - 1 : t);      // (the host checks ids; a clamped read stays in bounds whatever arrives)
    if (tok && tid == 0) tok[row] = (int32_t)id;
    f32x4 x[NV];
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        x[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i >= Wp) continue;
        const f32x4 e = ld4(table + id * Wp + i);
#pragma unroll
        for (int q = 0; q < 4; q++) {
            float s = 0.f;
            if (i + q < W && freq) { const float a = pos * freq[(i + q) >> 1]; s = (q & 1) ? cosf(a) : sinf(a); }
            x[j][q] = e[q] + s;
        }
        *(f32x4*)(xo + (int64_t)row * Wp + i) = x[j];
        if (x0) st4(x0 + (int64_t)row * ldx0 + i, x[j]);
    }
    sink_store<T, TPB, NV>(x, Wp, W, eps, to, row, red, tid);
}

template <typename T, int TPB, int NV>
__global__ __launch_bounds__(TPB) void lm_post_kernel(const LmPostIn in, int M, int Wp, int W, float eps, float* __restrict__ xio,
                                                      const float* __restrict__ gain_b, int replace, const LmSink to) {
    __shared__ float red[TPB / 64];
    const int tid = threadIdx.x;
    const int64_t row = blockIdx.x;
    f32x4 y[NV], x[NV];
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        x[j] = y[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i >= Wp) continue;
        if (!replace) x[j] = *(const f32x4*)(xio + row * Wp + i);
        if (in.slices) {                                       // K-slices of a weight-streaming product, in slice order
            for (int k = 0; k < in.slices; k += 4) {
                f32x4 v[4];
#pragma unroll
                for (int q = 0; q < 4; q++) v[q] = k + q < in.slices ? *(const f32x4*)((const float*)in.Y + ((int64_t)(k + q) * M + row) * in.ldy + i) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int q = 0; q < 4; q++) y[j] += v[q];
            }
        } else if (!in.top) y[j] = ld4((const T*)in.Y + row * in.ldy + i);
        else                                                   // the row's experts, in the order they were chosen
            for (int k = 0; k < in.top; k += 4) {
                f32x4 v[4];
                float w[4];
#pragma unroll
                for (int q = 0; q < 4; q++) {
                    const int64_t a = row * in.top + min(k + q, in.top - 1);
                    v[q] = ld4((const T*)in.Y + a * in.ldy + i);
                    w[q] = k + q < in.top ? in.wt[a] : 0.f;
                }
#pragma unroll
                for (int q = 0; q < 4; q++)
                    if (k + q < in.top) y[j] += w[q] * v[q];
            }
    }
    float rs = 1.f;
    if (gain_b) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NV; j++) ss += sumsq4(y[j]);
        rs = 1.0f / sqrtf(block_sum<TPB>(ss, red, tid) / (float)W + eps);
    }
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        if (i >= Wp) continue;
        x[j] += gain_b ? y[j] * rs * *(const f32x4*)(gain_b + i) : y[j];
        *(f32x4*)(xio + row * Wp + i) = x[j];
    }
    sink_store<T, TPB, NV>(x, Wp, W, eps, to, row, red, tid);
}

template <typename T, int TPB, int NV>
__global__ __launch_bounds__(TPB) void lm_pick_rows_kernel(const float* __restrict__ X, const int32_t* __restrict__ rows, int Wp, int W, float eps, T* __restrict__ h, const float* __restrict__ gain) {
    __shared__ float red[TPB / 64];
    const int tid = threadIdx.x;
    const int64_t src = rows ? rows[blockIdx.x] : blockIdx.x;
    f32x4 x[NV];
#pragma unroll
    for (int j = 0; j < NV; j++) {
        const int i = 4 * tid + 4 * TPB * j;
        x[j] = i < Wp ? *(const f32x4*)(X + src * Wp + i) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    norm_store<T, TPB, NV>(x, Wp, W, eps, gain, h + (int64_t)blockIdx.x * Wp, red, tid);
}

// RMS norm with a plain weight over n columns of a row; writes the padded row to one or two places.  `at` reads four columns (the padding columns are zero).
template <typename T, typename F>
__device__ __forceinline__ void latent_norm(F at, int n, int np, float eps, const float* gain, T* o1, T* o2, float* red, int tid) {
    float ss = 0.f;
    f32x4 keep[2];                                             // rows of up to 2048 columns stay in registers
#pragma unroll
    for (int q = 0; q < 2; q++) {
        const int i = 4 * tid + 1024 * q;
        keep[q] = i < np ? at(i) : f32x4{0.f, 0.f, 0.f, 0.f};
        ss += sumsq4(keep[q]);
    }
    for (int i = 4 * tid + 2048; i < np; i += 1024) ss += sumsq4(at(i));
    const float rs = 1.0f / sqrtf(block_sum<256>(ss, red, tid) / (float)n + eps);
#pragma unroll
    for (int q = 0; q < 2; q++) {
        const int i = 4 * tid + 1024 * q;
        if (i >= np) break;
        const f32x4 v = keep[q] * rs * *(const f32x4*)(gain + i);
        st4(o1 + i, v);
        if (o2) st4(o2 + i, v);
    }
    for (int i = 4 * tid + 2048; i < np; i += 1024) {
        const f32x4 v = at(i) * rs * *(const f32x4*)(gain + i);
        st4(o1 + i, v);
        if (o2) st4(o2 + i, v);
    }
}

// part (decode): the down projection arrives as fp32 K-slices [slices][M][Na] instead of rows `a`; the gate's columns are then rounded into `a` for the kernel that applies them.
// blockIdx.y: 0 = queries, 1 = cached latent, 2 = gate and padding (one workgroup each when rows are few, all three in turn otherwise)
template <typename T>
__global__ __launch_bounds__(256) void lm_latents_kernel(T* __restrict__ a, const float* __restrict__ part, int slices, int M, int Na, int q_rank, int Qp, int off_c, int kv_rank, int Rp,
                                                         int off_g, float eps, const float* __restrict__ nq, const float* __restrict__ nc, T* __restrict__ cq, T* __restrict__ c_dense,
                                                         T* __restrict__ cache, int max_tokens, const LmRowIndex ix, T* __restrict__ ao, int n_ao, int Gp) {
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const int64_t row = blockIdx.x;
    T* ar = a + row * Na;
    auto at = [&](int i) -> f32x4 {
        if (!part) return ld4(ar + i);
        f32x4 v[4], s = {0.f, 0.f, 0.f, 0.f};
        for (int k = 0; k < slices; k += 4) {
#pragma unroll
            for (int q = 0; q < 4; q++) v[q] = k + q < slices ? *(const f32x4*)(part + ((int64_t)(k + q) * M + row) * Na + i) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int q = 0; q < 4; q++) s += v[q];
        }
        return s;
    };
    const bool all = gridDim.y == 1;
    if (all || blockIdx.y == 0) latent_norm<T>(at, q_rank, Qp, eps, nq, cq + row * Qp, (T*)nullptr, red, tid);
    if (all || blockIdx.y == 1) {
        T* dst = cache + ((int64_t)row_seq(ix, row) * max_tokens + row_pos(ix, row)) * Rp;
        latent_norm<T>([&](int i) { return at(off_c + i); }, kv_rank, Rp, eps, nc, dst, c_dense ? c_dense + row * Rp : (T*)nullptr, red, tid);
    }
    if (all || blockIdx.y == 2) {
        if (part)
            for (int i = 4 * tid; i < Gp; i += 1024) st4(ar + off_g + i, at(off_g + i));
        for (int i = n_ao + tid; i < Gp; i += 256) ao[row * Gp + i] = (T)0.f;       // the padding columns the output projection's K runs over
    }
}

}  // namespace

// workgroup width and vectors per thread by row length and row count
#define LM_ROW_LAUNCH(KERNEL, T, TPB, NV, n, ...) hipLaunchKernelGGL((KERNEL<T, TPB, NV>), dim3((unsigned)(n)), dim3(TPB), 0, st, __VA_ARGS__)
#define LM_NV_DISPATCH(KERNEL, T, n, ...)                                                                             \
    do {                                                                                                              \
        const bool few_ = (n) <= 512;                                                                                 \
        if (lm.Wp <= 1024) LM_ROW_LAUNCH(KERNEL, T, 256, 1, n, __VA_ARGS__);                                          \
        else if (lm.Wp <= 2048) { if (few_) LM_ROW_LAUNCH(KERNEL, T, 512, 1, n, __VA_ARGS__); else LM_ROW_LAUNCH(KERNEL, T, 256, 2, n, __VA_ARGS__); }   \
        else if (lm.Wp <= 4096) { if (few_) LM_ROW_LAUNCH(KERNEL, T, 1024, 1, n, __VA_ARGS__); else LM_ROW_LAUNCH(KERNEL, T, 256, 4, n, __VA_ARGS__); }  \
        else if (lm.Wp <= 8192) LM_ROW_LAUNCH(KERNEL, T, 1024, 2, n, __VA_ARGS__);                                    \
        else if (lm.Wp <= 16384) LM_ROW_LAUNCH(KERNEL, T, 1024, 4, n, __VA_ARGS__);                                   \
        else return cr_fail(CR_ERR_ARG, "described decoder: width %d", lm.d.width);                                    \
        CR_HIP(hipGetLastError());                                                                                    \
        return CR_OK;                                                                                                 \
    } while (0)

int launch_lm_embed(bool f32, const Lm& lm, int M, const int64_t* tokens, const LmRowIndex& ix, const int64_t* gen, const int32_t* ngen, int gen_cap, float* x, const LmSink& to, int32_t* tok,
                    void* x0, int64_t ldx0, hipStream_t st) {
    if (f32) LM_NV_DISPATCH(lm_embed_kernel, float, M, (const float*)lm.embed, lm.freq, lm.Wp, lm.d.width, lm.d.vocab, lm.d.eps, tokens, ix, gen, ngen, gen_cap, x, to, tok, (float*)x0, ldx0);
    LM_NV_DISPATCH(lm_embed_kernel, bf16, M, (const bf16*)lm.embed, lm.freq, lm.Wp, lm.d.width, lm.d.vocab, lm.d.eps, tokens, ix, gen, ngen, gen_cap, x, to, tok, (bf16*)x0, ldx0);
}

int launch_lm_post(bool f32, const Lm& lm, int M, const LmPostIn& in, float* x, const float* gain_b, bool replace, const LmSink& to, hipStream_t st) {
    if (f32) LM_NV_DISPATCH(lm_post_kernel, float, M, in, M, lm.Wp, lm.d.width, lm.d.eps, x, gain_b, (int)replace, to);
    LM_NV_DISPATCH(lm_post_kernel, bf16, M, in, M, lm.Wp, lm.d.width, lm.d.eps, x, gain_b, (int)replace, to);
}

int launch_lm_pick_rows(bool f32, const Lm& lm, int n, const float* x, const int32_t* rows, void* h, const float* gain, hipStream_t st) {
    if (f32) LM_NV_DISPATCH(lm_pick_rows_kernel, float, n, x, rows, lm.Wp, lm.d.width, lm.d.eps, (float*)h, gain);
    LM_NV_DISPATCH(lm_pick_rows_kernel, bf16, n, x, rows, lm.Wp, lm.d.width, lm.d.eps, (bf16*)h, gain);
}

int launch_lm_latents(bool f32, const Lm& lm, const LmLayer& L, int M, void* a, const float* part, int slices, void* cq, void* c_dense, void* cache, int max_tokens, const LmRowIndex& ix,
                      void* ao, hipStream_t st) {
    const int n_ao = L.s.heads * L.s.vdim;
    const dim3 grid((unsigned)M, M <= 512 ? 3 : 1);
    if (f32)
        hipLaunchKernelGGL(lm_latents_kernel<float>, grid, dim3(256), 0, st, (float*)a, part, slices, M, L.Na, L.s.q_rank, L.Qp, L.off_c, L.s.kv_rank, L.Rp, L.off_g, lm.d.eps, L.nq, L.nc,
                           (float*)cq, (float*)c_dense, (float*)cache, max_tokens, ix, (float*)ao, n_ao, L.Gp);
    else
        hipLaunchKernelGGL(lm_latents_kernel<bf16>, grid, dim3(256), 0, st, (bf16*)a, part, slices, M, L.Na, L.s.q_rank, L.Qp, L.off_c, L.s.kv_rank, L.Rp, L.off_g, lm.d.eps, L.nq, L.nc,
                           (bf16*)cq, (bf16*)c_dense, (bf16*)cache, max_tokens, ix, (bf16*)ao, n_ao, L.Gp);
    CR_HIP(hipGetLastError());
    return CR_OK;
}

namespace {
// z[m][n] = gelu_tanh(sum of K-slices) * side[tok[m]][n], one thread per four columns
__global__ __launch_bounds__(256) void lm_side_act_kernel(const float* __restrict__ part, int slices, int M, int Sp, const bf16* __restrict__ side, int64_t lds, const int32_t* __restrict__ tok,
                                                          bf16* __restrict__ z) {
    const int i = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= M * Sp) return;
    const int m = i / Sp, n = i - m * Sp;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < slices; k += 8) {
        f32x4 v[8];
#pragma unroll
        for (int q = 0; q < 8; q++) v[q] = k + q < slices ? *(const f32x4*)(part + ((int64_t)(k + q) * M + m) * Sp + n) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int q = 0; q < 8; q++) s += v[q];
    }
    const f32x4 e = ld4(side + (int64_t)tok[m] * lds + n);
    st4(z + i, f32x4{gelu_tanh(s[0]) * e[0], gelu_tanh(s[1]) * e[1], gelu_tanh(s[2]) * e[2], gelu_tanh(s[3]) * e[3]});
}

// the same z for up to 16 rows, kept in LDS, and y = z . W^T behind it: a workgroup forms z for itself (a few KiB from L2) and multiplies 64 rows of W, 16 per wave
__global__ __launch_bounds__(256) void lm_side_proj_kernel(const float* __restrict__ part, int slices, int M, int Sp, const bf16* __restrict__ side, int64_t lds, const int32_t* __restrict__ tok,
                                                           const bf16* __restrict__ W, int N, bf16* __restrict__ y) {
    extern __shared__ __attribute__((aligned(16))) bf16 sz[];              // [16][Sp + 8]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ld = Sp + 8, n0 = blockIdx.x * 64 + wave * 16;
    const bf16* w = W + (int64_t)min(n0 + (lane & 15), N - 1) * Sp + (lane >> 4) * 8;
    bf16x8 wf[8];
#pragma unroll
    for (int k = 0; k < 8; k++) wf[k] = *(const bf16x8*)(w + min(k * 32, Sp - 32));      // the first 256 columns travel under z
    for (int i = tid * 4; i < 16 * Sp; i += 1024) {
        const int m = i / Sp, n = i - m * Sp;
        f32x4 z = {0.f, 0.f, 0.f, 0.f};
        if (m < M) {
            f32x4 s = {0.f, 0.f, 0.f, 0.f};
            for (int k = 0; k < slices; k += 8) {
                f32x4 v[8];
#pragma unroll
                for (int q = 0; q < 8; q++) v[q] = k + q < slices ? *(const f32x4*)(part + ((int64_t)(k + q) * M + m) * Sp + n) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int q = 0; q < 8; q++) s += v[q];
            }
            const f32x4 e = ld4(side + (int64_t)tok[m] * lds + n);
#pragma unroll
            for (int q = 0; q < 4; q++) z[q] = gelu_tanh(s[q]) * e[q];
        }
        st4(sz + m * ld + n, z);
    }
    __syncthreads();
    const bf16* zr = sz + (lane & 15) * ld + (lane >> 4) * 8;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < Sp; k0 += 256) {
#pragma unroll
        for (int k = 0; k < 8; k++)
            if (k0 + k * 32 < Sp) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[k], *(const bf16x8*)(zr + k0 + k * 32), acc, 0, 0, 0);
        if (k0 + 256 < Sp) {
#pragma unroll
            for (int k = 0; k < 8; k++) wf[k] = *(const bf16x8*)(w + min(k0 + 256 + k * 32, Sp - 32));
        }
    }
    // lane: columns n0 + 4 (lane >> 4) + 0..3 of row lane & 15
    const int m = lane & 15, n = n0 + 4 * (lane >> 4);
    if (m < M && n + 4 <= N) *(bf16x4*)(y + (int64_t)m * N + n) = bf16x4{f2bf(acc[0]), f2bf(acc[1]), f2bf(acc[2]), f2bf(acc[3])};
}
}  // namespace

int launch_lm_side_act(const Lm& lm, int M, const float* part, int slices, const void* side, int64_t lds, const int32_t* tok, void* z, hipStream_t st) {
    hipLaunchKernelGGL(lm_side_act_kernel, dim3((M * lm.Sp / 4 + 255) / 256), dim3(256), 0, st, part, slices, M, lm.Sp, (const bf16*)side, lds, tok, (bf16*)z);
    CR_HIP(hipGetLastError());
    return CR_OK;
}

bool lm_side_proj_supported(const Lm& lm, int M) { return !lm.f32 && M <= 16 && lm.Sp <= 1024; }
int launch_lm_side_proj(const Lm& lm, int M, const float* part, int slices, const void* side, int64_t lds, const int32_t* tok, const void* W, void* y, hipStream_t st) {
    if (!lm_side_proj_supported(lm, M) || M <= 0 || slices <= 0) return cr_fail(CR_ERR_ARG, "token side: %d rows of %d columns", M, lm.Sp);
    hipLaunchKernelGGL(lm_side_proj_kernel, dim3((lm.Wp + 63) / 64), dim3(256), 16 * (lm.Sp + 8) * 2, st, part, slices, M, lm.Sp, (const bf16*)side, lds, tok, (const bf16*)W, lm.Wp, (bf16*)y);
    CR_HIP(hipGetLastError());
    return CR_OK;
}
