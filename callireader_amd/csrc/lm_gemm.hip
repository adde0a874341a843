// Matrix products of described decoders that the dense bf16 kernels do not take: everything in true fp32 (v_mfma_f32_16x16x4_f32), products batched over heads, and products
// grouped over experts with gathered rows and scattered results.  C = epi(A[M,K] . W[N,K]^T), K % 64 == 0.
//
// 64 x 64 tile, 4 waves of 32 x 32 (2 x 2 accumulators of 16 x 16), K in steps of 32 through LDS.  The weights are the MFMA's A operand, so a lane's accumulator holds four
// consecutive output columns of one row (the same roles as gemm256 / gemm_skinny).  A row's sum runs over K in ascending steps whatever tile it sits in.
#include "lm.hpp"

namespace {

constexpr int BM = LM_TILE_M, BN = 64, BK = 32;

template <typename T> struct Frag;
template <> struct Frag<bf16> {
    static constexpr int LD = BK + 8;              // elements per LDS row: 80 bytes, 16-byte aligned, rows spread over the banks
    static constexpr int VEC = 8;
    typedef bf16x8 vec;
    static __device__ __forceinline__ f32x4 mma(const bf16* w, const bf16* a, int lane, f32x4 acc) {
        const bf16x8 wf = *(const bf16x8*)(w + 8 * (lane >> 4)), af = *(const bf16x8*)(a + 8 * (lane >> 4));
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, af, acc, 0, 0, 0);
    }
};
template <> struct Frag<float> {
    static constexpr int LD = BK + 4;
    static constexpr int VEC = 4;
    typedef f32x4 vec;
    static __device__ __forceinline__ f32x4 mma(const float* w, const float* a, int lane, f32x4 acc) {
#pragma unroll
        for (int k = 0; k < BK / 4; k++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(w[4 * k + (lane >> 4)], a[4 * k + (lane >> 4)], acc, 0, 0, 0);
        return acc;
    }
};

template <typename T, int EPI>
__global__ __launch_bounds__(256) void lm_gemm_kernel(const LmGemmParams p) {
    typedef Frag<T> F;
    __shared__ __attribute__((aligned(16))) T sA[BM][F::LD];
    __shared__ __attribute__((aligned(16))) T sW[BN][F::LD];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int n0 = blockIdx.x * BN;
    const T* A = (const T*)p.A + (int64_t)blockIdx.z * p.a_bs;
    const T* W = (const T*)p.W;
    int m0 = blockIdx.y * BM, rows = p.M - m0, pos0 = m0;
    if (p.tiles) {                                            // grouped: this tile's expert and its slice of the sorted assignments
        if ((int)blockIdx.y >= *p.n_tiles) return;            // (uniform: the grid is sized for the worst split)
        const int4 t = p.tiles[blockIdx.y];
        W += (int64_t)t.x * p.w_bs;
        pos0 = t.y; rows = t.z;
    } else W += (int64_t)blockIdx.z * p.w_bs;
    if (rows > BM) rows = BM;

    constexpr int CPR = BK / F::VEC;                          // vectors per tile row
    constexpr int NL = BM * CPR / 256;                        // vectors per thread and operand
    const T* ga[NL];
    const T* gw[NL];
#pragma unroll
    for (int i = 0; i < NL; i++) {
        const int v = tid + i * 256, r = v / CPR, c = (v % CPR) * F::VEC;
        const int m = pos0 + min(r, rows - 1);
        const int64_t ar = (p.perm && p.gather_div) ? p.perm[m] / p.gather_div : m;
        ga[i] = A + ar * p.lda + c;
        gw[i] = W + (int64_t)min(n0 + r, p.N - 1) * p.ldw + c;
    }
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int wn = (wave & 1) * 32, wm = (wave >> 1) * 32;
    typename F::vec ra[NL], rw[NL];
#pragma unroll
    for (int i = 0; i < NL; i++) { ra[i] = *(const typename F::vec*)ga[i]; rw[i] = *(const typename F::vec*)gw[i]; }
    for (int k0 = 0; k0 < p.K; k0 += BK) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NL; i++) {
            const int v = tid + i * 256, r = v / CPR, c = (v % CPR) * F::VEC;
            *(typename F::vec*)&sA[r][c] = ra[i];
            *(typename F::vec*)&sW[r][c] = rw[i];
        }
        __syncthreads();
        if (k0 + BK < p.K) {
#pragma unroll
            for (int i = 0; i < NL; i++) { ra[i] = *(const typename F::vec*)(ga[i] + k0 + BK); rw[i] = *(const typename F::vec*)(gw[i] + k0 + BK); }
        }
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int j = 0; j < 2; j++) acc[i][j] = F::mma(&sW[wn + 16 * i + (lane & 15)][0], &sA[wm + 16 * j + (lane & 15)][0], lane, acc[i][j]);
    }

    // lane: columns n0 + wn + 16 i + 4 (lane >> 4) + e of row wm + 16 j + (lane & 15)
#pragma unroll
    for (int j = 0; j < 2; j++) {
        const int r = wm + 16 * j + (lane & 15);
        const bool live = r < rows;
        const int m = pos0 + (live ? r : rows - 1);
        const int64_t cr = (p.perm && p.scatter) ? p.perm[m] : m;
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int n = n0 + wn + 16 * i + 4 * (lane >> 4);
            f32x4 v = acc[i][j];
            if (EPI == LM_GLU) {
                // rows 0..7 of a 16-row weight tile are gates, 8..15 the matching ups: the partner's accumulator is 32 lanes away
                f32x4 u;
#pragma unroll
                for (int e = 0; e < 4; e++) u[e] = __shfl_xor(v[e], 32, 64);
                if (!live || (lane >> 4) >= 2 || n >= p.N) continue;
                T* c = (T*)p.C + cr * p.ldc + (n0 + wn + 16 * i) / 2 + 4 * (lane >> 4);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const float g = fminf(v[e], p.limit), up = fminf(fmaxf(u[e], -p.limit), p.limit);
                    c[e] = (T)(g / (1.0f + expf(-1.702f * g)) * (up + 1.0f));
                }
                continue;
            }
            if (!live) continue;
            if (EPI == LM_RAW32) {
                float* c = (float*)p.C + (int64_t)blockIdx.z * p.c_bs + cr * p.ldc + n;
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (n + e < p.N) c[e] = p.softcap > 0.f ? p.softcap * tanhf(v[e] / p.softcap) : v[e];
                continue;
            }
            T* c = (T*)p.C + (int64_t)blockIdx.z * p.c_bs + cr * p.ldc + n;
            if (EPI == LM_GATE) {
                const T* g = (const T*)p.gate + (int64_t)blockIdx.z * p.g_bs + cr * p.ldg + n;
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (n + e < p.N) c[e] = (T)(v[e] / (1.0f + expf(-(float)g[e])));
            } else if (EPI == LM_SIDE) {
                const T* g = (const T*)p.gate + (int64_t)p.tok[cr] * p.ldg + n;
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (n + e < p.N) c[e] = (T)(gelu_tanh(v[e]) * (float)g[e]);
            } else if (EPI == LM_RELU2) {
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (n + e < p.N) c[e] = (T)relu2(v[e]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (n + e < p.N) c[e] = (T)v[e];
            }
        }
    }
}

template <typename T>
int launch_t(int epi, const LmGemmParams& p, hipStream_t st) {
    const dim3 grid((p.N + BN - 1) / BN, p.tiles ? p.max_tiles : (p.M + BM - 1) / BM, p.batch > 0 ? p.batch : 1), block(256);
    switch (epi) {
        case LM_STORE: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_STORE>), grid, block, 0, st, p); break;
        case LM_RAW32: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_RAW32>), grid, block, 0, st, p); break;
        case LM_GLU: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_GLU>), grid, block, 0, st, p); break;
        case LM_GATE: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_GATE>), grid, block, 0, st, p); break;
        case LM_RELU2: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_RELU2>), grid, block, 0, st, p); break;
        case LM_SIDE: hipLaunchKernelGGL((lm_gemm_kernel<T, LM_SIDE>), grid, block, 0, st, p); break;
        default: return cr_fail(CR_ERR_ARG, "lm_gemm: epilogue %d", epi);
    }
    CR_HIP(hipGetLastError());
    return CR_OK;
}

}  // namespace

int launch_lm_gemm(bool f32, int epi, const LmGemmParams& p, hipStream_t st) {
    const int vec = f32 ? 4 : 8;
    if (p.N <= 0 || p.K <= 0 || p.K % 64 || p.lda % vec || p.ldw % vec || p.a_bs % vec || p.w_bs % vec || (p.tiles ? p.max_tiles <= 0 || p.batch > 1 || !p.n_tiles : p.M <= 0) ||
        (p.gather_div && !p.perm) || (epi == LM_GLU && (p.N % 16 || p.batch > 1)) || ((epi == LM_GATE || epi == LM_SIDE) && !p.gate) || (epi == LM_SIDE && !p.tok) || (((uintptr_t)p.A | (uintptr_t)p.W) & 15))
        return cr_fail(CR_ERR_ARG, "lm_gemm(epi=%d M=%d N=%d K=%d): bad argument", epi, p.M, p.N, p.K);
    return f32 ? launch_t<float>(epi, p, st) : launch_t<bf16>(epi, p, st);
}
