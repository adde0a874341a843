// Retention: S <- decay S + k v^T, o = S^T q per head, with S in fp32; a head's o over its root mean square, gated by silu(g).
//
// Decode: one workgroup per (row, head) streams the state through registers once (a state is 4 Kp Vp bytes, read and written: the step's whole cost), in a layout of its own
// (lm.hpp: 1 KiB per load instruction) that keeps the contraction over dk inside a wave.
//
// Prompts in bf16, matrix form: the sequence is cut into chunks of RET_CHUNK rows.  Within a chunk o_i = sum_j decay^(i-j) (q_i . k_j) v_j, what came before enters as
// decay^(i+1) S^T q_i with S the state ahead of the chunk.  Three launches: ret_chunk_kernel forms what each chunk adds to the state, all chunks at once; ret_scan_kernel carries the
// state through them (in place: a chunk's addition becomes the state ahead of it); ret_out_kernel computes the outputs, again all chunks at once.  Operands that are not bf16 by nature (rotated q and k, decayed k, states, decayed scores) enter the matrix
// cores as two bf16 terms, value and remainder, products of two remainders left out: 2^-16 relative, against fp32's place in the recurrence.
// Powers of the decay come from a table in fp32 made from double (decay^0 .. decay^RET_CHUNK): no logarithm, so decays of 0 and 1 are ordinary.
//
// Prompts in fp32, and sizes past the matrix form: the recurrence token by token, state in registers, then a norm-and-gate kernel.
#include <algorithm>

#include "attention_merge.hpp"
#include "lm.hpp"

namespace {

// element of a (sequence, head) state
__device__ __forceinline__ int64_t ret_state_at(int dk, int col, int NR) {
    return ((int64_t)(col >> 4) * NR + dk % NR) * 256 + ((dk / NR) * 4 + ((col & 15) >> 2)) * 4 + (col & 3);
}
template <typename T> __device__ __forceinline__ f32x4 ld4f(const T* p);
template <> __device__ __forceinline__ f32x4 ld4f<float>(const float* p) { return *(const f32x4*)p; }
template <> __device__ __forceinline__ f32x4 ld4f<bf16>(const bf16* p) {
    const bf16x4 v = *(const bf16x4*)p;
    return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
// the sixteen dk groups of a wave sit four lanes apart
__device__ __forceinline__ f32x4 sum_groups(f32x4 o) {
#pragma unroll
    for (int s = 4; s < 64; s <<= 1)
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] += __shfl_xor(o[e], s, 64);
    return o;
}
__device__ __forceinline__ float silu32(float x) { return x / (1.0f + expf(-x)); }

constexpr int dec_waves(int NR) { return NR > 16 ? 8 : 16; }

// workgroups past the heads merge the attention's key splits of the same row (the mixer beside this one), a wave per 64 columns: two short launches in one
template <typename T, int NR>
__global__ __launch_bounds__(dec_waves(NR) * 64) void ret_decode_kernel(const RetParams p, const AttnParams merge, int merge_dim) {
    __shared__ float so[LM_MAX_HEAD], red[LM_MAX_HEAD / 16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
    const int h = blockIdx.x, row = blockIdx.y;
    if (h >= p.H) {
        const int u = (h - p.H) * nw + wave, parts = merge_dim / 64, hq = u / parts;
        if (hq < merge.H * merge.Sq) attn_merge_splits(merge, merge_dim, row, hq / merge.Sq, hq % merge.Sq, (u % parts) * 64 + lane);
        return;
    }
    const int seq = p.ix.seqs[row];
    const bool fresh = p.ix.lens[seq] == 0;                   // a state starts at zero, whatever the slot held before
    const int g = lane >> 2, c4 = (lane & 3) * 4, blocks = p.Vp >> 4;
    float* st = p.state + ((int64_t)seq * p.H + h) * p.Vp * p.Kp;
    const float decay = p.pw[h * (RET_CHUNK + 1) + 1];
    const float* qr = p.rq + ((int64_t)row * p.H + h) * p.Kp + g * NR;
    const float* kr = p.rk + ((int64_t)row * p.H + h) * p.Kp + g * NR;
    for (int b = wave; b < blocks; b += nw) {
        f32x4 s[NR];
        float* sb = st + (int64_t)b * NR * 256 + lane * 4;
#pragma unroll
        for (int r = 0; r < NR; r++) s[r] = fresh ? f32x4{0.f, 0.f, 0.f, 0.f} : __builtin_nontemporal_load((const f32x4*)(sb + r * 256));
        float q[NR], k[NR];
#pragma unroll
        for (int r = 0; r < NR; r += 4) {
            const f32x4 a = *(const f32x4*)(qr + r), c = *(const f32x4*)(kr + r);
#pragma unroll
            for (int e = 0; e < 4; e++) { q[r + e] = a[e]; k[r + e] = c[e]; }
        }
        const f32x4 v = ld4f((const T*)p.v + (int64_t)row * p.lda + h * p.Vp + b * 16 + c4);
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < NR; r++) {
            s[r] = s[r] * decay + k[r] * v;
            o += s[r] * q[r];
            __builtin_nontemporal_store(s[r], (f32x4*)(sb + r * 256));
        }
        o = sum_groups(o);
        if (lane < 4) *(f32x4*)&so[b * 16 + c4] = o;
        float ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
        ss += __shfl_xor(ss, 1, 64);
        ss += __shfl_xor(ss, 2, 64);
        if (lane == 0) red[b] = ss;
    }
    __syncthreads();
    float ss = 0.f;
    for (int b = 0; b < blocks; b++) ss += red[b];
    const float rs = p.out_scale / sqrtf(ss / (float)p.vdim + p.eps);
    for (int c = tid; c < p.vdim; c += blockDim.x)
        ((T*)p.ao)[(int64_t)row * p.ldo + (int64_t)h * p.vdim + c] = (T)(so[c] * rs * silu32((float)((const T*)p.g)[(int64_t)row * p.lda + h * p.Vp + c]));
}

// one wave = 16 value columns, the tokens of a segment in turn
template <typename T, int NR>
__global__ __launch_bounds__(256) void ret_recurrent_kernel(const RetParams p) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int b = blockIdx.x * 4 + wave, h = blockIdx.y;
    const int32_t* sg = p.seg + 4 * blockIdx.z;
    const int row0 = sg[0], S = sg[1], seq = sg[3];
    const int g = lane >> 2, c4 = (lane & 3) * 4;
    float* sb = p.state + ((int64_t)seq * p.H + h) * p.Vp * p.Kp + (int64_t)b * NR * 256 + lane * 4;
    const float decay = p.pw[h * (RET_CHUNK + 1) + 1];
    f32x4 s[NR];
#pragma unroll
    for (int r = 0; r < NR; r++) s[r] = sg[2] == 0 ? f32x4{0.f, 0.f, 0.f, 0.f} : *(const f32x4*)(sb + r * 256);
    f32x4 q[NR / 4], k[NR / 4], v;
    auto load = [&](int t) {
        const int64_t o = ((int64_t)(row0 + t) * p.H + h) * p.Kp + g * NR;
#pragma unroll
        for (int r = 0; r < NR / 4; r++) { q[r] = *(const f32x4*)(p.rq + o + 4 * r); k[r] = *(const f32x4*)(p.rk + o + 4 * r); }
        v = ld4f((const T*)p.v + (int64_t)(row0 + t) * p.lda + h * p.Vp + b * 16 + c4);
    };
    load(0);
    for (int t = 0; t < S; t++) {
        f32x4 qc[NR / 4], kc[NR / 4];
        const f32x4 vc = v;
#pragma unroll
        for (int r = 0; r < NR / 4; r++) { qc[r] = q[r]; kc[r] = k[r]; }
        load(min(t + 1, S - 1));
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < NR; r++) {
            s[r] = s[r] * decay + kc[r / 4][r % 4] * vc;
            o += s[r] * qc[r / 4][r % 4];
        }
        o = sum_groups(o);
        if (lane < 4) *(f32x4*)(p.raw + ((int64_t)(row0 + t) * p.H + h) * p.Vp + b * 16 + c4) = o;
    }
#pragma unroll
    for (int r = 0; r < NR; r++) *(f32x4*)(sb + r * 256) = s[r];
}

// one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void ret_gate_kernel(const RetParams p) {
    const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int64_t row = blockIdx.x;
    if (h >= p.H) return;
    const float* o = p.raw + (row * p.H + h) * p.Vp;
    float ss = 0.f;
    for (int c = lane; c < p.Vp; c += 64) ss += o[c] * o[c];
    const float rs = p.out_scale / sqrtf(wave_sum(ss) / (float)p.vdim + p.eps);
    for (int c = lane; c < p.vdim; c += 64)
        ((T*)p.ao)[row * p.ldo + (int64_t)h * p.vdim + c] = (T)(o[c] * rs * silu32((float)((const T*)p.g)[row * p.lda + h * p.Vp + c]));
}

// ---- matrix form ----
template <int D> __device__ __forceinline__ int kswz(int r) { return D == 64 ? ((r >> 1) & 7) : (r & 15); }          // (attention.hip: 16-byte chunks of a K row, read as rows)
template <int D> __device__ __forceinline__ int vswz(int r) { return D == 64 ? (((r >> 1) & 1) << 2) : ((r & 3) << 2); }   // (... of a V row, read transposed)
typedef __attribute__((ext_vector_type(4))) unsigned u32x4;
__device__ __forceinline__ unsigned pack2(float a, float b) {
    typedef __attribute__((ext_vector_type(2))) float f2;
    return __builtin_bit_cast(unsigned, __builtin_convertvector(f2{a, b}, bf16x2));
}
__device__ __forceinline__ float lo16(unsigned pk) { return __uint_as_float(pk << 16); }
__device__ __forceinline__ float hi16(unsigned pk) { return __uint_as_float(pk & 0xffff0000u); }
// sixteen rows x 32 columns of a row-major LDS tile as an MFMA operand with the ROW as the contraction index (the row order inside the operand is the same for every tile)
__device__ __forceinline__ bf16x8 read_tr(const char* at, int row_bytes) {
    const bf16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4*)CR_LDS(at));
    const bf16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4*)CR_LDS(at + 8 * row_bytes));
    return bf16x8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
}

// A chunk's addition and the state ahead of it share the bytes of RetParams::snap: per (chunk, head) blocks of 32 value columns x 16 dk, 2 KiB each; lane = value column % 32 (+ 32 for
// the second eight dk).  Addition: fp32, [dk % 8 / 4][lane][dk % 4].  State: two bf16 terms, [term][lane][dk % 8] -- ret_out_kernel's A operand, 1 KiB per load instruction.

// U[64 dk][64 dv] of one (chunk, head): sum over the chunk's n rows of decay^(n-1-j) k_j v_j^T.  Two tiles of 64 rows are under way while one is multiplied.
__global__ __launch_bounds__(256) void ret_chunk_kernel(const RetParams p) {
    __shared__ __attribute__((aligned(16))) char sm[2][3][8192];          // [buffer][v, k, k's remainder][64 rows][64 columns]
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int kt = blockIdx.x % (p.Kp / 64), vt = blockIdx.x / (p.Kp / 64), h = blockIdx.y;
    const int row0 = p.chunks[2 * blockIdx.z], S = p.chunks[2 * blockIdx.z + 1];
    const float* pw = p.pw + h * (RET_CHUNK + 1);
    const int64_t plane = (int64_t)p.M * p.H * p.Kp;
    const int l31 = lane & 31, hh = lane >> 5, wv = wave & 1, wk = wave >> 1;
    const int dv = vt * 64 + wv * 32 + l31, dk0 = kt * 64 + wk * 32 + 4 * hh;      // lane: value column dv, element e: dk0 + (e & 3) + 8 (e >> 2)
    f32x16 acc[2];
#pragma unroll
    for (int e = 0; e < 16; e++) acc[0][e] = acc[1][e] = 0.f;

    // staging: a thread carries 16 columns of one row
    const int r = tid >> 2, c0 = (tid & 3) * 2;
    const bf16* vp = (const bf16*)p.v + (int64_t)row0 * p.lda + h * p.Vp + vt * 64 + c0 * 8;
    const bf16* kp = p.rk2 + ((int64_t)row0 * p.H + h) * p.Kp + kt * 64 + c0 * 8;
    struct Tile { bf16x8 v[2], a[2], b[2]; float w; };
    const int nt = (S + 63) / 64;
    auto load = [&](int t, Tile& x) {
        const int q = t * 64 + r, qc = min(q, S - 1);
        x.w = q < S ? pw[S - 1 - qc] : 0.f;
#pragma unroll
        for (int i = 0; i < 2; i++) {
            x.v[i] = *(const bf16x8*)(vp + (int64_t)qc * p.lda + i * 8);
            x.a[i] = *(const bf16x8*)(kp + (int64_t)qc * p.H * p.Kp + i * 8);
            x.b[i] = *(const bf16x8*)(kp + plane + (int64_t)qc * p.H * p.Kp + i * 8);
        }
    };
    auto store = [&](const Tile& x, int buf) {
#pragma unroll
        for (int i = 0; i < 2; i++) {
            u32x4 hi, lo;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const float x0 = ((float)x.a[i][2 * e] + (float)x.b[i][2 * e]) * x.w, x1 = ((float)x.a[i][2 * e + 1] + (float)x.b[i][2 * e + 1]) * x.w;
                hi[e] = pack2(x0, x1);
                lo[e] = pack2(x0 - lo16(hi[e]), x1 - hi16(hi[e]));
            }
            const int at = r * 128 + (((c0 + i) ^ vswz<64>(r)) << 4);
            *(bf16x8*)(sm[buf][0] + at) = x.v[i];
            *(u32x4*)(sm[buf][1] + at) = hi;
            *(u32x4*)(sm[buf][2] + at) = lo;
        }
    };
    const int gq = lane >> 4, li = lane & 15, tq = li >> 2, tp = li & 3;
    const int lrow = 4 * hh + tq, clow = (gq & 1) * 2 + (tp >> 1), sw = vswz<64>(lrow), loff = lrow * 128 + (tp & 1) * 8;
    // tile t from LDS buffer `cur`; tile t + 1 goes from `x` to the other buffer, then tile t + 3 is requested into `x`
    auto step = [&](int t, int cur, Tile& x) {
#pragma unroll
        for (int s = 0; s < 4; s++) {
            const bf16x8 vf = read_tr(sm[cur][0] + 16 * s * 128 + loff + ((((wv * 4) ^ sw) | clow) << 4), 128);
            const bf16x8 kf = read_tr(sm[cur][1] + 16 * s * 128 + loff + ((((wk * 4) ^ sw) | clow) << 4), 128);
            const bf16x8 kl = read_tr(sm[cur][2] + 16 * s * 128 + loff + ((((wk * 4) ^ sw) | clow) << 4), 128);
            acc[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, vf, acc[0], 0, 0, 0);
            acc[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kl, vf, acc[1], 0, 0, 0);
        }
        if (t + 1 < nt) store(x, cur ^ 1);
        if (t + 3 < nt) load(t + 3, x);
        __syncthreads();
    };
    Tile a, b;
    load(0, a);
    load(min(1, nt - 1), b);
    store(a, 0);
    load(min(2, nt - 1), a);
    __syncthreads();
    for (int t = 0; t < nt; t += 2) {
        step(t, 0, b);
        if (t + 1 < nt) step(t + 1, 1, a);
    }
    float* u = (float*)p.snap + ((int64_t)blockIdx.z * p.H + h) * p.Vp * p.Kp;
#pragma unroll
    for (int g = 0; g < 4; g++) {
        const int dk = dk0 + 8 * g;
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = acc[0][4 * g + e] + acc[1][4 * g + e];
        *(f32x4*)(u + ((int64_t)(dv >> 5) * (p.Kp >> 4) + (dk >> 4)) * 512 + hh * 256 + ((dv & 31) + ((dk & 8) << 2)) * 4) = o;
    }
}

// the state of one (segment, head) through its chunks, eight dk of one value column per thread; what a thread reads of a chunk it overwrites with the state ahead of it
__global__ __launch_bounds__(256) void ret_scan_kernel(const RetParams p) {
    const int t = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, lane = t & 63, blk = t >> 6, NR = p.Kp >> 4;
    if (t * 8 >= p.Vp * p.Kp) return;
    const int32_t* sg = p.seg + 4 * blockIdx.z;
    const int n = (sg[1] + RET_CHUNK - 1) / RET_CHUNK, dv = blk / NR * 32 + (lane & 31), dk = blk % NR * 16 + (lane >> 5) * 8;
    const float* pw = p.pw + h * (RET_CHUNK + 1);
    float* st = p.state + ((int64_t)sg[3] * p.H + h) * p.Vp * p.Kp;
    float* u = (float*)p.snap + ((int64_t)p.snap0[blockIdx.z] * p.H + h) * p.Vp * p.Kp + (int64_t)blk * 512 + lane * 4;
    const int64_t step = (int64_t)p.H * p.Vp * p.Kp;
    float s[8];
#pragma unroll
    for (int e = 0; e < 8; e++) s[e] = sg[2] == 0 ? 0.f : st[ret_state_at(dk + e, dv, NR)];
    f32x4 a = *(const f32x4*)u, b = *(const f32x4*)(u + 256);
    for (int c = 0; c < n; c++) {
        const f32x4 na = *(const f32x4*)(u + min(c + 1, n - 1) * step), nb = *(const f32x4*)(u + min(c + 1, n - 1) * step + 256);
        const float w = pw[min(RET_CHUNK, sg[1] - c * RET_CHUNK)];
        bf16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; e++) {
            hi[e] = f2bf(s[e]);
            lo[e] = f2bf(s[e] - rbf(s[e]));
            s[e] = s[e] * w + (e < 4 ? a[e] : b[e - 4]);
        }
        *(bf16x8*)(u + c * step) = hi;
        *(bf16x8*)(u + c * step + 256) = lo;
        a = na; b = nb;
    }
#pragma unroll
    for (int e = 0; e < 8; e++) st[ret_state_at(dk + e, dv, NR)] = s[e];
}

// LDS-DMA from inline asm (M0 = LDS base, saved and restored inside the statement): the compiler does not order a tile's LDS reads behind the fills of later tiles
__device__ __forceinline__ void dma16(const void* base, unsigned off, unsigned dst) {
    unsigned keep;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0" : "=&s"(keep) : "v"(off), "s"(base), "s"(dst) : "memory");
}
// all but the last N of this wave's loads have landed, for every wave of the workgroup
template <int N> __device__ __forceinline__ void tile_barrier() { asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(N) : "memory"); }

// 128 rows of one (segment, head): four waves of 32 (attention.hip's operand roles: queries on the lanes).  One stream of tiles through a ring of three LDS buffers, two under way:
// the state ahead of the chunk in tiles of 32 value columns (what they give is exactly their block of the output), then the chunk's keys and values in tiles of 32 rows.
template <int KP, int VP>
__global__ __launch_bounds__(256, (KP > 128 || VP > 128) ? 1 : 2) void ret_out_kernel(const RetParams p) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    constexpr int KB = 32 * KP * 2, VB = 32 * VP * 2, BUF = 2 * KB + VB;
    constexpr int KS = KP / 16, DB = VP / 32;
    constexpr int NK = KB / 4096, NV = VB / 4096, NTILE = 2 * NK + NV, NSTATE = 2 * NK;      // load instructions per wave: keys (one term), values, a tile, a state tile
    float* pwl = (float*)(smem + 3 * BUF);                    // 32 zeros, then decay^0 .. decay^RET_CHUNK: a key behind its query weighs nothing
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l31 = lane & 31, hh = lane >> 5;
    const int blk = blockIdx.x, h = blockIdx.y;
    const int32_t* sg = p.seg + 4 * blockIdx.z;
    const int row0 = sg[0], S = sg[1];
    if (blk * 128 >= S) return;
    const int chunk = blk / (RET_CHUNK / 128), c0 = chunk * RET_CHUNK;
    const int w0 = blk * 128 + wave * 32, qi = w0 + l31, qc = min(qi, S - 1);
    const int64_t plane = (int64_t)p.M * p.H * KP;
    const bool prior = chunk > 0 || sg[2] > 0;

    const bf16* kb = p.rk2 + ((int64_t)(row0 + c0) * p.H + h) * KP;
    const bf16* vb = (const bf16*)p.v + (int64_t)(row0 + c0) * p.lda + h * VP;
    const bf16* sn = p.snap + ((int64_t)(p.snap0[blockIdx.z] + chunk) * p.H + h) * 2 * VP * KP;
    const int last = S - 1 - c0;                              // last row of the segment, counted from the chunk
    const unsigned lds = (unsigned)(size_t)(__attribute__((address_space(3))) char*)smem;
    const int ns = prior ? DB : 0, nt = (min(blk * 128 + 128, S) - c0 + 31) / 32;
    // tile u of the stream: a state tile (u < ns), else keys and values; chunks of 16 bytes swizzled on the source side
    auto stage = [&](int buf, int u) {
        const unsigned base = lds + buf * BUF;
        if (u < ns) {
#pragma unroll
            for (int i = 0; i < NSTATE; i++) dma16(sn, (unsigned)(u * 2 * KB + (wave * NSTATE + i) * 1024 + lane * 16), base + (wave * NSTATE + i) * 1024);
            return;
        }
        constexpr int KR = 1024 / (KP * 2), VR = 1024 / (VP * 2);         // rows per load instruction
        const int key = (u - ns) * 32;
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int r = (wave * NK + i) * KR + lane / (KP / 8), cp = lane % (KP / 8);
            const unsigned off = (unsigned)min(key + r, last) * (unsigned)(p.H * KP * 2) + (unsigned)((cp ^ kswz<KP>(r)) * 16);
            dma16(kb, off, base + (wave * NK + i) * 1024);
            dma16(kb + plane, off, base + KB + (wave * NK + i) * 1024);
        }
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int r = (wave * NV + i) * VR + lane / (VP / 8), cp = lane % (VP / 8);
            dma16(vb, (unsigned)min(key + r, last) * (unsigned)(p.lda * 2) + (unsigned)((cp ^ vswz<VP>(r)) * 16), base + 2 * KB + (wave * NV + i) * 1024);
        }
    };
    const int total = ns + nt;
    // behind tile u: tile u + 1 has landed, tile u + 2 may be under way
    auto close = [&](int u) {
        if (u + 2 >= total) tile_barrier<0>();
        else if (u + 2 < ns) tile_barrier<NSTATE>();
        else tile_barrier<NTILE>();
    };

    bf16x8 qh[KS], ql[KS];
    {
        const bf16* q = p.rq2 + ((int64_t)(row0 + qc) * p.H + h) * KP + hh * 8;
#pragma unroll
        for (int ks = 0; ks < KS; ks++) { qh[ks] = *(const bf16x8*)(q + ks * 16); ql[ks] = *(const bf16x8*)(q + plane + ks * 16); }
    }
    for (int i = tid; i < RET_CHUNK + 33; i += 256) pwl[i] = i < 32 ? 0.f : p.pw[h * (RET_CHUNK + 1) + i - 32];
    __builtin_amdgcn_s_waitcnt(0x0F70);       // vmcnt(0) the compiler sees: without it the queries' first use waits for the fills below
    stage(0, 0);
    if (total > 1) stage(1, 1);
    f32x16 oacc[DB];
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int e = 0; e < 16; e++) oacc[db][e] = 0.f;
    close(-1);
    int slot = 0;                                             // ring place of the current tile
    auto ring = [](int i) { return i >= 3 ? i - 3 : i; };
    if (prior) {                                              // what came before the chunk
#pragma unroll
        for (int db = 0; db < DB; db++) {
            if (db + 2 < total) stage(ring(slot + 2), db + 2);
            if (w0 < S) {
                const char* base = smem + slot * BUF + lane * 16;
#pragma unroll
                for (int ks = 0; ks < KS; ks++) {
                    const bf16x8 sh = *(const bf16x8*)(base + ks * 2048), sl = *(const bf16x8*)(base + ks * 2048 + 1024);
                    oacc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sh, qh[ks], oacc[db], 0, 0, 0);
                    oacc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sl, qh[ks], oacc[db], 0, 0, 0);
                    oacc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sh, ql[ks], oacc[db], 0, 0, 0);
                }
            }
            close(db);
            slot = ring(slot + 1);
        }
        const float w = pwl[32 + qc - c0 + 1];
#pragma unroll
        for (int db = 0; db < DB; db++)
#pragma unroll
            for (int e = 0; e < 16; e++) oacc[db][e] *= w;
    }

    const int k_sw = kswz<KP>(l31);
    const int gq = lane >> 4, li = lane & 15, tq = li >> 2, tp = li & 3;
    const int v_row = 4 * hh + tq, v_sw = vswz<VP>(v_row), v_clow = (gq & 1) * 2 + (tp >> 1), v_off = v_row * VP * 2 + (tp & 1) * 8;
    for (int kt = 0; kt < nt; kt++) {
        const int key0 = c0 + kt * 32, u = ns + kt;
        if (u + 2 < total) stage(ring(slot + 2), u + 2);
        const char* base = smem + slot * BUF;
        if (w0 < S && key0 <= w0) {                           // (tiles and waves both start at multiples of 32: a later tile is all behind the wave's queries)
            f32x16 s;
#pragma unroll
            for (int e = 0; e < 16; e++) s[e] = 0.f;
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                const int at = l31 * KP * 2 + (((2 * ks + hh) ^ k_sw) * 16);
                const bf16x8 kf = *(const bf16x8*)(base + at), kl = *(const bf16x8*)(base + KB + at);
                s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qh[ks], s, 0, 0, 0);
                s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kl, qh[ks], s, 0, 0, 0);
                s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, ql[ks], s, 0, 0, 0);
            }
            unsigned ph[8], pl[8];
            const float* wl = pwl + 32 + qc - key0 - 4 * hh;  // decay of the lane's first key
#pragma unroll
            for (int i = 0; i < 8; i++) {
                const int e = 2 * i, k = (e & 3) + 8 * (e >> 2);
                const float x0 = s[e] * wl[-k], x1 = s[e + 1] * wl[-k - 1];
                ph[i] = pack2(x0, x1);
                pl[i] = pack2(x0 - lo16(ph[i]), x1 - hi16(ph[i]));
            }
#pragma unroll
            for (int ss = 0; ss < 2; ss++) {
                const bf16x8 pf = __builtin_bit_cast(bf16x8, (u32x4{ph[4 * ss], ph[4 * ss + 1], ph[4 * ss + 2], ph[4 * ss + 3]}));
                const bf16x8 lf = __builtin_bit_cast(bf16x8, (u32x4{pl[4 * ss], pl[4 * ss + 1], pl[4 * ss + 2], pl[4 * ss + 3]}));
#pragma unroll
                for (int db = 0; db < DB; db++) {
                    const bf16x8 vf = read_tr(base + 2 * KB + 16 * ss * VP * 2 + v_off + ((((db * 4) ^ v_sw) | v_clow) << 4), VP * 2);
                    oacc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf, oacc[db], 0, 0, 0);
                    oacc[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, lf, oacc[db], 0, 0, 0);
                }
            }
        }
        close(u);
        slot = ring(slot + 1);
    }

    // ---- norm over the head, gate, store: lane (query, half) owns d = 32 db + 8 g4 + 4 hh + 0..3 ----
    float ss = 0.f;
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int e = 0; e < 16; e++) ss += oacc[db][e] * oacc[db][e];
    ss += __shfl_xor(ss, 32, 64);
    if (qi >= S) return;
    const float rs = p.out_scale / sqrtf(ss / (float)p.vdim + p.eps);
    const bf16* gp = (const bf16*)p.g + (int64_t)(row0 + qi) * p.lda + h * VP + 4 * hh;
    bf16* op = (bf16*)p.ao + (int64_t)(row0 + qi) * p.ldo + (int64_t)h * p.vdim + 4 * hh;
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
        for (int g4 = 0; g4 < 4; g4++) {
            const int d = 32 * db + 8 * g4;
            if (d + 4 * hh >= p.vdim) continue;
            const bf16x4 gv = *(const bf16x4*)(gp + d);
            bf16x4 o;
#pragma unroll
            for (int e = 0; e < 4; e++) o[e] = f2bf(oacc[db][4 * g4 + e] * rs * silu(bf2f(gv[e])));
            if ((p.vdim & 3) == 0) *(bf16x4*)(op + d) = o;
            else
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (d + 4 * hh + e < p.vdim) op[d + e] = o[e];
        }
}

template <int KP, int VP>
int launch_out(const RetParams& p, hipStream_t st) {
    constexpr int LDS = 3 * 32 * 2 * (2 * KP + VP) + (RET_CHUNK + 36) * 4;
    static std::atomic<uint64_t> attr_done{0};
    if (!cr_dyn_lds_once(attr_done, (const void*)ret_out_kernel<KP, VP>, LDS)) return cr_fail(CR_ERR_HIP, "retention: LDS");
    hipLaunchKernelGGL((ret_out_kernel<KP, VP>), dim3((p.longest + 127) / 128, p.H, p.n_segs), dim3(256), LDS, st, p);
    CR_HIP(hipGetLastError());
    return CR_OK;
}
template <int KP>
int launch_out_k(const RetParams& p, hipStream_t st) {
    switch (p.Vp) {
        case 64: return launch_out<KP, 64>(p, st);
        case 128: return launch_out<KP, 128>(p, st);
        case 256: return launch_out<KP, 256>(p, st);
    }
    return cr_fail(CR_ERR_ARG, "retention: value size %d", p.Vp);
}

int check(const char* who, const RetParams& p) {
    auto size = [](int n) { return n == 64 || n == 128 || n == 256 || n == 512; };
    if (p.M <= 0 || p.H <= 0 || !size(p.Kp) || !size(p.Vp) || p.vdim <= 0 || p.vdim > p.Vp || !p.state || !p.pw || (p.lda & 7)) return cr_fail(CR_ERR_ARG, "%s: rows %d, heads %d, sizes %d / %d", who, p.M, p.H, p.Kp, p.Vp);
    return CR_OK;
}

template <typename T, int NR>
int decode_n(const RetParams& p, const AttnParams* merge, int dim, hipStream_t st) {
    const int waves = min(p.Vp / 16, dec_waves(NR)), extra = merge ? (merge->H * merge->Sq * (dim / 64) + waves - 1) / waves : 0;
    hipLaunchKernelGGL((ret_decode_kernel<T, NR>), dim3(p.H + extra, p.M), dim3(64 * waves), 0, st, p, merge ? *merge : AttnParams{}, dim);
    CR_HIP(hipGetLastError());
    return CR_OK;
}
template <typename T>
int decode_t(const RetParams& p, const AttnParams* merge, int dim, hipStream_t st) {
    switch (p.Kp) {
        case 64: return decode_n<T, 4>(p, merge, dim, st);
        case 128: return decode_n<T, 8>(p, merge, dim, st);
        case 256: return decode_n<T, 16>(p, merge, dim, st);
    }
    return decode_n<T, 32>(p, merge, dim, st);
}

template <typename T>
int recurrent_t(const RetParams& p, hipStream_t st) {
    const dim3 grid(p.Vp / 64, p.H, p.n_segs);
    switch (p.Kp) {
        case 64: hipLaunchKernelGGL((ret_recurrent_kernel<T, 4>), grid, dim3(256), 0, st, p); break;
        case 128: hipLaunchKernelGGL((ret_recurrent_kernel<T, 8>), grid, dim3(256), 0, st, p); break;
        case 256: hipLaunchKernelGGL((ret_recurrent_kernel<T, 16>), grid, dim3(256), 0, st, p); break;
        default: hipLaunchKernelGGL((ret_recurrent_kernel<T, 32>), grid, dim3(256), 0, st, p); break;
    }
    CR_HIP(hipGetLastError());
    hipLaunchKernelGGL(ret_gate_kernel<T>, dim3((unsigned)p.M, (p.H + 3) / 4), dim3(256), 0, st, p);
    CR_HIP(hipGetLastError());
    return CR_OK;
}

}  // namespace

bool ret_matrix_supported(int Kp, int Vp) { return Kp <= 256 && Vp <= 256; }

int launch_ret_decode(bool f32, const RetParams& p, const AttnParams* merge, int merge_dim, hipStream_t st) {
    CR_TRY(check("retention (decode)", p));
    if (!p.rq || !p.rk || !p.ix.seqs || !p.ix.lens) return cr_fail(CR_ERR_ARG, "retention (decode): operands");
    if (merge && (merge_dim <= 0 || merge_dim % 64 || merge->B != p.M || merge->H <= 0 || merge->Sq <= 0 || merge->nsplit <= 0 || !merge->part_o || !merge->part_ml || !merge->O))
        return cr_fail(CR_ERR_ARG, "retention (decode): splits to merge");
    return f32 ? decode_t<float>(p, merge, merge_dim, st) : decode_t<bf16>(p, merge, merge_dim, st);
}

int launch_ret_recurrent(bool f32, const RetParams& p, hipStream_t st) {
    CR_TRY(check("retention (recurrent)", p));
    if (!p.rq || !p.rk || !p.raw || !p.seg || p.n_segs <= 0) return cr_fail(CR_ERR_ARG, "retention (recurrent): operands");
    return f32 ? recurrent_t<float>(p, st) : recurrent_t<bf16>(p, st);
}

int launch_ret_matrix(const RetParams& p, hipStream_t st) {
    CR_TRY(check("retention (matrix)", p));
    if (!ret_matrix_supported(p.Kp, p.Vp) || !p.rq2 || !p.rk2 || !p.snap || !p.seg || !p.snap0 || !p.chunks || p.n_chunks <= 0 || p.n_segs <= 0 || p.longest <= 0 || p.n_segs > 65535 ||
        (int64_t)RET_CHUNK * std::max<int64_t>(p.lda * 2, (int64_t)p.H * p.Kp * 2) >= (1ll << 31)) return cr_fail(CR_ERR_ARG, "retention (matrix): operands");
    for (int i = 0; i < p.n_chunks; i += 32768) {             // (a grid's third dimension)
        RetParams q = p;
        q.chunks += 2 * (size_t)i; q.snap += (int64_t)i * p.H * 2 * p.Vp * p.Kp;
        hipLaunchKernelGGL(ret_chunk_kernel, dim3(p.Kp / 64 * (p.Vp / 64), p.H, min(32768, p.n_chunks - i)), dim3(256), 0, st, q);
        CR_HIP(hipGetLastError());
    }
    hipLaunchKernelGGL(ret_scan_kernel, dim3((p.Vp * p.Kp / 8 + 255) / 256, p.H, p.n_segs), dim3(256), 0, st, p);
    CR_HIP(hipGetLastError());
    switch (p.Kp) {
        case 64: return launch_out_k<64>(p, st);
        case 128: return launch_out_k<128>(p, st);
        case 256: return launch_out_k<256>(p, st);
    }
    return CR_ERR_ARG;
}
