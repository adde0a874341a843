// Merge of the key splits of one decoded query row (attention.hip, attention_decode.hip leave the partials): a device function, so that a kernel beside the attention can do it.
#pragma once
#include "attention.hpp"

// out[b][q][h][d] = sum_s exp(m_s - M) O_s / sum_s exp(m_s - M) l_s   (splits in index order: reproducible); the 64 lanes of a wave hold 64 values of d, D columns in all
// A wave's lane s fetches split s's (m, l) -- one round trip for up to 64 splits, maximum and weights by shuffles -- and the O rows are
// loaded eight at a time with independent loads (a plain loop over the run-time split count waited for every load in turn: 13
// dependent round trips per launch at 3 300 cached tokens, 11.5 us x 32 layers per decode step).
__device__ __forceinline__ void attn_merge_splits(const AttnParams& p, int D, int batch, int head, int q, int d) {
    const int lane = threadIdx.x & 63;
    const int64_t base = ((int64_t)batch * p.H + head) * p.nsplit;
    float M = -INFINITY;
    for (int s0 = 0; s0 < p.nsplit; s0 += 64) {
        const int s = s0 + lane;
        M = fmaxf(M, wave_max(s < p.nsplit ? p.part_ml[((base + s) * p.Sq + q) * 2] : -INFINITY));
    }
    float L = 0.f, acc = 0.f;
    for (int s0 = 0; s0 < p.nsplit; s0 += 64) {
        const int s = s0 + lane;
        const bool in = s < p.nsplit;
        const int64_t row = (base + (in ? s : 0)) * p.Sq + q;
        const float w = in ? __expf(p.part_ml[row * 2] - M) : 0.f;
        const float wl = in ? w * p.part_ml[row * 2 + 1] : 0.f;
        const int n = min(64, p.nsplit - s0);
        for (int j0 = 0; j0 < n; j0 += 8) {
            float o[8];
#pragma unroll
            for (int j = 0; j < 8; j++) o[j] = j0 + j < n ? p.part_o[((base + s0 + j0 + j) * p.Sq + q) * D + d] : 0.f;
#pragma unroll
            for (int j = 0; j < 8; j++) {                    // index order; lanes past the count carry weight 0
                L += __shfl(wl, j0 + j, 64);
                acc += __shfl(w, j0 + j, 64) * o[j];
            }
        }
    }
    if (p.wide && d >= p.vdim) return;
    p.O[(int64_t)batch * p.o_bs + (int64_t)q * p.o_rs + (int64_t)head * p.o_hs + d] = f2bf(p.wide && p.out_mul != 0.f ? p.out_mul * acc / L : acc / L);
}
