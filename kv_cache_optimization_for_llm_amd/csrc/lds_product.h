// A bf16 product of many rows on the matrix cores, operands through LDS: the middle of kernels that differ in
// where their operands' rows lie and in what they do with the result (experts' products, products per head).
//
// A workgroup of four wavefronts takes 32 RT rows of x and 128 outputs (rows of w), a wavefront half of
// either.  64 elements of K of both operands go through LDS at a time, two deep (the next ones' loads are in
// flight while these are multiplied), in rows padded so that a fragment's 16 lanes lie on banks of their own.
// K (a multiple of 8) is added in ascending order into one accumulator an output.
#pragma once
#include "common.h"
#include "attention_frag.h"

#define LDSP_K 64
#define LDSP_STRIDE 72
#define LDSP_N 128

template <int RT>
struct LdsProduct {
    static constexpr int ROWS = 32 * RT;
    static constexpr int XI = ROWS * LDSP_K / 8 / 256, WI = LDSP_N * LDSP_K / 8 / 256;      // 16-byte pieces a thread loads
    struct Shared {
        bf16_t x[2][ROWS * LDSP_STRIDE], w[2][LDSP_N * LDSP_STRIDE];
    };
    // Thread t loads elements 8 (t % 8) .. of rows t / 8 + 32 i of x: `xp` points at its first element of the row.
    // Its pieces of w are the caller's choice: `wp` their first elements, `wkc` their place in the 64 elements,
    // `wat` where they go in LDS; `wmul` elements of w's storage go by per element of K.
    const bf16_t *xp[XI], *wp[WI];
    int wat[WI], wkc[WI], wmul;

    __device__ __forceinline__ static int row() { return threadIdx.x / 8; }
    __device__ __forceinline__ static int element() { return 8 * (threadIdx.x % 8); }

    // w row by row, rows n0 .. n0 + 127 (past the last one the last one again)
    __device__ __forceinline__ void plain_w(const bf16_t *w, int N, int K, int n0) {
        wmul = 1;
#pragma unroll
        for (int i = 0; i < WI; ++i) {
            wkc[i] = element();
            wat[i] = (row() + 32 * i) * LDSP_STRIDE + wkc[i];
            wp[i] = w + (size_t)min(n0 + row() + 32 * i, N - 1) * K + wkc[i];
        }
    }
    // w in operand order [N / 16][K / 32][lane][8]: a wavefront's pieces are neighbouring bytes
    __device__ __forceinline__ void tiled_w(const bf16_t *w, int N, int K, int n0) {
        const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
        wmul = 16;
#pragma unroll
        for (int i = 0; i < WI; ++i) {
            const int f = wave + 4 * i, nt = f >> 1;
            wkc[i] = 32 * (f & 1) + 8 * g;
            wat[i] = (16 * nt + r) * LDSP_STRIDE + wkc[i];
            wp[i] = w + (size_t)min(n0 + 16 * nt, N - 16) * K + (f & 1) * 16 * 32 + 8 * lane;
        }
    }

    // acc[nt][rt]: lane (r = lane % 16, g = lane / 16) of wavefront (half of the rows wave % 2, of the outputs
    // wave / 2) gets outputs 64 (wave / 2) + 16 nt + 4 g .. + 3 of row (wave % 2) 16 RT + 16 rt + r
    __device__ __forceinline__ void run(Shared &s, int K, f32x4 (&acc)[4][RT]) const {
        const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
        const int wr = wave & 1, wn = wave >> 1, kc = element();
        uint4 xv[XI], wv[WI];
#define LDSP_LOAD(K0)                                                                                                    \
    {                                                                                                                    \
        _Pragma("unroll") for (int i = 0; i < XI; ++i)                                                                   \
            xv[i] = (K0) + kc < K ? *reinterpret_cast<const uint4 *>(xp[i] + (K0)) : make_uint4(0u, 0u, 0u, 0u);          \
        _Pragma("unroll") for (int i = 0; i < WI; ++i)                                                                   \
            wv[i] = (K0) + wkc[i] < K ? *reinterpret_cast<const uint4 *>(wp[i] + (K0) * wmul) : make_uint4(0u, 0u, 0u, 0u); \
    }
#pragma unroll
        for (int nt = 0; nt < 4; ++nt)
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) acc[nt][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
        LDSP_LOAD(0)
        int buf = 0;
        for (int k0 = 0; k0 < K; k0 += LDSP_K, buf ^= 1) {
#pragma unroll
            for (int i = 0; i < XI; ++i) *reinterpret_cast<uint4 *>(&s.x[buf][(row() + 32 * i) * LDSP_STRIDE + kc]) = xv[i];
#pragma unroll
            for (int i = 0; i < WI; ++i) *reinterpret_cast<uint4 *>(&s.w[buf][wat[i]]) = wv[i];
            __syncthreads();            // (a buffer was read last two turns ago: every wavefront has passed the barrier between)
            if (k0 + LDSP_K < K) LDSP_LOAD(k0 + LDSP_K)
            const bf16_t *xr = &s.x[buf][(wr * 16 * RT + r) * LDSP_STRIDE + 8 * g], *wrow = &s.w[buf][(wn * 64 + r) * LDSP_STRIDE + 8 * g];
            Frag8 xf[2][RT], wf[2][4];
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
#pragma unroll
                for (int nt = 0; nt < 4; ++nt) wf[ks][nt].u4 = *reinterpret_cast<const uint4 *>(wrow + nt * 16 * LDSP_STRIDE + 32 * ks);
#pragma unroll
                for (int rt = 0; rt < RT; ++rt) xf[ks][rt].u4 = *reinterpret_cast<const uint4 *>(xr + rt * 16 * LDSP_STRIDE + 32 * ks);
            }
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                for (int nt = 0; nt < 4; ++nt)
#pragma unroll
                    for (int rt = 0; rt < RT; ++rt)
                        acc[nt][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[ks][nt].v, xf[ks][rt].v, acc[nt][rt], 0, 0, 0);
        }
#undef LDSP_LOAD
    }
};

// Workgroup id -> place in the work list such that neighbours of the list run on one of the 8 dies (the hardware
// deals workgroups out in turn): what they share is read into one L2.
__device__ __forceinline__ int die_order(int id, int total) {
    const int die = id % 8, q = total / 8, rem = total % 8;
    return die * q + min(die, rem) + id / 8;
}
