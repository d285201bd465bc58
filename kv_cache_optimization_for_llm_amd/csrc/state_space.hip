// The recurrence of a state-space mixer whose decay is one number per head and token:
//
//     S_t = exp(-rate_h dt_t) S_(t-1) + dt_t B_t x_t^T,    y_t = S_t^T C_t + D_h x_t,
//
// S [state, value] per head, dt_t = softplus(y[t, dt_off + h] + dt_bias_h), rate_h = exp(A_log_h).  B and C
// belong to groups of heads.  S is fp32, starts at zero and lives in the seat's state row between steps.
//
// kva_state_space_scan walks the tokens.  Value columns of S are independent of each other: a workgroup of
// four wavefronts takes 16 of a head's, a wavefront 4, the 16 lanes of a row of the wavefront share a column
// and keep its part of S in registers (rows 4 (16 j + r) .. + 3 for lane r).  A chunk of tokens - B, C, the
// 16 columns of x, the two numbers of every token - is staged in LDS for the four wavefronts while the one
// before is walked.  The order of every sum depends on the sizes alone: a token's result is the same bit for
// bit however the request's tokens were cut into steps and whatever else the step holds.
#include "common.h"
#include <math.h>

#define SSM_COLS 4           // columns a wavefront
#define SSM_LANES 16         // lanes that share a column
#define SSM_WAVES 4
#define SSM_BLOCK_COLS (SSM_COLS * SSM_WAVES)
#define SSM_THREADS (KVA_WAVE * SSM_WAVES)
#define SSM_MAX_STATE 512

struct SsmArgs {
    float *out;                 // [T, heads * vdim] fp32
    float *state;               // seat rows; this mixer's S [heads, state, vdim] at state_off
    size_t seat_stride;
    int state_off;
    const int *entry_q_start, *entry_seat;
    const float *xbc;           // [T, xbc_stride]: x (heads x vdim), B (groups x state), C (groups x state)
    int xbc_stride;
    const void *y;              // the projection's rows, which hold dt's input
    int y_dtype, y_stride, dt_off;
    const float *a_log, *dt_bias, *d_skip;
    int heads, groups, n, vdim; // n: the state's size
};

__device__ inline float ssm_ld(const void *p, int dtype, size_t i) {
    return dtype == KVA_BF16 ? bf16_bits_to_float(reinterpret_cast<const uint16_t *>(p)[i]) : reinterpret_cast<const float *>(p)[i];
}
__device__ inline float ssm_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

template <int RP, int CH>
__global__ void __launch_bounds__(SSM_THREADS)
state_space_scan_kernel(SsmArgs a) {
    constexpr int NP = SSM_LANES * RP, NS = NP + 4, PER = CH * NP / SSM_THREADS;    // token rows 4 banks apart
    constexpr int VPER = CH * SSM_BLOCK_COLS / SSM_THREADS < 1 ? 1 : CH * SSM_BLOCK_COLS / SSM_THREADS;
    __shared__ __attribute__((aligned(16))) float bs[CH * NS];
    __shared__ __attribute__((aligned(16))) float cs[CH * NS];
    __shared__ float xs[CH * SSM_BLOCK_COLS], os[CH * SSM_BLOCK_COLS], keep_s[CH], dt_s[CH];
    const int tid = threadIdx.x, lane = tid % KVA_WAVE, wave = tid / KVA_WAVE;
    const int c = lane / SSM_LANES, r = lane % SSM_LANES;
    const int slices = (a.vdim + SSM_BLOCK_COLS - 1) / SSM_BLOCK_COLS;
    const int head = blockIdx.x / slices, col0 = (blockIdx.x % slices) * SSM_BLOCK_COLS;
    const int col = col0 + wave * SSM_COLS + c;
    const int e = blockIdx.y;
    const int q0 = a.entry_q_start[e], len = a.entry_q_start[e + 1] - q0;
    if (len <= 0) return;
    const int n = a.n, dv = a.vdim, grp = head / (a.heads / a.groups);
    const bool on = col < dv;
    float *Sg = a.state + (size_t)a.entry_seat[e] * a.seat_stride + a.state_off + (size_t)head * n * dv;
    float S[RP];
#pragma unroll
    for (int j = 0; j < RP; ++j) {
        const int i = 4 * (SSM_LANES * (j / 4) + r) + j % 4;
        S[j] = (on && i < n) ? Sg[(size_t)i * dv + col] : 0.f;
    }
    const int x_col = head * dv + col0, b_col = a.heads * dv + grp * n, c_col = b_col + a.groups * n;
    const float rate = expf(a.a_log[head]), bias = a.dt_bias[head], skip = a.d_skip[head];
    float pb[PER], pc[PER], px[VPER], pd = 0.f;
    auto fetch = [&](int t0, int m) {
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            pb[j] = pc[j] = 0.f;
            if (SSM_THREADS * j / NP >= m) continue;        // (the whole workgroup: a decoded token loads one row)
            const int x = tid + SSM_THREADS * j, tt = x / NP, i = x % NP;
            if (tt >= m || i >= n) continue;
            const float *row = a.xbc + (size_t)(q0 + t0 + tt) * a.xbc_stride;
            pb[j] = row[b_col + i];
            pc[j] = row[c_col + i];
        }
#pragma unroll
        for (int j = 0; j < VPER; ++j) {
            const int x = tid + SSM_THREADS * j, tt = x / SSM_BLOCK_COLS, cc = x % SSM_BLOCK_COLS;
            px[j] = (tt < m && col0 + cc < dv) ? a.xbc[(size_t)(q0 + t0 + tt) * a.xbc_stride + x_col + cc] : 0.f;
        }
        if (tid < m) pd = ssm_ld(a.y, a.y_dtype, (size_t)(q0 + t0 + tid) * a.y_stride + a.dt_off + head);
    };
    fetch(0, min(CH, len));
    for (int t0 = 0; t0 < len; t0 += CH) {
        const int m = min(CH, len - t0);
        __syncthreads();
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int x = tid + SSM_THREADS * j, at = (x / NP) * NS + x % NP;
            bs[at] = pb[j];
            cs[at] = pc[j];
        }
#pragma unroll
        for (int j = 0; j < VPER; ++j)
            if (tid + SSM_THREADS * j < CH * SSM_BLOCK_COLS) xs[tid + SSM_THREADS * j] = px[j];
        if (tid < m) {
            const float dt = ssm_softplus(pd + bias);
            dt_s[tid] = dt;
            keep_s[tid] = expf(-rate * dt);
        }
        __syncthreads();
        if (t0 + CH < len) fetch(t0 + CH, min(CH, len - t0 - CH));
        // four tokens at a time: only S is handed from token to token, the four read-outs' sums over the rows
        // are independent of each other and stand side by side
        auto step = [&](int tt, float (&o)[4], float &xv) {
            const float4 *b4 = reinterpret_cast<const float4 *>(bs + tt * NS) + r;
            const float4 *c4 = reinterpret_cast<const float4 *>(cs + tt * NS) + r;
            const float keep = keep_s[tt];
            xv = xs[tt * SSM_BLOCK_COLS + wave * SSM_COLS + c];
            const float v = dt_s[tt] * xv;
            o[0] = o[1] = o[2] = o[3] = 0.f;
#pragma unroll
            for (int j = 0; j < RP / 4; ++j) {
                const float4 bb = b4[SSM_LANES * j], cc = c4[SSM_LANES * j];
                S[4 * j] = keep * S[4 * j] + bb.x * v;
                S[4 * j + 1] = keep * S[4 * j + 1] + bb.y * v;
                S[4 * j + 2] = keep * S[4 * j + 2] + bb.z * v;
                S[4 * j + 3] = keep * S[4 * j + 3] + bb.w * v;
                o[0] += S[4 * j] * cc.x;
                o[1] += S[4 * j + 1] * cc.y;
                o[2] += S[4 * j + 2] * cc.z;
                o[3] += S[4 * j + 3] * cc.w;
            }
        };
        int tt = 0;
        for (; tt + 4 <= m; tt += 4) {
            float o[4][4], xv[4], sum[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) step(tt + i, o[i], xv[i]);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum[i] = (o[i][0] + o[i][1]) + (o[i][2] + o[i][3]);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum[i] += row16_rotated<8>(sum[i]);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum[i] += row16_rotated<4>(sum[i]);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum[i] += row16_rotated<2>(sum[i]);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum[i] += row16_rotated<1>(sum[i]);
            if (r == 0)
#pragma unroll
                for (int i = 0; i < 4; ++i) os[(tt + i) * SSM_BLOCK_COLS + wave * SSM_COLS + c] = sum[i] + skip * xv[i];
        }
        for (; tt < m; ++tt) {
            float o[4], xv;
            step(tt, o, xv);
            const float sum = row16_sum((o[0] + o[1]) + (o[2] + o[3]));
            if (r == 0) os[tt * SSM_BLOCK_COLS + wave * SSM_COLS + c] = sum + skip * xv;
        }
        __syncthreads();
        // the chunk's read-outs leave together, 16 neighbouring columns a token
#pragma unroll
        for (int j = 0; j < VPER; ++j) {
            const int x = tid + SSM_THREADS * j, tt = x / SSM_BLOCK_COLS, cc = x % SSM_BLOCK_COLS;
            if (tt < m && col0 + cc < dv) a.out[(size_t)(q0 + t0 + tt) * a.heads * dv + x_col + cc] = os[x];
        }
    }
    if (on)
#pragma unroll
        for (int j = 0; j < RP; ++j) {
            const int i = 4 * (SSM_LANES * (j / 4) + r) + j % 4;
            if (i < n) Sg[(size_t)i * dv + col] = S[j];
        }
}

extern "C" int kva_state_space_scan(float *out, float *state, long long seat_stride, int state_off, const float *xbc,
                                    int xbc_stride, const void *y, int y_dtype, int y_stride, int dt_off, const float *a_log,
                                    const float *dt_bias, const float *d_skip, const int *entry_q_start,
                                    const int *entry_seat, int entries, int heads, int groups, int n, int vdim,
                                    hipStream_t stream) {
    KVA_REQUIRE(out && state && xbc && y && a_log && dt_bias && d_skip && entry_q_start && entry_seat,
                "state_space_scan: missing operand");
    KVA_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && vdim > 0, "state_space_scan: %d heads in %d groups", heads, groups);
    KVA_REQUIRE(n > 0 && n <= SSM_MAX_STATE, "state_space_scan: state size %d must lie in 1..%d", n, SSM_MAX_STATE);
    KVA_REQUIRE(xbc_stride >= heads * vdim + 2 * groups * n && dt_off >= 0 && y_stride >= dt_off + heads,
                "state_space_scan: the rows are too short for what they hold");
    KVA_REQUIRE(entries >= 0 && entries <= 65535, "state_space_scan: %d entries", entries);
    if (entries == 0) return KVA_OK;
    const SsmArgs a{out, state, (size_t)seat_stride, state_off, entry_q_start, entry_seat, xbc, xbc_stride, y, y_dtype,
                    y_stride, dt_off, a_log, dt_bias, d_skip, heads, groups, n, vdim};
    const dim3 grid(heads * ((vdim + SSM_BLOCK_COLS - 1) / SSM_BLOCK_COLS), entries);
    if (n <= 64) hipLaunchKernelGGL((state_space_scan_kernel<4, 32>), grid, dim3(SSM_THREADS), 0, stream, a);
    else if (n <= 128) hipLaunchKernelGGL((state_space_scan_kernel<8, 32>), grid, dim3(SSM_THREADS), 0, stream, a);
    else if (n <= 256) hipLaunchKernelGGL((state_space_scan_kernel<16, 16>), grid, dim3(SSM_THREADS), 0, stream, a);
    else hipLaunchKernelGGL((state_space_scan_kernel<32, 8>), grid, dim3(SSM_THREADS), 0, stream, a);
    KVA_CHECK_LAUNCH("state_space_scan");
    return KVA_OK;
}
