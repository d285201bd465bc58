// The recurrence of a state-space mixer whose decay is one number per head and token:
//
//     S_t = exp(-rate_h dt_t) S_(t-1) + dt_t B_t x_t^T,    y_t = S_t^T C_t + D_h x_t,
//
// S [state, value] per head, dt_t = softplus(y[t, dt_off + h] + dt_bias_h), rate_h = exp(A_log_h).  B and C
// belong to groups of heads.  S is fp32, starts at zero and lives in the seat's state row between steps.
//
// Three kernels; each takes the entries whose number of tokens lies in a range the caller names.
//
//  * state_space_scan_kernel walks the tokens.  Value columns of S are independent of each other: a workgroup
//    of four wavefronts takes 16 of a head's, a wavefront 4, the 16 lanes of a row of the wavefront share a
//    column and keep its part of S in registers (rows 4 (16 j + r) .. + 3 for lane r).  A chunk of tokens - B,
//    C, the 16 columns of x, the two numbers of every token - is staged in LDS for the four wavefronts while
//    the one before is walked.  The order of every sum depends on the sizes alone.
//  * state_space_token_kernel is a single token: S passes through registers once, 16 bytes a lane.
//  * state_space_chunk_kernel (bf16 rows) takes chunks of 64 tokens on the matrix cores.  With c_t the sum of
//    -rate dt up to t inside the chunk and S_0 the state in front of it,
//        y_t = sum_(s <= t) (C_t . B_s) e^(c_t - c_s) dt_s x_s + e^(c_t) S_0^T C_t + D x_t,
//        S   = e^(c_64) S_0 + sum_s B_s (e^(c_64 - c_s) dt_s x_s)^T.
//    B, C and x are what the convolution left in bf16 and enter the products as they are; what is formed in
//    32-bit here - the weights of the first sum, S_0 and the weighted x - enters as the sum of two bf16 numbers
//    (a product each, some 17 bits), the accumulators and S are fp32.
#include "common.h"
#include "attention_frag.h"
#include "lds_product.h"
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
    const void *xbc;            // [T, xbc_stride]: x (heads x vdim), B (groups x state), C (groups x state)
    int xbc_dtype, xbc_stride;
    const void *y;              // the projection's rows, which hold dt's input
    int y_dtype, y_stride, dt_off;
    const float *a_log, *dt_bias, *d_skip;
    int heads, groups, n, vdim; // n: the state's size
    int len_lo, len_hi;         // entries of so many tokens
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
    if (len < a.len_lo || len > a.len_hi) return;
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
            const size_t row = (size_t)(q0 + t0 + tt) * a.xbc_stride;
            pb[j] = ssm_ld(a.xbc, a.xbc_dtype, row + b_col + i);
            pc[j] = ssm_ld(a.xbc, a.xbc_dtype, row + c_col + i);
        }
#pragma unroll
        for (int j = 0; j < VPER; ++j) {
            const int x = tid + SSM_THREADS * j, tt = x / SSM_BLOCK_COLS, cc = x % SSM_BLOCK_COLS;
            px[j] = (tt < m && col0 + cc < dv) ? ssm_ld(a.xbc, a.xbc_dtype, (size_t)(q0 + t0 + tt) * a.xbc_stride + x_col + cc) : 0.f;
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


// ---- a single token -----------------------------------------------------------------------------------
// A workgroup takes 64 value columns of a head, thread (row group rg of 16, column group cg of 16) the four
// columns 4 cg .. of rows rg, rg + 16, ..: 8 rows' loads in flight, 16 bytes each.  The read-out's sums meet in
// LDS in a fixed order.  (vdim is a multiple of 4.)
#define SSM_TOKEN_ROWS 8

__global__ void __launch_bounds__(256)
state_space_token_kernel(SsmArgs a) {
    __shared__ float4 red[4][16];
    const int slices = (a.vdim + 63) / 64;
    const int head = blockIdx.x / slices, e = blockIdx.y;
    const int q0 = a.entry_q_start[e], len = a.entry_q_start[e + 1] - q0;
    if (len < a.len_lo || len > a.len_hi) return;
    const int cg = threadIdx.x % 16, rg = threadIdx.x / 16, lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE;
    const int n = a.n, dv = a.vdim, grp = head / (a.heads / a.groups), col = (blockIdx.x % slices) * 64 + 4 * cg;
    const bool on = col < dv;
    float *Sg = a.state + (size_t)a.entry_seat[e] * a.seat_stride + a.state_off + (size_t)head * n * dv + col;
    const size_t row = (size_t)q0 * a.xbc_stride;
    const size_t b_at = row + a.heads * dv + (size_t)grp * n, c_at = b_at + (size_t)a.groups * n;
    const float dt = ssm_softplus(ssm_ld(a.y, a.y_dtype, (size_t)q0 * a.y_stride + a.dt_off + head) + a.dt_bias[head]);
    const float keep = expf(-expf(a.a_log[head]) * dt), skip = a.d_skip[head];
    float x[4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) x[i] = on ? ssm_ld(a.xbc, a.xbc_dtype, row + head * dv + col + i) : 0.f;
    for (int r0 = rg; r0 < n; r0 += 16 * SSM_TOKEN_ROWS) {
        float4 S[SSM_TOKEN_ROWS];
        float b[SSM_TOKEN_ROWS], c[SSM_TOKEN_ROWS];
#pragma unroll
        for (int k = 0; k < SSM_TOKEN_ROWS; ++k) {
            const int r = r0 + 16 * k;
            const bool in = on && r < n;
            S[k] = in ? *reinterpret_cast<const float4 *>(Sg + (size_t)r * dv) : make_float4(0.f, 0.f, 0.f, 0.f);
            b[k] = in ? ssm_ld(a.xbc, a.xbc_dtype, b_at + r) : 0.f;
            c[k] = in ? ssm_ld(a.xbc, a.xbc_dtype, c_at + r) : 0.f;
        }
#pragma unroll
        for (int k = 0; k < SSM_TOKEN_ROWS; ++k) {
            const int r = r0 + 16 * k;
            const float w = b[k] * dt;
            S[k].x = keep * S[k].x + w * x[0];
            S[k].y = keep * S[k].y + w * x[1];
            S[k].z = keep * S[k].z + w * x[2];
            S[k].w = keep * S[k].w + w * x[3];
            o[0] += S[k].x * c[k];
            o[1] += S[k].y * c[k];
            o[2] += S[k].z * c[k];
            o[3] += S[k].w * c[k];
            if (on && r < n) *reinterpret_cast<float4 *>(Sg + (size_t)r * dv) = S[k];
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = quad_rows_sum(o[i]);       // the wavefront's four row groups
    if (lane < 16) red[wave][cg] = make_float4(o[0], o[1], o[2], o[3]);
    __syncthreads();
    if (threadIdx.x >= 16 || !on) return;
    float4 v = red[0][cg];
#pragma unroll
    for (int w = 1; w < 4; ++w) {
        v.x += red[w][cg].x; v.y += red[w][cg].y; v.z += red[w][cg].z; v.w += red[w][cg].w;
    }
    *reinterpret_cast<float4 *>(a.out + (size_t)q0 * a.heads * dv + head * dv + col) =
        make_float4(v.x + skip * x[0], v.y + skip * x[1], v.z + skip * x[2], v.w + skip * x[3]);
}

// ---- chunks of 64 tokens on the matrix cores -------------------------------------------------------------
// A workgroup takes 16 value columns of a head and walks the entry's chunks; NK = state size / 32 (rounded up,
// the rest is zero).  Everything is computed transposed: lane (r = lane % 16, g = lane / 16) of a product's result
// holds rows 4 g .. + 3 of column r.  Wavefront w takes the chunk's tokens t = 16 w .. + 15 as columns:
//   (1) G^T[s, t] = B_s . C_t for the tiles s <= t;
//   (2) the weights e^(c_t - c_s) dt_s G, in registers the second operand of y^T[p, t] = sum_s x^T[p, s] W^T[s, t],
//       whose first operand is x read from LDS with the transposing load (k index: the permutation of 32 tokens
//       in which (1) left them);
//   (3) e^(c_t) S_0^T C with S_0^T [p, state] in LDS;
//   (4) the wavefront's part of the state, tiles of 16 state rows w, w + 4, ..: S^T[p, n] = e^(c_64) S^T + sum_s
//       (weighted x)^T[p, s] B[s, n], both operands by transposing loads.
// S lives in registers and lies, as two bf16 numbers, in LDS for (3), two buffers deep: two barriers a chunk.  The
// next chunk's rows are loaded while this one is worked on.
#define SSM_CHUNK 64
#define SSM_XS 24                // LDS stride of rows of 16 columns of x

typedef __attribute__((address_space(3))) s16x4 ssm_lds_s16x4;

// row stride in LDS, in elements, of rows of n (a multiple of 32): an odd multiple of 4 words whose first three
// multiples stay 8 banks away from each other
constexpr int ssm_stride(int n) {
    for (int words = n / 2;; ++words) {
        bool fits = words % 8 == 4;
        for (int i = 1; i < 4; ++i) {
            const int d = (i * words) % 64;
            fits = fits && d >= 8 && d <= 56;
        }
        if (fits) return 2 * words;
    }
}

// 8 tokens (rows) of column r behind `at` as an operand: `at` is the lane's place in the 32 rows (row 4 g + r / 4,
// column 4 (r % 4))
__device__ __forceinline__ Frag8 ssm_transposed(const bf16_t *at, int stride) {
    union { s16x4 t[2]; Frag8 f; } u;
    u.t[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ssm_lds_s16x4 *)at);
    u.t[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ssm_lds_s16x4 *)(at + 16 * stride));
    return u.f;
}

__device__ __forceinline__ void ssm_split(float v, uint16_t &hi, uint16_t &lo) {
    hi = float_to_bf16_bits(v);
    lo = float_to_bf16_bits(v - bf16_bits_to_float(hi));
}

template <int NK>
struct SsmChunkLds {
    static constexpr int ST = ssm_stride(32 * NK);
    bf16_t b[SSM_CHUNK * ST], c[SSM_CHUNK * ST];
    bf16_t s[2][2][16 * ST];                            // [buffer][high, low part][p][state]
    bf16_t x[SSM_CHUNK * SSM_XS], wx[2][SSM_CHUNK * SSM_XS];
    float cum[SSM_CHUNK], dt[SSM_CHUNK];
};

template <int NK>
__global__ void __launch_bounds__(256)
state_space_chunk_kernel(SsmArgs a) {
    constexpr int NP = 32 * NK, ST = SsmChunkLds<NK>::ST, TILES = (2 * NK + 3) / 4;      // tiles of 16 state rows a wavefront
    constexpr int PIECES = SSM_CHUNK * NP / 8 / 256;                                     // 16-byte pieces of B (and of C) a thread
    constexpr float LOG2E = 1.44269504088896340736f;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    SsmChunkLds<NK> &L = *reinterpret_cast<SsmChunkLds<NK> *>(lds_raw);
    const int tid = threadIdx.x, lane = tid % KVA_WAVE, w = tid / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int slices = (a.vdim + 15) / 16, id = die_order(blockIdx.x, gridDim.x);
    const int head = id / slices, p0 = (id % slices) * 16, e = blockIdx.y;
    const int q0 = a.entry_q_start[e], len = a.entry_q_start[e + 1] - q0;
    if (len < a.len_lo || len > a.len_hi) return;
    const int n = a.n, dv = a.vdim, grp = head / (a.heads / a.groups);
    const bf16_t *xbc = reinterpret_cast<const bf16_t *>(a.xbc);
    const int x_col = head * dv + p0, b_col = a.heads * dv + grp * n, c_col = b_col + a.groups * n;
    const float rate = expf(a.a_log[head]) * LOG2E, bias = a.dt_bias[head], skip = a.d_skip[head];
    float *Sg = a.state + (size_t)a.entry_seat[e] * a.seat_stride + a.state_off + (size_t)head * n * dv + p0 + 4 * g;
    const bool p_on = p0 + 4 * g < dv;                                   // (dv is a multiple of 4)
    // S^T tile k of this wavefront: rows p = 4 g .. + 3, column 16 (w + 4 k) + r
    f32x4 S[TILES];
#pragma unroll
    for (int k = 0; k < TILES; ++k) {
        const int i = 16 * (w + 4 * k) + r;
        S[k] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (p_on && i < n) {
            const float4 v = *reinterpret_cast<const float4 *>(Sg + (size_t)i * dv);
            S[k] = f32x4{v.x, v.y, v.z, v.w};
        }
    }
    auto leave_state = [&](int buf) {
#pragma unroll
        for (int k = 0; k < TILES; ++k) {
            const int i = 16 * (w + 4 * k) + r;
            if (i >= NP) continue;
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                uint16_t hi, lo;
                ssm_split(S[k][q], hi, lo);
                L.s[buf][0][(4 * g + q) * ST + i].bits = hi;
                L.s[buf][1][(4 * g + q) * ST + i].bits = lo;
            }
        }
    };
    leave_state(0);

    uint4 pb[PIECES], pc[PIECES];
    uint2 px;
    float pd;
    auto fetch = [&](int t0, int m) {
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + 256 * j, tt = i / (NP / 8), k = 8 * (i % (NP / 8));
            const bool in = tt < m && k < n;                             // (n is a multiple of 8)
            const bf16_t *row = xbc + (size_t)(q0 + t0 + (in ? tt : 0)) * a.xbc_stride;
            pb[j] = in ? *reinterpret_cast<const uint4 *>(row + b_col + k) : make_uint4(0u, 0u, 0u, 0u);
            pc[j] = in ? *reinterpret_cast<const uint4 *>(row + c_col + k) : make_uint4(0u, 0u, 0u, 0u);
        }
        const int tt = tid / 4, p = 4 * (tid % 4);
        px = (tt < m && p0 + p < dv) ? *reinterpret_cast<const uint2 *>(xbc + (size_t)(q0 + t0 + tt) * a.xbc_stride + x_col + p)
                                     : make_uint2(0u, 0u);
        pd = lane < m ? ssm_ld(a.y, a.y_dtype, (size_t)(q0 + t0 + lane) * a.y_stride + a.dt_off + head) : 0.f;
    };
    fetch(0, min(SSM_CHUNK, len));
    int buf = 0;
    for (int t0 = 0; t0 < len; t0 += SSM_CHUNK, buf ^= 1) {
        const int m = min(SSM_CHUNK, len - t0);
        // lane = token: its step size, the sum of the logarithms (base 2) up to it, its weight in the new state
        const float dt = lane < m ? ssm_softplus(pd + bias) : 0.f;
        float cum = -rate * dt;
#pragma unroll
        for (int o = 1; o < SSM_CHUNK; o <<= 1) {
            const float up = __shfl_up(cum, o, KVA_WAVE);
            if (lane >= o) cum += up;
        }
        const float total = __shfl(cum, SSM_CHUNK - 1, KVA_WAVE);
        const float into = dt * __builtin_amdgcn_exp2f(total - cum);
        const float xw = __shfl(into, 16 * w + lane / 4, KVA_WAVE);      // of the token whose x this thread stages
        __syncthreads();                                                  // whoever still reads the chunk before is done
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + 256 * j, at = (i / (NP / 8)) * ST + 8 * (i % (NP / 8));
            *reinterpret_cast<uint4 *>(&L.b[at]) = pb[j];
            *reinterpret_cast<uint4 *>(&L.c[at]) = pc[j];
        }
        {
            const int at = (tid / 4) * SSM_XS + 4 * (tid % 4);
            *reinterpret_cast<uint2 *>(&L.x[at]) = px;
            const float f[4] = {__uint_as_float(px.x << 16), __uint_as_float(px.x & 0xffff0000u), __uint_as_float(px.y << 16),
                                __uint_as_float(px.y & 0xffff0000u)};
            Frag4 hi, lo;
#pragma unroll
            for (int q = 0; q < 4; ++q) ssm_split(f[q] * xw, hi.h[q], lo.h[q]);
            *reinterpret_cast<uint2 *>(&L.wx[0][at]) = hi.u2;
            *reinterpret_cast<uint2 *>(&L.wx[1][at]) = lo.u2;
        }
        if (w == 0) {
            L.cum[lane] = cum;
            L.dt[lane] = dt;
        }
        __syncthreads();
        if (t0 + SSM_CHUNK < len) fetch(t0 + SSM_CHUNK, min(SSM_CHUNK, len - t0 - SSM_CHUNK));
        const int t = 16 * w + r;
        const float cum_t = L.cum[t];
        Frag8 cf[NK];
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) cf[ks].u4 = *reinterpret_cast<const uint4 *>(&L.c[t * ST + 32 * ks + 8 * g]);
        // (3) what the state in front of the chunk says
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int part = 0; part < 2; ++part)
#pragma unroll
            for (int ks = 0; ks < NK; ++ks) {
                Frag8 sf;
                sf.u4 = *reinterpret_cast<const uint4 *>(&L.s[buf][part][r * ST + 32 * ks + 8 * g]);
                y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sf.v, cf[ks].v, y, 0, 0, 0);
            }
        const float from_start = __builtin_amdgcn_exp2f(cum_t);
#pragma unroll
        for (int q = 0; q < 4; ++q) y[q] *= from_start;
        // (1), (2): pairs of tiles of 16 earlier tokens
        const int lane_row = (4 * g + r / 4), lane_col = 4 * (r % 4);
        for (int u = 0; u <= w / 2; ++u) {
            Frag8 hi, lo;
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const int st = 2 * u + h;
                f32x4 gt = {0.f, 0.f, 0.f, 0.f};
                if (st <= w) {
#pragma unroll
                    for (int ks = 0; ks < NK; ++ks) {
                        Frag8 bf;
                        bf.u4 = *reinterpret_cast<const uint4 *>(&L.b[(16 * st + r) * ST + 32 * ks + 8 * g]);
                        gt = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf.v, cf[ks].v, gt, 0, 0, 0);
                    }
                }
                const float4 cs = *reinterpret_cast<const float4 *>(&L.cum[16 * st + 4 * g]);
                const float4 ds = *reinterpret_cast<const float4 *>(&L.dt[16 * st + 4 * g]);
                const float cum_s[4] = {cs.x, cs.y, cs.z, cs.w}, dt_s[4] = {ds.x, ds.y, ds.z, ds.w};
#pragma unroll
                for (int q = 0; q < 4; ++q) {
                    const bool seen = 16 * st + 4 * g + q <= t;
                    const float wgt = seen ? gt[q] * (__builtin_amdgcn_exp2f(cum_t - cum_s[q]) * dt_s[q]) : 0.f;
                    ssm_split(wgt, hi.h[4 * h + q], lo.h[4 * h + q]);
                }
            }
            const Frag8 xf = ssm_transposed(&L.x[(32 * u + lane_row) * SSM_XS + lane_col], SSM_XS);
            y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf.v, hi.v, y, 0, 0, 0);
            y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf.v, lo.v, y, 0, 0, 0);
        }
        if (t < m && p_on) {
            const uint2 xv = *reinterpret_cast<const uint2 *>(&L.x[t * SSM_XS + 4 * g]);
            *reinterpret_cast<float4 *>(a.out + (size_t)(q0 + t0 + t) * a.heads * dv + x_col + 4 * g) =
                make_float4(y[0] + skip * __uint_as_float(xv.x << 16), y[1] + skip * __uint_as_float(xv.x & 0xffff0000u),
                            y[2] + skip * __uint_as_float(xv.y << 16), y[3] + skip * __uint_as_float(xv.y & 0xffff0000u));
        }
        // (4) the state behind the chunk
        const float keep = __builtin_amdgcn_exp2f(total);
        Frag8 wx[2][2];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int part = 0; part < 2; ++part)
                wx[u][part] = ssm_transposed(&L.wx[part][(32 * u + lane_row) * SSM_XS + lane_col], SSM_XS);
#pragma unroll
        for (int k = 0; k < TILES; ++k) {
            const int i0 = 16 * (w + 4 * k);
            if (i0 >= NP) continue;
#pragma unroll
            for (int q = 0; q < 4; ++q) S[k][q] *= keep;
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const Frag8 bf = ssm_transposed(&L.b[(32 * u + lane_row) * ST + i0 + lane_col], ST);
                S[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wx[u][0].v, bf.v, S[k], 0, 0, 0);
                S[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wx[u][1].v, bf.v, S[k], 0, 0, 0);
            }
        }
        leave_state(buf ^ 1);
    }
#pragma unroll
    for (int k = 0; k < TILES; ++k) {
        const int i = 16 * (w + 4 * k) + r;
        if (p_on && i < n) *reinterpret_cast<float4 *>(Sg + (size_t)i * dv) = make_float4(S[k][0], S[k][1], S[k][2], S[k][3]);
    }
}

template <int NK>
static int ssm_chunk_launch(const SsmArgs &a, int entries, hipStream_t stream) {
    const int lds = (int)sizeof(SsmChunkLds<NK>);
    if (lds > 64 * 1024)
        hipFuncSetAttribute(reinterpret_cast<const void *>(state_space_chunk_kernel<NK>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    hipLaunchKernelGGL(state_space_chunk_kernel<NK>, dim3(a.heads * ((a.vdim + 15) / 16), entries), dim3(256), lds, stream, a);
    KVA_CHECK_LAUNCH("state_space_chunk");
    return KVA_OK;
}

enum SsmKernel { SSM_SCAN = 0, SSM_TOKEN = 1, SSM_CHUNKS = 2 };

// whether a kernel takes these sizes (rows of x, B and C as the convolution leaves them, 16-byte aligned)
extern "C" int kva_state_space_supported(int kernel, int heads, int groups, int n, int vdim, int xbc_dtype) {
    if (kernel == SSM_SCAN) return n <= SSM_MAX_STATE;
    if (kernel == SSM_TOKEN) return vdim % 4 == 0;
    return kernel == SSM_CHUNKS && xbc_dtype == KVA_BF16 && n % 8 == 0 && n <= 256 && vdim % 4 == 0 && heads * vdim % 8 == 0;
}

extern "C" int kva_state_space(int kernel, int len_lo, int len_hi, float *out, float *state, long long seat_stride,
                               int state_off, const void *xbc, int xbc_dtype, int xbc_stride, const void *y, int y_dtype,
                               int y_stride, int dt_off, const float *a_log, const float *dt_bias, const float *d_skip,
                               const int *entry_q_start, const int *entry_seat, int entries, int heads, int groups, int n,
                               int vdim, hipStream_t stream) {
    KVA_REQUIRE(out && state && xbc && y && a_log && dt_bias && d_skip && entry_q_start && entry_seat,
                "state_space: missing operand");
    KVA_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && vdim > 0, "state_space: %d heads in %d groups", heads, groups);
    KVA_REQUIRE(n > 0 && n <= SSM_MAX_STATE, "state_space: state size %d must lie in 1..%d", n, SSM_MAX_STATE);
    KVA_REQUIRE(xbc_stride >= heads * vdim + 2 * groups * n && dt_off >= 0 && y_stride >= dt_off + heads,
                "state_space: the rows are too short for what they hold");
    KVA_REQUIRE(entries >= 0 && entries <= 65535 && len_lo >= 1, "state_space: %d entries, of %d tokens at least", entries, len_lo);
    KVA_REQUIRE(kva_state_space_supported(kernel, heads, groups, n, vdim, xbc_dtype), "state_space: kernel %d does not take a "
                "state of %d and %d heads of %d", kernel, n, heads, vdim);
    KVA_REQUIRE(kernel != SSM_TOKEN || (len_lo == 1 && len_hi == 1), "state_space: the kernel of a single token takes entries of one");
    const bool rows16 = seat_stride % 4 == 0 && state_off % 4 == 0 && ((reinterpret_cast<uintptr_t>(state) | reinterpret_cast<uintptr_t>(out)) & 15) == 0;
    KVA_REQUIRE(kernel == SSM_SCAN || rows16, "state_space: states and results must start at multiples of 16 bytes");
    KVA_REQUIRE(kernel != SSM_CHUNKS || (xbc_stride % 8 == 0 && (reinterpret_cast<uintptr_t>(xbc) & 15) == 0),
                "state_space: rows must start at multiples of 16 bytes");
    if (entries == 0) return KVA_OK;
    const SsmArgs a{out, state, (size_t)seat_stride, state_off, entry_q_start, entry_seat, xbc, xbc_dtype, xbc_stride, y,
                    y_dtype, y_stride, dt_off, a_log, dt_bias, d_skip, heads, groups, n, vdim, len_lo, len_hi};
    if (kernel == SSM_CHUNKS) {
        if (n <= 32) return ssm_chunk_launch<1>(a, entries, stream);
        if (n <= 64) return ssm_chunk_launch<2>(a, entries, stream);
        if (n <= 128) return ssm_chunk_launch<4>(a, entries, stream);
        return ssm_chunk_launch<8>(a, entries, stream);
    }
    if (kernel == SSM_TOKEN) {
        hipLaunchKernelGGL(state_space_token_kernel, dim3(heads * ((vdim + 63) / 64), entries), dim3(256), 0, stream, a);
        KVA_CHECK_LAUNCH("state_space_token");
        return KVA_OK;
    }
    const dim3 grid(heads * ((vdim + SSM_BLOCK_COLS - 1) / SSM_BLOCK_COLS), entries);
    if (n <= 64) hipLaunchKernelGGL((state_space_scan_kernel<4, 32>), grid, dim3(SSM_THREADS), 0, stream, a);
    else if (n <= 128) hipLaunchKernelGGL((state_space_scan_kernel<8, 32>), grid, dim3(SSM_THREADS), 0, stream, a);
    else if (n <= 256) hipLaunchKernelGGL((state_space_scan_kernel<16, 16>), grid, dim3(SSM_THREADS), 0, stream, a);
    else hipLaunchKernelGGL((state_space_scan_kernel<32, 8>), grid, dim3(SSM_THREADS), 0, stream, a);
    KVA_CHECK_LAUNCH("state_space_scan");
    return KVA_OK;
}
