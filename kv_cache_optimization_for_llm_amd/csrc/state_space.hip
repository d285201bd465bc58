// The recurrence of a state-space mixer whose decay is one number per head and token:
//
//     S_t = exp(-rate_h dt_t) S_(t-1) + dt_t B_t x_t^T,    y_t = S_t^T C_t + D_h x_t,
//
// S [state, value] per head, dt_t = softplus(y[t, dt_off + h] + dt_bias_h), rate_h = exp(A_log_h).  B and C
// belong to groups of heads.  S is fp32, starts at zero and lives in the seat's state row between steps.
//
// Kernels for three kinds of entries; each takes the entries whose number of tokens lies in a range the caller names.
//
//  * state_space_scan_kernel walks the tokens.  Value columns of S are independent of each other: a workgroup
//    of four wavefronts takes 16 of a head's, a wavefront 4, the 16 lanes of a row of the wavefront share a
//    column and keep its part of S in registers (rows 4 (16 j + r) .. + 3 for lane r).  A chunk of tokens - B,
//    C, the 16 columns of x, the two numbers of every token - is staged in LDS for the four wavefronts while
//    the one before is walked.  The order of every sum depends on the sizes alone.
//  * state_space_token_kernel is a single token: S passes through registers once, 16 bytes a lane.
//  * state_space_states_kernel and state_space_outputs_kernel (bf16 rows) take chunks of 64 tokens on the matrix cores.  With c_t the sum of
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
// Two kernels.  state_space_states_kernel walks an entry's chunks and does nothing but hand S on: for every chunk it
// leaves the state in front of it in a workspace.  state_space_outputs_kernel takes the chunks side by side.
//
// Lane (r = lane % 16, g = lane / 16) of a product's result holds rows 4 g .. + 3 of column r.  S [state, value] is kept
// so - a value column a lane, NK = state size / 32 (rounded up, the rest is zero) pairs of tiles of 16 state rows -
// and a pair of tiles is then, as it lies in the registers, an operand whose k index is the permutation (j / 4) 16 +
// 4 g + j % 4 of 32 state rows; C and B are read in the same permutation (two pieces of 4 elements).
#define SSM_CHUNK 64

typedef __attribute__((address_space(3))) s16x4 ssm_lds_s16x4;

// row stride in LDS, in elements, of rows of n (a multiple of 16): an odd multiple of 4 words whose first three
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

// softplus as a chain of few instructions: log(1 + e) with e = exp(-|z|) by the hardware's logarithm, or where that
// would lose digits by the series (the sixth term is below 2e-8 of the sum there)
__device__ __forceinline__ float ssm_softplus_short(float z) {
    const float e = __builtin_amdgcn_exp2f(-fabsf(z) * 1.44269504088896340736f);
    const float series = e * (1.f - e * (0.5f - e * (1.f / 3.f - e * (0.25f - e * 0.2f))));
    return fmaxf(z, 0.f) + (e < 0.04f ? series : 0.69314718055994530942f * __builtin_amdgcn_logf(1.f + e));
}

// two numbers as the sums of two bf16 numbers each
__device__ __forceinline__ void ssm_split2(float a, float b, b16x2 &hi, b16x2 &lo) {
    union { b16x2 p; uint32_t u; } h;
    h.p = pack_bf16(a, b);
    hi = h.p;
    lo = pack_bf16(a - __uint_as_float(h.u << 16), b - __uint_as_float(h.u & 0xffff0000u));
}

// inclusive sum over the wavefront's lanes: rotations' kin inside rows of 16 lanes, then the rows' totals
template <int SHIFT>
__device__ __forceinline__ float ssm_shifted(float v) {                  // lane - SHIFT of the row of 16, 0 in front of it
    return __uint_as_float(__builtin_amdgcn_update_dpp(0u, __float_as_uint(v), 0x110 | SHIFT, 0xf, 0xf, false));
}
__device__ __forceinline__ float ssm_lane(float v, int lane) { return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(v), lane)); }
__device__ __forceinline__ float ssm_prefix(float v) {
    v += ssm_shifted<1>(v);
    v += ssm_shifted<2>(v);
    v += ssm_shifted<4>(v);
    v += ssm_shifted<8>(v);
    const float r0 = ssm_lane(v, 15), r1 = ssm_lane(v, 31), r2 = ssm_lane(v, 47);
    const int row = (threadIdx.x % KVA_WAVE) / 16;
    return v + (row > 0 ? r0 : 0.f) + (row > 1 ? r1 : 0.f) + (row > 2 ? r2 : 0.f);
}

// a chunk's place in the workspace: entries' chunks lie one behind the other with room for a part-filled one each
__device__ __forceinline__ size_t ssm_chunk_at(int q0, int e, int chunk) { return (size_t)q0 / SSM_CHUNK + e + chunk; }

struct SsmChunks {
    SsmArgs a;
    uint4 *work;            // [chunk][head][tile of 16 value columns][NK][high, low part][lane]
    int max_chunks;         // chunks of the longest entry
};

// A workgroup takes 16 value columns of a head, wavefront w the state rows of the pairs of tiles w, w + 4, ..:
//     S[n, p] = e^(c_64) S + sum_s B^T[n, s] (e^(c_64 - c_s) dt_s x[s, p]),
// both operands by transposing loads from LDS, the second one as the sum of two bf16 numbers.  Two buffers in LDS: a
// barrier a chunk; the rows of the two chunks behind this one are on their way while it is worked on.
template <int NK>
struct SsmStatesLds {
    static constexpr int ST = ssm_stride(32 * NK), XS = ssm_stride(16);
    bf16_t b[2][SSM_CHUNK * ST], wx[2][2][SSM_CHUNK * XS];
};

template <int NK>
__global__ void __launch_bounds__(256)
state_space_states_kernel(SsmChunks k) {
    using Lds = SsmStatesLds<NK>;
    constexpr int NP = 32 * NK, ST = Lds::ST, XS = Lds::XS, PAIRS = (NK + 3) / 4;
    constexpr int PIECES = SSM_CHUNK * NP / 8 / 256;                     // 16-byte pieces of B a thread
    constexpr float LOG2E = 1.44269504088896340736f;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
    Lds &L = *reinterpret_cast<Lds *>(lds_raw);
    const SsmArgs &a = k.a;
    const int tid = threadIdx.x, lane = tid % KVA_WAVE, w = tid / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int slices = (a.vdim + 15) / 16, id = die_order(blockIdx.x, gridDim.x);
    const int head = id / slices, slice = id % slices, p0 = 16 * slice, e = blockIdx.y;
    const int q0 = a.entry_q_start[e], len = a.entry_q_start[e + 1] - q0;
    if (len < a.len_lo || len > a.len_hi) return;
    const int n = a.n, dv = a.vdim, grp = head / (a.heads / a.groups);
    const bf16_t *xbc = reinterpret_cast<const bf16_t *>(a.xbc);
    const int b_col = a.heads * dv + grp * n;
    const float rate = expf(a.a_log[head]) * LOG2E, bias = a.dt_bias[head];
    float *Sg = a.state + (size_t)a.entry_seat[e] * a.seat_stride + a.state_off + (size_t)head * n * dv + p0 + r;
    const bool p_on = p0 + r < dv;
    f32x4 S[PAIRS][2];
#pragma unroll
    for (int j = 0; j < PAIRS; ++j)
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int i = 32 * (w + 4 * j) + 16 * h + 4 * g + q;
                S[j][h][q] = p_on && i < n ? Sg[(size_t)i * dv] : 0.f;
            }
    struct Ahead {                      // a chunk's rows on their way
        kva_u32x4 b[PIECES];
        kva_u32x2 x;
        uint16_t d;
    } ahead0, ahead1;
    // (no branch around a load, nothing formed from it here: tokens past the chunk's last one repeat that one, with
    // weight zero; columns past the last one repeat others, into rows and columns of S that nobody stores)
    auto fetch = [&](Ahead &f, int t0) {
        const int last = min(SSM_CHUNK, len - t0) - 1;
        const bf16_t *first = xbc + (size_t)(q0 + t0) * a.xbc_stride;
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + 256 * j, tt = min(i / (NP / 8), last), c = min(8 * (i % (NP / 8)), n - 8);      // (n is a multiple of 8)
            f.b[j] = *reinterpret_cast<const kva_u32x4 *>(first + (size_t)tt * a.xbc_stride + b_col + c);
        }
        // x: lane = token, wavefront w the columns 4 w .. + 3 (dv is a multiple of 4)
        const int tt = min(lane, last);
        f.x = *reinterpret_cast<const kva_u32x2 *>(first + (size_t)tt * a.xbc_stride + head * dv + min(p0 + 4 * w, dv - 4));
        f.d = reinterpret_cast<const uint16_t *>(a.y)[(size_t)(q0 + t0 + tt) * a.y_stride + a.dt_off + head];
    };
    const int lane_row = 4 * g + r / 4, lane_col = 4 * (r % 4);
    auto turn = [&](Ahead &f, int t0, int buf) {
        const int m = min(SSM_CHUNK, len - t0);
        // the state in front of the chunk, as the operand that the outputs' kernel reads
        uint4 *work = k.work + (((ssm_chunk_at(q0, e, t0 / SSM_CHUNK) * a.heads + head) * slices + slice) * NK * 2) * KVA_WAVE + lane;
#pragma unroll
        for (int j = 0; j < PAIRS; ++j) {
            const int ks = w + 4 * j;
            if (ks >= NK) continue;
            Frag8 hi, lo;
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                ssm_split2(S[j][h][0], S[j][h][1], hi.p2[2 * h], lo.p2[2 * h]);
                ssm_split2(S[j][h][2], S[j][h][3], hi.p2[2 * h + 1], lo.p2[2 * h + 1]);
            }
            work[(2 * ks) * KVA_WAVE] = hi.u4;
            work[(2 * ks + 1) * KVA_WAVE] = lo.u4;
        }
        // lane = token: its step size, the sum of the logarithms (base 2) up to it, its weight in the new state
        const float dt = lane < m ? ssm_softplus_short(bf16_bits_to_float(f.d) + bias) : 0.f;
        const float cum = ssm_prefix(-rate * dt), total = ssm_lane(cum, SSM_CHUNK - 1);
        const float into = dt * __builtin_amdgcn_exp2f(total - cum);
#pragma unroll
        for (int j = 0; j < PIECES; ++j) {
            const int i = tid + 256 * j;
            *reinterpret_cast<kva_u32x4 *>(&L.b[buf][(i / (NP / 8)) * ST + 8 * (i % (NP / 8))]) = f.b[j];
        }
        union { b16x2 p[2]; uint2 u; } hi, lo;
        ssm_split2(__uint_as_float(f.x.x << 16) * into, __uint_as_float(f.x.x & 0xffff0000u) * into, hi.p[0], lo.p[0]);
        ssm_split2(__uint_as_float(f.x.y << 16) * into, __uint_as_float(f.x.y & 0xffff0000u) * into, hi.p[1], lo.p[1]);
        *reinterpret_cast<uint2 *>(&L.wx[buf][0][lane * XS + 4 * w]) = hi.u;
        *reinterpret_cast<uint2 *>(&L.wx[buf][1][lane * XS + 4 * w]) = lo.u;
        if (t0 + 2 * SSM_CHUNK < len) fetch(f, t0 + 2 * SSM_CHUNK);
        __syncthreads();            // (a buffer was read last two turns ago: every wavefront has passed the barrier between)
        const float keep = __builtin_amdgcn_exp2f(total);
        Frag8 wx[2][2];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int part = 0; part < 2; ++part)
                wx[u][part] = ssm_transposed(&L.wx[buf][part][(32 * u + lane_row) * XS + lane_col], XS);
#pragma unroll
        for (int j = 0; j < PAIRS; ++j) {
            if (w + 4 * j >= NK) continue;
            Frag8 bf[2][2];
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int u = 0; u < 2; ++u)
                    bf[h][u] = ssm_transposed(&L.b[buf][(32 * u + lane_row) * ST + 32 * (w + 4 * j) + 16 * h + lane_col], ST);
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int q = 0; q < 4; ++q) S[j][h][q] *= keep;
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int part = 0; part < 2; ++part)
#pragma unroll
                    for (int h = 0; h < 2; ++h)
                        S[j][h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf[h][u].v, wx[u][part].v, S[j][h], 0, 0, 0);
        }
    };
    fetch(ahead0, 0);
    if (SSM_CHUNK < len) fetch(ahead1, SSM_CHUNK);
    for (int t0 = 0; t0 < len; t0 += 2 * SSM_CHUNK) {
        turn(ahead0, t0, 0);
        if (t0 + SSM_CHUNK < len) turn(ahead1, t0 + SSM_CHUNK, 1);
    }
#pragma unroll
    for (int j = 0; j < PAIRS; ++j)
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int i = 32 * (w + 4 * j) + 16 * h + 4 * g + q;
                if (p_on && i < n) Sg[(size_t)i * dv] = S[j][h][q];
            }
}

// A workgroup takes a chunk, a head and up to 64 of its value columns.  Everything is computed transposed, wavefront w
// the tokens t = 16 w .. + 15 as columns: G^T[s, t] = B_s . C_t for the tiles s <= t (B in LDS, C from memory); the
// weights e^(c_t - c_s) dt_s G, in registers the second operand of y^T[p, t] = sum_s x^T[p, s] W^T[s, t] (x in LDS, by
// transposing loads); and per tile of 16 value columns e^(c_t) S_0^T C + that + D x.
template <int NK>
struct SsmOutputsLds {
    static constexpr int ST = ssm_stride(32 * NK), XS = ssm_stride(64);
    bf16_t b[SSM_CHUNK * ST], x[SSM_CHUNK * XS];
    float cum[SSM_CHUNK], dt[SSM_CHUNK];
};

template <int NK>
__global__ void __launch_bounds__(256)
state_space_outputs_kernel(SsmChunks k) {
    using Lds = SsmOutputsLds<NK>;
    constexpr int NP = 32 * NK, ST = Lds::ST, XS = Lds::XS, PIECES = SSM_CHUNK * NP / 8 / 256;
    constexpr float LOG2E = 1.44269504088896340736f;
    __shared__ __attribute__((aligned(16))) Lds L;
    const SsmArgs &a = k.a;
    const int tid = threadIdx.x, lane = tid % KVA_WAVE, w = tid / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int slices = (a.vdim + 15) / 16, blocks = (a.vdim + 63) / 64, per_chunk = a.heads * blocks;
    const int id = die_order(blockIdx.x, gridDim.x), chunk = id / per_chunk, head = id % per_chunk / blocks, block = id % blocks;
    const int e = blockIdx.y;
    const int q0 = a.entry_q_start[e], len = a.entry_q_start[e + 1] - q0, t0 = chunk * SSM_CHUNK;
    if (len < a.len_lo || len > a.len_hi || t0 >= len) return;
    const int n = a.n, dv = a.vdim, grp = head / (a.heads / a.groups), m = min(SSM_CHUNK, len - t0), p0 = 64 * block;
    const bf16_t *rows = reinterpret_cast<const bf16_t *>(a.xbc) + (size_t)(q0 + t0) * a.xbc_stride;
    const int x_col = head * dv + p0, b_col = a.heads * dv + grp * n, c_col = b_col + a.groups * n;
    const float rate = expf(a.a_log[head]) * LOG2E, skip = a.d_skip[head];
    // (no branch around a load: tokens past the chunk's last one repeat that one - nobody sees them or stores what they
    // see - and columns of B and x past the last one repeat others, which meet zeros of C or are not stored)
    const uint16_t pd = reinterpret_cast<const uint16_t *>(a.y)[(size_t)(q0 + t0 + min(lane, m - 1)) * a.y_stride + a.dt_off + head];
    uint4 pb[PIECES];
#pragma unroll
    for (int j = 0; j < PIECES; ++j) {
        const int i = tid + 256 * j, tt = min(i / (NP / 8), m - 1), c = min(8 * (i % (NP / 8)), n - 8);
        pb[j] = *reinterpret_cast<const uint4 *>(rows + (size_t)tt * a.xbc_stride + b_col + c);
    }
    uint2 px[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int i = tid + 256 * j, tt = min(i / 16, m - 1), p = min(p0 + 4 * (i % 16), dv - 4);
        px[j] = *reinterpret_cast<const uint2 *>(rows + (size_t)tt * a.xbc_stride + head * dv + p);
    }
    const int t = 16 * w + r;
    Frag8 cf[NK];
#pragma unroll
    for (int ks = 0; ks < NK; ++ks)
#pragma unroll
        for (int h = 0; h < 2; ++h)
            cf[ks].u2[h] = *reinterpret_cast<const uint2 *>(rows + (size_t)min(t, m - 1) * a.xbc_stride + c_col +
                                                            min(32 * ks + 16 * h + 4 * g, n - 4));
#pragma unroll
    for (int ks = 0; ks < NK; ++ks)
#pragma unroll
        for (int h = 0; h < 2; ++h)
            if (32 * ks + 16 * h + 4 * g >= n) cf[ks].u2[h] = make_uint2(0u, 0u);
    const float dt = lane < m ? ssm_softplus_short(bf16_bits_to_float(pd) + a.dt_bias[head]) : 0.f;
    const float cum = ssm_prefix(-rate * dt);
#pragma unroll
    for (int j = 0; j < PIECES; ++j) {
        const int i = tid + 256 * j;
        *reinterpret_cast<uint4 *>(&L.b[(i / (NP / 8)) * ST + 8 * (i % (NP / 8))]) = pb[j];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int i = tid + 256 * j;
        *reinterpret_cast<uint2 *>(&L.x[(i / 16) * XS + 4 * (i % 16)]) = px[j];
    }
    if (w == 0) {
        L.cum[lane] = cum;
        L.dt[lane] = dt;
    }
    __syncthreads();
    const float cum_t = L.cum[t];
    Frag8 hi[2], lo[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        hi[u].u4 = lo[u].u4 = make_uint4(0u, 0u, 0u, 0u);
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const int st = 2 * u + h;
            if (st > w) continue;                                           // (the whole wavefront: later tokens)
            f32x4 gt = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < NK; ++ks) {
                Frag8 bf;
                const bf16_t *brow = &L.b[(16 * st + r) * ST + 32 * ks + 4 * g];
                bf.u2[0] = *reinterpret_cast<const uint2 *>(brow);
                bf.u2[1] = *reinterpret_cast<const uint2 *>(brow + 16);
                gt = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf.v, cf[ks].v, gt, 0, 0, 0);
            }
            const float4 cs = *reinterpret_cast<const float4 *>(&L.cum[16 * st + 4 * g]);
            const float4 ds = *reinterpret_cast<const float4 *>(&L.dt[16 * st + 4 * g]);
            const float cum_s[4] = {cs.x, cs.y, cs.z, cs.w}, dt_s[4] = {ds.x, ds.y, ds.z, ds.w};
            float wgt[4];
#pragma unroll
            for (int q = 0; q < 4; ++q)
                wgt[q] = 16 * st + 4 * g + q <= t ? gt[q] * (__builtin_amdgcn_exp2f(cum_t - cum_s[q]) * dt_s[q]) : 0.f;
            ssm_split2(wgt[0], wgt[1], hi[u].p2[2 * h], lo[u].p2[2 * h]);
            ssm_split2(wgt[2], wgt[3], hi[u].p2[2 * h + 1], lo[u].p2[2 * h + 1]);
        }
    }
    const float from_start = __builtin_amdgcn_exp2f(cum_t);
    const int lane_row = 4 * g + r / 4, lane_col = 4 * (r % 4);
    const uint4 *work = k.work + (((ssm_chunk_at(q0, e, chunk) * a.heads + head) * slices + 4 * block) * NK * 2) * KVA_WAVE + lane;
    float *orow = a.out + (size_t)(q0 + t0 + t) * a.heads * dv + x_col + 4 * g;
#pragma unroll
    for (int pt = 0; pt < 4; ++pt) {
        if (p0 + 16 * pt >= dv) break;
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < NK; ++ks)
#pragma unroll
            for (int part = 0; part < 2; ++part) {
                Frag8 sf;
                sf.u4 = work[((pt * NK + ks) * 2 + part) * KVA_WAVE];
                y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sf.v, cf[ks].v, y, 0, 0, 0);
            }
#pragma unroll
        for (int q = 0; q < 4; ++q) y[q] *= from_start;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            if (2 * u > w) continue;
            const Frag8 xf = ssm_transposed(&L.x[(32 * u + lane_row) * XS + 16 * pt + lane_col], XS);
            y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf.v, hi[u].v, y, 0, 0, 0);
            y = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf.v, lo[u].v, y, 0, 0, 0);
        }
        if (t < m && p0 + 16 * pt + 4 * g < dv) {                           // (dv is a multiple of 4)
            const uint2 xv = *reinterpret_cast<const uint2 *>(&L.x[t * XS + 16 * pt + 4 * g]);
            *reinterpret_cast<float4 *>(orow + 16 * pt) =
                make_float4(y[0] + skip * __uint_as_float(xv.x << 16), y[1] + skip * __uint_as_float(xv.x & 0xffff0000u),
                            y[2] + skip * __uint_as_float(xv.y << 16), y[3] + skip * __uint_as_float(xv.y & 0xffff0000u));
        }
    }
}

static int ssm_pairs(int n) { return n <= 32 ? 1 : n <= 64 ? 2 : n <= 128 ? 4 : 8; }

// bytes of workspace the chunks of a step of so many tokens and entries need
extern "C" long long kva_state_space_workspace(int tokens, int entries, int heads, int n, int vdim) {
    return ((long long)tokens / SSM_CHUNK + entries + 1) * heads * ((vdim + 15) / 16) * ssm_pairs(n) * 2 * KVA_WAVE * 16;
}

template <int NK>
static int ssm_chunk_launch(const SsmChunks &k, int entries, hipStream_t stream) {
    const SsmArgs &a = k.a;
    const int lds = (int)sizeof(SsmStatesLds<NK>);
    if (lds > 64 * 1024)
        hipFuncSetAttribute(reinterpret_cast<const void *>(state_space_states_kernel<NK>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    hipLaunchKernelGGL(state_space_states_kernel<NK>, dim3(a.heads * ((a.vdim + 15) / 16), entries), dim3(256), lds, stream, k);
    KVA_CHECK_LAUNCH("state_space_states");
    hipLaunchKernelGGL(state_space_outputs_kernel<NK>, dim3((unsigned)((long long)k.max_chunks * a.heads * ((a.vdim + 63) / 64)), entries),
                       dim3(256), 0, stream, k);
    KVA_CHECK_LAUNCH("state_space_outputs");
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
                               int vdim, void *work, long long work_bytes, int tokens, int max_len, hipStream_t stream) {
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
    KVA_REQUIRE(kernel != SSM_CHUNKS || (y_dtype == KVA_BF16 && xbc_stride % 8 == 0 && (reinterpret_cast<uintptr_t>(xbc) & 15) == 0),
                "state_space: bf16 rows that start at multiples of 16 bytes");
    if (entries == 0) return KVA_OK;
    const SsmArgs a{out, state, (size_t)seat_stride, state_off, entry_q_start, entry_seat, xbc, xbc_dtype, xbc_stride, y,
                    y_dtype, y_stride, dt_off, a_log, dt_bias, d_skip, heads, groups, n, vdim, len_lo, len_hi};
    if (kernel == SSM_CHUNKS) {
        KVA_REQUIRE(work && (reinterpret_cast<uintptr_t>(work) & 15) == 0 && tokens > 0 && max_len > 0 && max_len <= tokens &&
                        work_bytes >= kva_state_space_workspace(tokens, entries, heads, n, vdim),
                    "state_space: %lld bytes of workspace are too few for %d tokens in %d entries", work_bytes, tokens, entries);
        const SsmChunks k{a, (uint4 *)work, (max_len + SSM_CHUNK - 1) / SSM_CHUNK};
        KVA_REQUIRE((long long)k.max_chunks * heads * ((vdim + 63) / 64) < (1LL << 31), "state_space: too many chunks for one launch");
        switch (ssm_pairs(n)) {
        case 1: return ssm_chunk_launch<1>(k, entries, stream);
        case 2: return ssm_chunk_launch<2>(k, entries, stream);
        case 4: return ssm_chunk_launch<4>(k, entries, stream);
        default: return ssm_chunk_launch<8>(k, entries, stream);
        }
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
