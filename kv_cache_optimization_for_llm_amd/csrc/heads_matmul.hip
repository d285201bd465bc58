// One small matrix product per head: out[t, h, :] = W[h] x[t, h, :] for W [heads, N, K].
//
// It serves projections that differ from head to head (a low-rank key/value entry expanded per
// head, or the same expansion moved to the query side).  x and out are addressed with a row
// stride and a head stride each, so both may be column ranges of wider buffers.  Operands are
// fp32 or bf16; sums are fp32 with k ascending into one accumulator per output, so a row's result
// does not depend on the other rows of the launch.
//
// Two things may ride on the launch.  A sigmoid gate in the epilogue, one number a head or one an output
// element.  And a rotation (HeadsRotate): heads whose product covers only their first elements (queries with
// a rotated part behind the unrotated one) have the rest rotated into place by workgroups of their own.
#include "common.h"
#include <math.h>

// out *= sigmoid(p[row * row_stride + head * head_stride (+ n)])
struct HeadsGate {
    const void *p;
    int row, head, per_element;
};

template <typename T>
__device__ inline float heads_gate(const HeadsGate &g, size_t m, int h, int n) {
    const T *p = reinterpret_cast<const T *>(g.p);
    return 1.0f / (1.0f + expf(-to_float(p[m * g.row + (size_t)h * g.head + (g.per_element ? n : 0)])));
}

// dst[row, head, 0..rot) = the rotation of src[row, head, 0..rot) by the row's position: pair i is (2 i, 2 i + 1)
// (`interleaved`) or (i, i + rot / 2); cos and sin are fp32 [positions, rot / 2]
struct HeadsRotate {
    const void *src;
    void *dst;
    const float *cos_table, *sin_table;
    const int *positions;
    int src_row, src_head, dst_row, dst_head, rot, interleaved;
};

template <typename T>
__device__ inline void heads_rotate(const HeadsRotate &ro, int h, int row0, int row1) {
    const int half = ro.rot / 2;
    for (int w = threadIdx.x; w < (row1 - row0) * half; w += blockDim.x) {
        const int m = row0 + w / half, i = w % half;
        const size_t at = (size_t)ro.positions[m] * half + i;
        const float co = ro.cos_table[at], si = ro.sin_table[at];
        const int a = ro.interleaved ? 2 * i : i, b = ro.interleaved ? 2 * i + 1 : i + half;
        const T *src = reinterpret_cast<const T *>(ro.src) + (size_t)m * ro.src_row + (size_t)h * ro.src_head;
        T *dst = reinterpret_cast<T *>(ro.dst) + (size_t)m * ro.dst_row + (size_t)h * ro.dst_head;
        const float u = to_float(src[a]), v = to_float(src[b]);
        dst[a] = from_float<T>(u * co - v * si);
        dst[b] = from_float<T>(v * co + u * si);
    }
}

#define HM_BM 64
#define HM_BN 64
#define HM_BK 16

template <typename T>
__global__ void __launch_bounds__(256)
heads_matmul_kernel(T *__restrict__ out, int o_row, int o_head, const T *__restrict__ x, int x_row, int x_head,
                    const T *__restrict__ w, int M, int N, int K, HeadsGate gate, HeadsRotate ro) {
    if (ro.rot > 0 && blockIdx.x == gridDim.x - 1) {            // the last column of workgroups rotates
        heads_rotate<T>(ro, blockIdx.z, blockIdx.y * HM_BM, min(M, (int)(blockIdx.y + 1) * HM_BM));
        return;
    }
    __shared__ float Xs[HM_BK][HM_BM + 4];
    __shared__ float Ws[HM_BK][HM_BN + 4];
    const int h = blockIdx.z;
    const int tid = threadIdx.x, tx = tid % 16, ty = tid / 16;
    const int m0 = blockIdx.y * HM_BM, n0 = blockIdx.x * HM_BN;
    const int lrow = tid / 4, lk = (tid % 4) * 4;
    const T *xh = x + (size_t)h * x_head, *wh = w + (size_t)h * N * K;
    float acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = 0.f;
    for (int k0 = 0; k0 < K; k0 += HM_BK) {
        float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
        const int am = m0 + lrow, wn = n0 + lrow, kk = k0 + lk;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            if (am < M && kk + e < K) a[e] = to_float(xh[(size_t)am * x_row + kk + e]);
            if (wn < N && kk + e < K) b[e] = to_float(wh[(size_t)wn * K + kk + e]);
        }
        __syncthreads();
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            Xs[lk + e][lrow] = a[e];
            Ws[lk + e][lrow] = b[e];
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < HM_BK; ++k) {
            float av[4], wv[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) av[i] = Xs[k][ty * 4 + i];
#pragma unroll
            for (int j = 0; j < 4; ++j) wv[j] = Ws[k][tx * 4 + j];
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(av[i], wv[j], acc[i][j]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int m = m0 + ty * 4 + i;
        if (m >= M) continue;
        const float gmul = gate.p && !gate.per_element ? heads_gate<T>(gate, m, h, 0) : 1.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tx * 4 + j;
            if (n >= N) continue;
            const float g = gate.per_element ? heads_gate<T>(gate, m, h, n) : gmul;
            out[(size_t)m * o_row + (size_t)h * o_head + n] = from_float<T>(acc[i][j] * g);
        }
    }
}

static int heads_options(HeadsGate &gate, HeadsRotate &ro, const void *g, int g_row, int g_head, int g_per_element,
                         const void *r_src, int r_src_row, int r_src_head, void *r_dst, int r_dst_row, int r_dst_head,
                         const float *cos_table, const float *sin_table, const int *positions, int rot, int interleaved,
                         int heads, int N) {
    KVA_REQUIRE(!g || (g_head >= (g_per_element ? N : 1) && g_row >= (heads - 1) * g_head + (g_per_element ? N : 1)),
                "heads_matmul: the gate's strides do not fit %d heads of %d", heads, N);
    KVA_REQUIRE(rot >= 0 && rot % 2 == 0 && (rot == 0 || (r_src && r_dst && cos_table && sin_table && positions)),
                "heads_matmul: a rotation of %d elements (an even number) needs source, target, tables and positions", rot);
    KVA_REQUIRE(rot == 0 || (r_src_head >= rot && r_dst_head >= rot && r_src_row >= (heads - 1) * r_src_head + rot &&
                             r_dst_row >= (heads - 1) * r_dst_head + rot),
                "heads_matmul: the rotation's strides do not fit %d heads of %d elements", heads, rot);
    gate = HeadsGate{g, g_row, g_head, g ? g_per_element : 0};
    ro = HeadsRotate{r_src, r_dst, cos_table, sin_table, positions, r_src_row, r_src_head, r_dst_row, r_dst_head, rot, interleaved};
    return KVA_OK;
}

#define HEADS_OPTION_ARGS                                                                                              \
    const void *gate_p, int g_row, int g_head, int g_per_element, const void *r_src, int r_src_row, int r_src_head,     \
        void *r_dst, int r_dst_row, int r_dst_head, const float *cos_table, const float *sin_table, const int *positions, \
        int rot, int interleaved
#define HEADS_OPTIONS(gate, ro)                                                                                        \
    HeadsGate gate;                                                                                                    \
    HeadsRotate ro;                                                                                                    \
    if (const int bad = heads_options(gate, ro, gate_p, g_row, g_head, g_per_element, r_src, r_src_row, r_src_head, r_dst, \
                                      r_dst_row, r_dst_head, cos_table, sin_table, positions, rot, interleaved, heads, N)) \
        return bad

extern "C" int kva_heads_matmul(void *out, int o_row, int o_head, const void *x, int x_row, int x_head,
                                const void *w, int rows, int heads, int N, int K, HEADS_OPTION_ARGS, int dtype,
                                hipStream_t stream) {
    KVA_REQUIRE(rows >= 0 && heads > 0 && heads <= 65535 && N > 0 && K > 0, "heads_matmul: bad sizes");
    KVA_REQUIRE(x_head >= K && o_head >= N && x_row >= (heads - 1) * x_head + K && o_row >= (heads - 1) * o_head + N,
                "heads_matmul: strides do not fit %d heads of %d -> %d", heads, K, N);
    HEADS_OPTIONS(gate, ro);
    if (rows == 0) return KVA_OK;
    dim3 grid((N + HM_BN - 1) / HM_BN + (rot > 0 ? 1 : 0), (rows + HM_BM - 1) / HM_BM, heads), block(256);
    KVA_REQUIRE(grid.y <= 65535, "heads_matmul: %d rows are too many for one launch", rows);
    if (dtype == KVA_F32)
        hipLaunchKernelGGL(heads_matmul_kernel<float>, grid, block, 0, stream, (float *)out, o_row, o_head,
                           (const float *)x, x_row, x_head, (const float *)w, rows, N, K, gate, ro);
    else if (dtype == KVA_BF16)
        hipLaunchKernelGGL(heads_matmul_kernel<bf16_t>, grid, block, 0, stream, (bf16_t *)out, o_row, o_head,
                           (const bf16_t *)x, x_row, x_head, (const bf16_t *)w, rows, N, K, gate, ro);
    else KVA_REQUIRE(false, "heads_matmul: unsupported dtype %d", dtype);
    KVA_CHECK_LAUNCH("heads_matmul");
    return KVA_OK;
}

// ---- the same product on the matrix cores (bf16) ------------------------------------------------
//
// A wavefront takes 16 outputs n of one head and walks over tiles of 16 rows t:
// out^T[n, t] = W[h][n, :] . x[t, h, :].  A = 16 rows of W[h] (16 bytes a lane, row-major), kept
// in registers for all the row tiles the wavefront visits; B = x^T: lane (row t, group g) loads 16
// bytes of its row.  K = 32 NKS.  blockIdx: (n tile, head, group of row tiles).
#include "attention_frag.h"

// outputs n .. n + 3 of row t, head h, under the gate
__device__ __forceinline__ void heads_store4(bf16_t *o, const f32x4 &acc, float gmul, const HeadsGate &gate, int t, int h, int n, int N,
                                             bool aligned) {
    float mul[4] = {gmul, gmul, gmul, gmul};
    if (gate.per_element) {
        const bf16_t *gp = reinterpret_cast<const bf16_t *>(gate.p) + (size_t)t * gate.row + (size_t)h * gate.head + n;
        Frag4 gv;
        gv.u2 = make_uint2(0u, 0u);
        if (n + 3 < N && ((reinterpret_cast<uintptr_t>(gp) & 7) == 0)) {
            gv.u2 = *reinterpret_cast<const uint2 *>(gp);
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (n + i < N) gv.h[i] = gp[i].bits;
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) mul[i] = 1.0f / (1.0f + expf(-bf16_bits_to_float(gv.h[i])));
    }
    if (n + 3 < N && aligned) {
        Frag4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v.h[i] = float_to_bf16_bits(acc[i] * mul[i]);
        *reinterpret_cast<uint2 *>(o) = v.u2;
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (n + i < N) o[i].bits = float_to_bf16_bits(acc[i] * mul[i]);
    }
}

template <int NKS, int NT>
__global__ void __launch_bounds__(KVA_WAVE)
heads_matmul_mfma_kernel(bf16_t *__restrict__ out, int o_row, int o_head, const bf16_t *__restrict__ x, int x_row,
                         int x_head, const bf16_t *__restrict__ w, int M, int N, int tiles_per_wave, HeadsGate gate,
                         HeadsRotate ro) {
    if (ro.rot > 0 && blockIdx.x == gridDim.x - 1) {            // the last column of workgroups rotates
        heads_rotate<bf16_t>(ro, blockIdx.y, min(M, (int)blockIdx.z * tiles_per_wave * 16),
                             min(M, (int)(blockIdx.z + 1) * tiles_per_wave * 16));
        return;
    }
    // NT neighbouring tiles of 16 outputs a wavefront: every fragment of x it loads serves NT products
    // (many rows: what a wavefront takes in per product is what bounds it); NT = 1 for few rows,
    // where more wavefronts matter more
    constexpr int K = NKS * 32;
    const int lane = threadIdx.x, r = lane & 15, g = lane >> 4;
    const int n_first = blockIdx.x * 16 * NT, h = blockIdx.y;
    Frag8 wf[NT][NKS];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
        const int n = min(n_first + 16 * nt + r, N - 1);
        const bf16_t *wrow = w + ((size_t)h * N + n) * K + 8 * g;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) wf[nt][ks].u4 = *reinterpret_cast<const uint4 *>(wrow + 32 * ks);
    }
    const int first = blockIdx.z * tiles_per_wave;
    for (int tile = first; tile < first + tiles_per_wave && tile * 16 < M; ++tile) {
        const int t = min(tile * 16 + r, M - 1);
        const bf16_t *xrow = x + (size_t)t * x_row + (size_t)h * x_head + 8 * g;
        Frag8 xf[NKS];
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) xf[ks].u4 = *reinterpret_cast<const uint4 *>(xrow + 32 * ks);
        float gmul = 1.f;
        if (gate.p && !gate.per_element) gmul = heads_gate<bf16_t>(gate, t, h, 0);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
            const int n0 = n_first + 16 * nt;
            if (n0 >= N) break;
            f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[nt][ks].v, xf[ks].v, acc, 0, 0, 0);
            // lane (row t = r, group g) holds outputs n0 + 4 g .. + 3 of its row
            if (tile * 16 + r < M) {
                heads_store4(out + (size_t)t * o_row + (size_t)h * o_head + n0 + 4 * g, acc, gmul, gate, t, h, n0 + 4 * g, N,
                             (o_row | o_head) % 4 == 0);
            }
        }
    }
}

// Many rows: a workgroup takes 32 RT rows and 128 outputs of one head, operands through LDS (lds_product.h).
#include "lds_product.h"

template <int RT>
__global__ void __launch_bounds__(256)
heads_matmul_lds_kernel(bf16_t *__restrict__ out, int o_row, int o_head, const bf16_t *__restrict__ x, int x_row, int x_head,
                        const bf16_t *__restrict__ w, int M, int N, int K, int n_blocks, int m_blocks, HeadsGate gate, HeadsRotate ro) {
    __shared__ __align__(16) typename LdsProduct<RT>::Shared shared;
    constexpr int ROWS = LdsProduct<RT>::ROWS;
    const int cols = n_blocks + (ro.rot > 0 ? 1 : 0);           // the last column of workgroups rotates
    const int id = die_order(blockIdx.x, gridDim.x);
    const int h = id / (cols * m_blocks), m0 = (id / cols) % m_blocks * ROWS, col = id % cols;
    if (col == n_blocks) {
        heads_rotate<bf16_t>(ro, h, m0, min(M, m0 + ROWS));
        return;
    }
    const int n0 = col * LDSP_N;
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    LdsProduct<RT> p;
#pragma unroll
    for (int i = 0; i < LdsProduct<RT>::XI; ++i)
        p.xp[i] = x + (size_t)min(m0 + p.row() + 32 * i, M - 1) * x_row + (size_t)h * x_head + p.element();
    p.plain_w(w + (size_t)h * N * K, N, K, n0);
    f32x4 acc[4][RT];
    p.run(shared, K, acc);
    // Results go out 16 bytes a lane, 256 neighbouring bytes a row: through LDS, where the operands were (a lane
    // holds 4 outputs of a row).  Rows that are not aligned for that are written as they are.
    constexpr int OUT_STRIDE = LDSP_N + 8;
    static_assert(sizeof(shared) >= ROWS * OUT_STRIDE * sizeof(bf16_t), "the results fit where the operands were");
    const bool through = (o_row | o_head | N) % 8 == 0 && (reinterpret_cast<uintptr_t>(out) & 15) == 0;
    bf16_t *tile = shared.x[0];
    if (through) __syncthreads();                               // nobody reads the operands any more
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int row = (wave & 1) * 16 * RT + 16 * rt + r, t = m0 + row;
        if (t >= M) continue;
        const float gmul = gate.p && !gate.per_element ? heads_gate<bf16_t>(gate, t, h, 0) : 1.f;
#pragma unroll
        for (int nt = 0; nt < 4; ++nt) {
            const int c = 64 * (wave >> 1) + 16 * nt + 4 * g, n = n0 + c;
            if (n >= N) continue;
            bf16_t *o = through ? tile + row * OUT_STRIDE + c : out + (size_t)t * o_row + (size_t)h * o_head + n;
            heads_store4(o, acc[nt][rt], gmul, gate, t, h, n, N, through || (o_row | o_head) % 4 == 0);
        }
    }
    if (!through) return;
    __syncthreads();
    const int c = 8 * (threadIdx.x % 16);
    if (n0 + c >= N) return;
    for (int row = threadIdx.x / 16; row < ROWS && m0 + row < M; row += 16)
        *reinterpret_cast<uint4 *>(out + (size_t)(m0 + row) * o_row + (size_t)h * o_head + n0 + c) =
            *reinterpret_cast<const uint4 *>(tile + row * OUT_STRIDE + c);
}

#define HM_LDS_ROWS 128         // more rows than this go through LDS
#define HM_INSTANCES(X) X(1) X(2) X(3) X(4) X(5) X(6) X(8) X(10) X(12) X(16)

extern "C" int kva_heads_matmul_mfma_supported(int K, int x_row, int x_head) {
    if (K % 32 || x_row % 8 || x_head % 8) return 0;
#define CHECK_ONE(NKS) if (K == NKS * 32) return 1;
    HM_INSTANCES(CHECK_ONE)
#undef CHECK_ONE
    return 0;
}

extern "C" int kva_heads_matmul_mfma(void *out, int o_row, int o_head, const void *x, int x_row, int x_head,
                                     const void *w, int rows, int heads, int N, int K, HEADS_OPTION_ARGS,
                                     hipStream_t stream) {
    KVA_REQUIRE(rows >= 0 && heads > 0 && heads <= 65535 && N > 0, "heads_matmul_mfma: bad sizes");
    KVA_REQUIRE(kva_heads_matmul_mfma_supported(K, x_row, x_head),
                "heads_matmul_mfma: no instance for K = %d with strides %d / %d", K, x_row, x_head);
    KVA_REQUIRE(x_head >= K && o_head >= N && x_row >= (heads - 1) * x_head + K && o_row >= (heads - 1) * o_head + N,
                "heads_matmul_mfma: strides do not fit %d heads of %d -> %d", heads, K, N);
    HEADS_OPTIONS(gate, ro);
    if (rows == 0) return KVA_OK;
    if (rows > HM_LDS_ROWS && N >= 64) {
        const int n_blocks = (N + LDSP_N - 1) / LDSP_N, cols = n_blocks + (rot > 0 ? 1 : 0);
        // the smaller tile where the larger would leave compute units without work
        const bool small = (long long)n_blocks * heads * ((rows + 127) / 128) < 512;
        const int tile = small ? 64 : 128, m_blocks = (rows + tile - 1) / tile;
        const long long blocks = (long long)cols * m_blocks * heads;
        KVA_REQUIRE(blocks <= 0x7fffffff, "heads_matmul_mfma: too many workgroups");
        auto kernel = small ? heads_matmul_lds_kernel<2> : heads_matmul_lds_kernel<4>;
        hipLaunchKernelGGL(kernel, dim3((unsigned)blocks), dim3(256), 0, stream, (bf16_t *)out, o_row, o_head, (const bf16_t *)x, x_row,
                           x_head, (const bf16_t *)w, rows, N, K, n_blocks, m_blocks, gate, ro);
        KVA_CHECK_LAUNCH("heads_matmul_mfma");
        return KVA_OK;
    }
    const int row_tiles = (rows + 15) / 16;
    const int n_tiles = (N + 15) / 16;
    // many rows: several output tiles a wavefront (at most 32 fragments of W in its registers)
    const bool wide = rows > 64;
    bool done = false;
#define LAUNCH_ONE(NKS)                                                                                          \
    if (!done && K == NKS * 32) {                                                                                \
        constexpr int NTW = NKS <= 8 ? 4 : (NKS <= 16 ? 2 : 1);                                                  \
        const int nt = wide ? NTW : 1;                                                                           \
        const int groups = (n_tiles + nt - 1) / nt;                                                              \
        /* enough wavefronts to fill the chip before a wavefront takes more than one row tile */                 \
        int per_wave = 1;                                                                                        \
        while (per_wave < 8 && (long long)groups * heads * ((row_tiles + per_wave - 1) / per_wave) > 4096) per_wave *= 2; \
        dim3 grid(groups + (rot > 0 ? 1 : 0), heads, (row_tiles + per_wave - 1) / per_wave), block(KVA_WAVE);                        \
        KVA_REQUIRE(grid.z <= 65535, "heads_matmul_mfma: %d rows are too many for one launch", rows);            \
        auto kernel = wide ? heads_matmul_mfma_kernel<NKS, NTW> : heads_matmul_mfma_kernel<NKS, 1>;              \
        hipLaunchKernelGGL(kernel, grid, block, 0, stream, (bf16_t *)out, o_row, o_head,                         \
                           (const bf16_t *)x, x_row, x_head, (const bf16_t *)w, rows, N, per_wave,               \
                           gate, ro);                                                                            \
        done = true;                                                                                             \
    }
    HM_INSTANCES(LAUNCH_ONE)
#undef LAUNCH_ONE
    KVA_CHECK_LAUNCH("heads_matmul_mfma");
    return KVA_OK;
}
