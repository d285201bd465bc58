// Attention over low-rank entries on the matrix cores (bf16, gfx950): prompt portions and decoded tokens.
//
// Every token keeps one row [latent (RANK) ; rotated key part] of KD elements for all heads
// (parts/latent_attention.py), in pages [page_size, KD].  A head's query is a row of the same KD elements,
// so all H heads of a token attend over the same rows: the 16 rows of a matrix-core tile are (token, head)
// pairs, row = token_in_entry * H + head, and each row of the cache that is loaded serves all of them.
//
// As in attention_mfma.hip everything is computed transposed:
//     S^T = K  Q^T   A = 16 rows of the cache x 32 of their elements (16 bytes a lane, row-major)
//     O^T = C^T P^T  A = 16 latent elements x 32 keys; the matrix core's k index of this product is the
//                    permutation of the 32 keys in which S^T left P in the registers (lane group g,
//                    element j <-> key (j / 4) * 16 + 4 g + j % 4)
// The latent is key and value at once, and it is read from memory ONCE: a block of 32 rows lies in LDS row by
// row, and the second product's operand is read there with the transposing load (ds_read_b64_tr_b16: of
// every 16 lanes, lane 4 k + c names 4 neighbouring elements of row k, and lane i gets element i of the four
// rows).  Rows are padded so that neither kind of read meets itself on a bank.
//
// Softmax is online in fp32, base 2.  A work item is (rows of one entry, a range of keys); it writes the
// normalised bf16 result itself when its range is all keys, otherwise an un-normalised partial (o, m, l)
// that latent_merge_kernel combines.  The sink of a head (one more term exp(sink) of its denominator) is
// added where the result is normalised.  Two kernels share the arithmetic:
//   * latent_attention_split_kernel: an item is 16 rows (a decoded token).  Its four wavefronts take the
//     blocks of the range in turn, each with LDS and a softmax of its own, and their results meet in LDS.
//   * latent_attention_rows_kernel: an item is 64 rows (a prompt portion), 16 a wavefront.  The four
//     wavefronts load a block together, a quarter each (two blocks deep: the next one's loads are in flight
//     while this one is multiplied), and all read it in LDS: a quarter of the traffic of wavefronts on their
//     own.
#include "common.h"
#include "attention_frag.h"
#include "kv_layout.h"
#include <math.h>

#define LAT_LOG2E 1.44269504088896340736f
#define LAT_WAVES 4

struct LatArgs {
    bf16_t *out;
    float *part_o, *part_ml;
    const bf16_t *q, *cache;
    const int *block_table, *item_entry, *item_row0, *entry_seat, *entry_q_start, *entry_start_pos;
    const float *sinks;
    int max_blocks, heads, page_size, window, keep_first, splits, per_split;
    float scale;
};

// what a wavefront knows of its 16 rows
struct LatRows {
    size_t first_row;               // of the entry, in q / out
    int row0, rows, start_pos;      // first row of the 16 inside the entry, rows of the entry
    int lo, hi, pos_lo, hi_lo;      // first visible key of row 0; newest key of any row; row 0's position; first visible key of the last row
    int my_row, my_pos, my_lo;      // of this lane's row (lane % 16)
    bool my_valid;
};

__device__ __forceinline__ LatRows lat_rows(const LatArgs &a, int e, int row0, int r) {
    LatRows w;
    const int q_start = a.entry_q_start[e], q_len = a.entry_q_start[e + 1] - q_start;
    w.start_pos = a.entry_start_pos[e];
    w.rows = q_len * a.heads;
    w.first_row = (size_t)q_start * a.heads;
    w.row0 = row0;
    const int last = min(row0 + 15, w.rows - 1), first = min(row0, w.rows - 1);
    w.hi = w.start_pos + last / a.heads;
    w.pos_lo = w.start_pos + first / a.heads;
    w.my_valid = row0 + r < w.rows;
    w.my_row = min(row0 + r, w.rows - 1);
    w.my_pos = w.start_pos + w.my_row / a.heads;
    w.lo = kva_first_visible(w.pos_lo, a.window, 0);
    w.hi_lo = kva_first_visible(w.hi, a.window, 0);
    w.my_lo = kva_first_visible(w.my_pos, a.window, 0);
    return w;
}

// LDS stride, in elements, of rows of n elements (a multiple of 32): a few more, so that the stride is an odd
// multiple of 4 words and rows 0 to 3 of a transposing read lie on banks of their own (64 banks of a word)
constexpr bool lat_stride_fits(int words) {
    for (int i = 1; i < 4; ++i) {
        const int d = (i * words) % 64;
        if (d < 8 || d > 56) return false;
    }
    return words % 8 == 4;
}
constexpr int lat_stride(int n) {
    int words = n / 2;
    while (!lat_stride_fits(words)) ++words;
    return 2 * words;
}

// the rows of the cache a lane reads of a block of 32 keys: key r of either tile of 16 (which lies in one page),
// from element 8 g on
struct LatBlock {
    const bf16_t *row[2];
    bool mapped[2];
};

template <int KD>
__device__ __forceinline__ LatBlock lat_block(const LatArgs &a, const int *bt, int kstart, int hi, int r, int g) {
    LatBlock b;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int key0 = kstart + 16 * t;
        const int p = key0 <= hi ? bt[key0 / a.page_size] : -1;
        b.mapped[t] = p >= 0;
        // (keys nobody sees are read from a page that exists)
        b.row[t] = a.cache + ((size_t)(p >= 0 ? p : 0) * a.page_size + (key0 + r) % a.page_size) * KD + 8 * g;
    }
    return b;
}

// Rows that no row of the item may see (past its newest key, outside its range, on an unmapped page) are made
// zero before they are multiplied: their probabilities are, and zero times whatever a page held before must
// stay zero.
__device__ __forceinline__ uint4 lat_zero_unless(bool on, uint4 v) {
    return on ? v : make_uint4(0u, 0u, 0u, 0u);
}

// 8 keys of latent element 16 dt + r as the second product's operand: `at` points at the lane's place in the
// block's first row (row 4 g + r / 4, element 4 (r % 4)), tile t and dt are constants behind it
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
template <int STRIDE>
__device__ __forceinline__ Frag8 lat_values(const bf16_t *at, int dt) {
    union { s16x4 t[2]; Frag8 f; } u;
    u.t[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4 *)(at + 16 * dt));
    u.t[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4 *)(at + 16 * STRIDE + 16 * dt));
    return u.f;
}

// mask, online softmax and P of one block: `s` are the two tiles of S^T, `o`, `m`, `l` are re-based when a row's
// running maximum moves (wave-uniform branch)
template <int NDT>
__device__ __forceinline__ Frag8 lat_softmax(const LatArgs &a, const LatRows &w, const f32x4 (&s)[2], const bool (&mapped)[2],
                                             int kstart, int k_begin, int k_end, int g, f32x4 (&o)[NDT], float &m, float &l) {
    const float scale2 = a.scale * LAT_LOG2E;
    const bool whole = mapped[0] && mapped[1] && kstart >= k_begin && kstart + 32 <= k_end && kstart + 31 <= w.pos_lo &&
                       (kstart >= w.hi_lo || kstart + 32 <= a.keep_first);
    float sv[8], mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            float x = s[t][i] * scale2;
            if (!whole) {
                const int key = kstart + 16 * t + 4 * g + i;
                const bool vis = w.my_valid && mapped[t] && key <= w.my_pos &&
                                 (key >= w.my_lo || key < a.keep_first) && key >= k_begin && key < k_end;
                x = vis ? x : -INFINITY;
            }
            sv[t * 4 + i] = x;
            mx = fmaxf(mx, x);
        }
    const float bm = quad_rows_max(mx);
    if (__builtin_amdgcn_ballot_w64(bm > m) != 0) {
        const float m_new = fmaxf(m, bm);
        const float corr = __builtin_amdgcn_exp2f(m - ((m_new == -INFINITY) ? 0.f : m_new));     // exp2(-inf) = 0
        l *= corr;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            o[dt][0] *= corr; o[dt][1] *= corr; o[dt][2] *= corr; o[dt][3] *= corr;
        }
        m = m_new;
    }
    const float ref = (m == -INFINITY) ? 0.f : m;
    Frag8 pf;
#pragma unroll
    for (int j = 0; j < 8; j += 2) {
        const float p0 = __builtin_amdgcn_exp2f(sv[j] - ref), p1 = __builtin_amdgcn_exp2f(sv[j + 1] - ref);
        l += p0 + p1;
        pf.p2[j / 2] = pack_bf16(p0, p1);
    }
    return pf;
}

// the factor that normalises a row, its head's sink included
__device__ __forceinline__ float lat_finish(const float *sinks, int head, float m, float l) {
    if (!sinks) return 1.f / l;
    const float sk = sinks[head] * LAT_LOG2E, m_new = fmaxf(m, sk);
    const float corr = __builtin_amdgcn_exp2f(m - m_new);
    return corr / (l * corr + __builtin_amdgcn_exp2f(sk - m_new));
}

__device__ __forceinline__ void lat_store4(bf16_t *p, float a, float b, float c, float d) {
    Frag4 w;
    w.h[0] = float_to_bf16_bits(a); w.h[1] = float_to_bf16_bits(b); w.h[2] = float_to_bf16_bits(c); w.h[3] = float_to_bf16_bits(d);
    *reinterpret_cast<uint2 *>(p) = w.u2;
}

template <int NDT /* RANK / 16 */, int NKS /* KD / 32 */>
__global__ void __launch_bounds__(LAT_WAVES *KVA_WAVE) __attribute__((amdgpu_waves_per_eu(1, 2)))
latent_attention_split_kernel(LatArgs a) {
    constexpr int RANK = NDT * 16, KD = NKS * 32, STRIDE = lat_stride(RANK), TILE = 32 * STRIDE;
    // a block's latents per wavefront; later the wavefronts' results [wave][dt][lane]
    constexpr int BYTES = LAT_WAVES * (TILE * 2 > NDT * KVA_WAVE * 16 ? TILE * 2 : NDT * KVA_WAVE * 16);
    __shared__ __align__(16) char lds[BYTES];
    __shared__ float ml_s[LAT_WAVES][16][2];
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int item = blockIdx.x, split = blockIdx.y;
    const int e = a.item_entry[item];
    const int *bt = a.block_table + (size_t)a.entry_seat[e] * a.max_blocks;
    const LatRows w = lat_rows(a, e, a.item_row0[item], r);
    int k_begin = 0, k_end = w.hi + 1;
    if (a.splits > 1) {
        k_begin = split * a.per_split;
        k_end = min(k_end, k_begin + a.per_split);
    }
    Frag8 qf[NKS];
    {
        const bf16_t *qrow = a.q + (w.first_row + w.my_row) * KD + 8 * g;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) qf[ks].u4 = *reinterpret_cast<const uint4 *>(qrow + 32 * ks);
    }
    bf16_t *tile = reinterpret_cast<bf16_t *>(lds) + wave * TILE;
    bf16_t *put = tile + r * STRIDE + 8 * g;
    const bf16_t *get = tile + (4 * g + (r >> 2)) * STRIDE + 4 * (r & 3);
    f32x4 o[NDT];
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;                           // m in the base-2 domain, l this lane's part
    Frag8 kf[2][NKS];
    bool mapped[2] = {false, false};
#define LAT_LOAD_BLOCK(KSTART)                                                                                   \
    {                                                                                                            \
        const LatBlock b = lat_block<KD>(a, bt, KSTART, w.hi, r, g);                                             \
        _Pragma("unroll") for (int t = 0; t < 2; ++t) {                                                          \
            mapped[t] = b.mapped[t];                                                                             \
            _Pragma("unroll") for (int ks = 0; ks < NKS; ++ks)                                                   \
                kf[t][ks].u4 = *reinterpret_cast<const uint4 *>(b.row[t] + 32 * ks);                             \
        }                                                                                                        \
    }
    // (blocks behind every row's window and past the kept positions are left out)
    int kstart = (k_begin & ~31) + 32 * wave;
    while (kstart < k_end && kstart + 32 <= w.lo && kstart >= a.keep_first) kstart += 32 * LAT_WAVES;
    if (kstart < k_end) LAT_LOAD_BLOCK(kstart);
    while (kstart < k_end) {
        const bool here[2] = {mapped[0], mapped[1]};
        if (!(here[0] && here[1] && kstart >= k_begin && kstart + 32 <= k_end)) {       // (wave-uniform, rare)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const int key = kstart + 16 * t + r;
                const bool on = here[t] && key >= k_begin && key < k_end;
#pragma unroll
                for (int ks = 0; ks < NKS; ++ks) kf[t][ks].u4 = lat_zero_unless(on, kf[t][ks].u4);
            }
        }
        f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                if (32 * ks < RANK) *reinterpret_cast<uint4 *>(put + 16 * t * STRIDE + 32 * ks) = kf[t][ks].u4;
                s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][ks].v, qf[ks].v, s[t], 0, 0, 0);
            }
        int next = kstart + 32 * LAT_WAVES;
        while (next < k_end && next + 32 <= w.lo && next >= a.keep_first) next += 32 * LAT_WAVES;
        if (next < k_end) LAT_LOAD_BLOCK(next);
        const Frag8 pf = lat_softmax<NDT>(a, w, s, here, kstart, k_begin, k_end, g, o, m, l);
        // what the lanes of this wavefront wrote, its other lanes read: in the wavefront's own order
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        constexpr int VC = 4;                               // value tiles read ahead
        Frag8 vf[2][VC];
#pragma unroll
        for (int j = 0; j < VC; ++j) vf[0][j] = lat_values<STRIDE>(get, j);
#pragma unroll
        for (int d0 = 0; d0 < NDT; d0 += VC) {
#pragma unroll
            for (int j = 0; j < VC; ++j)
                if (d0 + VC + j < NDT) vf[(d0 / VC + 1) & 1][j] = lat_values<STRIDE>(get, d0 + VC + j);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int j = 0; j < VC; ++j)
                if (d0 + j < NDT) o[d0 + j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[(d0 / VC) & 1][j].v, pf.v, o[d0 + j], 0, 0, 0);
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        kstart = next;
    }
#undef LAT_LOAD_BLOCK
    // the wavefronts' results meet: every one re-bases its own to the common maximum
    l = quad_rows_sum(l);
    if (g == 0) {
        ml_s[wave][r][0] = m;
        ml_s[wave][r][1] = l;
    }
    __syncthreads();                                        // (also: nobody reads a block any more)
    float m_all = -INFINITY;
#pragma unroll
    for (int v = 0; v < LAT_WAVES; ++v) m_all = fmaxf(m_all, ml_s[v][r][0]);
    const float corr = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - m_all);
    float4 *results = reinterpret_cast<float4 *>(lds);
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
        results[(wave * NDT + dt) * KVA_WAVE + lane] =
            make_float4(o[dt][0] * corr, o[dt][1] * corr, o[dt][2] * corr, o[dt][3] * corr);
    float l_all = 0.f;
#pragma unroll
    for (int v = 0; v < LAT_WAVES; ++v)
        l_all += ml_s[v][r][0] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(ml_s[v][r][0] - m_all) * ml_s[v][r][1];
    __syncthreads();
    // lane (row r, group g) of tile dt: elements 16 dt + 4 g .. + 3 of row r
    if (!w.my_valid) return;
    const size_t row = w.first_row + w.my_row;
    const float mul = a.splits > 1 ? 1.f : lat_finish(a.sinks, w.my_row % a.heads, m_all, l_all);
    if (a.splits > 1 && wave == 0 && g == 0) {
        a.part_ml[(row * a.splits + split) * 2] = m_all;
        a.part_ml[(row * a.splits + split) * 2 + 1] = l_all;
    }
    for (int dt = wave; dt < NDT; dt += LAT_WAVES) {
        float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int v = 0; v < LAT_WAVES; ++v) {
            const float4 x = results[(v * NDT + dt) * KVA_WAVE + lane];
            t.x += x.x; t.y += x.y; t.z += x.z; t.w += x.w;
        }
        if (a.splits > 1)
            *reinterpret_cast<float4 *>(a.part_o + (row * a.splits + split) * RANK + 16 * dt + 4 * g) = t;
        else
            lat_store4(a.out + row * RANK + 16 * dt + 4 * g, t.x * mul, t.y * mul, t.z * mul, t.w * mul);
    }
}

template <int NDT, int NKS>
__global__ void __launch_bounds__(LAT_WAVES *KVA_WAVE) __attribute__((amdgpu_waves_per_eu(1, 1)))
latent_attention_rows_kernel(LatArgs a) {
    constexpr int RANK = NDT * 16, KD = NKS * 32, STRIDE = lat_stride(KD), TILE = 32 * STRIDE;
    constexpr int KI = (NKS + 1) / 2;                       // 16-byte pieces of a block a lane loads: one tile, every second k step
    __shared__ __align__(16) bf16_t lds[2][TILE];
    const int lane = threadIdx.x % KVA_WAVE, wave = threadIdx.x / KVA_WAVE, r = lane & 15, g = lane >> 4;
    const int item = blockIdx.x, split = blockIdx.y;
    const int e = a.item_entry[item], item_row0 = a.item_row0[item];
    const int *bt = a.block_table + (size_t)a.entry_seat[e] * a.max_blocks;
    const LatRows w = lat_rows(a, e, item_row0 + 16 * wave, r);
    const int item_hi = w.start_pos + min(item_row0 + 16 * LAT_WAVES - 1, w.rows - 1) / a.heads;      // newest key of any row of the item
    const int item_lo = kva_first_visible(w.start_pos + item_row0 / a.heads, a.window, 0);
    int k_begin = 0, k_end = item_hi + 1;
    if (a.splits > 1) {
        k_begin = split * a.per_split;
        k_end = min(k_end, k_begin + a.per_split);
    }
    Frag8 qf[NKS];
    {
        const bf16_t *qrow = a.q + (w.first_row + w.my_row) * KD + 8 * g;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) qf[ks].u4 = *reinterpret_cast<const uint4 *>(qrow + 32 * ks);
    }
    f32x4 o[NDT];
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    const bool has_rows = w.row0 < w.rows;
    // this wavefront's quarter of a block: tile `my_t`, k steps my_ks, my_ks + 2, ... (an odd count: the last one twice)
    const int my_t = wave & 1, my_ks = wave >> 1;
    const int put = (16 * my_t + r) * STRIDE + 8 * g + 32 * my_ks;
    const int put_last = (16 * my_t + r) * STRIDE + 8 * g + 32 * min(my_ks + 2 * (KI - 1), NKS - 1);
    const int get_k = r * STRIDE + 8 * g, get_v = (4 * g + (r >> 2)) * STRIDE + 4 * (r & 3);
    uint4 ka[KI];
    bool on = false;                                        // whether the lane's row of the loaded block counts
    bool mapped[2] = {false, false};
#define LAT_LOAD_QUARTER(KSTART)                                                                                 \
    {                                                                                                            \
        const LatBlock b = lat_block<KD>(a, bt, KSTART, item_hi, r, g);                                          \
        mapped[0] = b.mapped[0]; mapped[1] = b.mapped[1];                                                        \
        const int key = (KSTART) + 16 * my_t + r;                                                                \
        on = (my_t ? mapped[1] : mapped[0]) && key >= k_begin && key < k_end;                                    \
        const bf16_t *row = (my_t ? b.row[1] : b.row[0]);                                                        \
        _Pragma("unroll") for (int i = 0; i < KI; ++i)                                                           \
            ka[i] = *reinterpret_cast<const uint4 *>(row + 32 * (i + 1 < KI ? my_ks + 2 * i : min(my_ks + 2 * i, NKS - 1))); \
    }
    // (blocks behind every row's window and past the kept positions are left out)
    int kstart = k_begin & ~31, buf = 0;
    while (kstart < k_end && kstart + 32 <= item_lo && kstart >= a.keep_first) kstart += 32;
    if (kstart < k_end) LAT_LOAD_QUARTER(kstart);
    while (kstart < k_end) {
        // (the buffer was read last two blocks ago: every wavefront has passed the barrier of the block between)
        const bool here[2] = {mapped[0], mapped[1]};
        bf16_t *tile = lds[buf];
#pragma unroll
        for (int i = 0; i < KI; ++i)
            *reinterpret_cast<uint4 *>(tile + (i + 1 < KI ? put + 64 * i : put_last)) = lat_zero_unless(on, ka[i]);
        __syncthreads();
        int next = kstart + 32;
        while (next < k_end && next + 32 <= item_lo && next >= a.keep_first) next += 32;
        if (next < k_end) LAT_LOAD_QUARTER(next);
        if (has_rows && kstart <= w.hi) {                   // (a later wavefront's rows may see keys that this one's do not)
            const bf16_t *kt = tile + get_k, *vt = tile + get_v;
            f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
            constexpr int GK = 3, VC = 4;                   // k steps, value tiles read ahead
            Frag8 kf[2][GK][2], vf[2][VC];
#define LAT_READ_KEYS(B, K0)                                                                                     \
    _Pragma("unroll") for (int j = 0; j < GK; ++j) _Pragma("unroll") for (int t = 0; t < 2; ++t)                 \
        if ((K0) + j < NKS) kf[B][j][t].u4 = *reinterpret_cast<const uint4 *>(kt + 16 * t * STRIDE + 32 * ((K0) + j));
            LAT_READ_KEYS(0, 0)
#pragma unroll
            for (int k0 = 0; k0 < NKS; k0 += GK) {
                if (k0 + GK < NKS) {
                    LAT_READ_KEYS((k0 / GK + 1) & 1, k0 + GK)
                } else {
#pragma unroll
                    for (int j = 0; j < VC; ++j) vf[0][j] = lat_values<STRIDE>(vt, j);
                }
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int j = 0; j < GK; ++j)
#pragma unroll
                    for (int t = 0; t < 2; ++t)
                        if (k0 + j < NKS)
                            s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[(k0 / GK) & 1][j][t].v, qf[k0 + j].v, s[t], 0, 0, 0);
            }
#undef LAT_READ_KEYS
            const Frag8 pf = lat_softmax<NDT>(a, w, s, here, kstart, k_begin, k_end, g, o, m, l);
#pragma unroll
            for (int d0 = 0; d0 < NDT; d0 += VC) {
#pragma unroll
                for (int j = 0; j < VC; ++j)
                    if (d0 + VC + j < NDT) vf[(d0 / VC + 1) & 1][j] = lat_values<STRIDE>(vt, d0 + VC + j);
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int j = 0; j < VC; ++j)
                    if (d0 + j < NDT) o[d0 + j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[(d0 / VC) & 1][j].v, pf.v, o[d0 + j], 0, 0, 0);
            }
        }
        kstart = next;
        buf ^= 1;
    }
#undef LAT_LOAD_QUARTER
    l = quad_rows_sum(l);
    if (!w.my_valid) return;
    const size_t row = w.first_row + w.my_row;
    if (a.splits > 1) {
        float *po = a.part_o + (row * a.splits + split) * RANK + 4 * g;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) *reinterpret_cast<float4 *>(po + 16 * dt) = make_float4(o[dt][0], o[dt][1], o[dt][2], o[dt][3]);
        if (g == 0) {
            a.part_ml[(row * a.splits + split) * 2] = m;
            a.part_ml[(row * a.splits + split) * 2 + 1] = l;
        }
        return;
    }
    const float mul = lat_finish(a.sinks, w.my_row % a.heads, m, l);
    bf16_t *orow = a.out + row * RANK + 4 * g;
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt) lat_store4(orow + 16 * dt, o[dt][0] * mul, o[dt][1] * mul, o[dt][2] * mul, o[dt][3] * mul);
}

// out[row] = sum_s w_s o_s / (sum_s w_s l_s + exp(sink)), w_s = exp2(m_s - max); one workgroup a row.  Threads
// take four neighbouring columns and every so-manyth range, and the groups' sums meet in LDS in a fixed
// order.  A range without a visible key (most of them under a window or chunks) has l = 0 and is not read.
#define LAT_MERGE_MAX_SPLITS 8192
__global__ void __launch_bounds__(256)
latent_merge_kernel(bf16_t *__restrict__ out, const float *__restrict__ part_o, const float *__restrict__ part_ml,
                    const float *__restrict__ sinks, int heads, int rank, int splits) {
    extern __shared__ float w_s[];                          // weights of the ranges
    __shared__ float4 sum_s[256];
    __shared__ float den_s;
    const size_t row = blockIdx.x;
    const float *ml = part_ml + row * splits * 2;
    if (threadIdx.x < KVA_WAVE) {
        const float sk = sinks ? sinks[row % heads] * LAT_LOG2E : -INFINITY;
        float m = sk;
        for (int s = threadIdx.x; s < splits; s += KVA_WAVE) m = fmaxf(m, ml[2 * s]);
        m = wave_max(m);
        float den = 0.f;
        for (int s = threadIdx.x; s < splits; s += KVA_WAVE) {
            const float l = ml[2 * s + 1], w = l != 0.f ? __builtin_amdgcn_exp2f(ml[2 * s] - m) : 0.f;
            w_s[s] = w;
            den += w * l;
        }
        den = wave_sum(den);
        if (threadIdx.x == 0) den_s = den + (sinks ? __builtin_amdgcn_exp2f(sk - m) : 0.f);
    }
    __syncthreads();
    const int cols = rank / 4, groups = blockDim.x / cols, col = threadIdx.x % cols, grp = threadIdx.x / cols;
    float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
    if (grp < groups) {
        const float *src = part_o + row * splits * rank + 4 * col;
        for (int s0 = grp; s0 < splits; s0 += 4 * groups) {
            float4 v[4];
            float w[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {                   // four ranges' loads in flight
                const int s = s0 + j * groups;
                w[j] = s < splits ? w_s[s] : 0.f;
                v[j] = w[j] != 0.f ? *reinterpret_cast<const float4 *>(src + (size_t)s * rank) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                acc.x += w[j] * v[j].x; acc.y += w[j] * v[j].y; acc.z += w[j] * v[j].z; acc.w += w[j] * v[j].w;
            }
        }
    }
    sum_s[threadIdx.x] = acc;
    __syncthreads();
    if (grp != 0) return;
    for (int k = 1; k < groups; ++k) {
        const float4 v = sum_s[k * cols + col];
        acc.x += v.x; acc.y += v.y; acc.z += v.z; acc.w += v.w;
    }
    const float inv = 1.f / den_s;
    lat_store4(out + row * rank + 4 * col, acc.x * inv, acc.y * inv, acc.z * inv, acc.w * inv);
}

static int latent_merge_launch(void *out, const float *part_o, const float *part_ml, const float *sinks, int total_rows, int heads,
                               int rank, int splits, hipStream_t stream) {
    KVA_REQUIRE(rank % 4 == 0 && rank <= 1024, "attention merge: rows of %d (a multiple of 4 up to 1,024)", rank);
    KVA_REQUIRE(splits <= LAT_MERGE_MAX_SPLITS, "attention merge: %d ranges (at most %d)", splits, LAT_MERGE_MAX_SPLITS);
    if (total_rows == 0) return KVA_OK;
    hipLaunchKernelGGL(latent_merge_kernel, dim3(total_rows), dim3(256), (size_t)splits * sizeof(float), stream, (bf16_t *)out, part_o,
                       part_ml, sinks, heads, rank, splits);
    KVA_CHECK_LAUNCH("attention_merge");
    return KVA_OK;
}

// The (rank, row size) pairs with an instance.
#define LAT_INSTANCES(X) X(4, 3) X(4, 4) X(6, 4) X(8, 5) X(8, 6) X(10, 6) X(12, 7) X(16, 9) X(16, 10) X(32, 18) X(24, 14)

extern "C" int kva_latent_attention_mfma_supported(int rank, int key_dim, int page_size) {
    if (page_size <= 0 || page_size % 16) return 0;
#define CHECK_ONE(NDT, NKS) if (rank == NDT * 16 && key_dim == NKS * 32) return 1;
    LAT_INSTANCES(CHECK_ONE)
#undef CHECK_ONE
    return 0;
}

// rows_per_item 16 (the kernel whose wavefronts share the keys of few rows) or 64 (the one whose wavefronts
// share the loads of many); with several key ranges the caller merges once all launches of the step are done
extern "C" int kva_latent_attention_mfma(void *out, float *part_o, float *part_ml, const void *q, const void *cache,
                                         const int *block_table, int max_blocks,
                                         const int *item_entry, const int *item_row0, const int *entry_seat,
                                         const int *entry_q_start, const int *entry_start_pos, int num_items,
                                         int rows_per_item, int heads, int rank, int key_dim, int page_size, float scale,
                                         int window, int keep_first, const float *sinks, int splits, int per_split,
                                         hipStream_t stream) {
    KVA_REQUIRE(kva_latent_attention_mfma_supported(rank, key_dim, page_size),
                "latent_attention_mfma: no instance for rank %d, rows of %d, pages of %d", rank, key_dim, page_size);
    KVA_REQUIRE(num_items >= 0 && heads > 0 && max_blocks > 0, "latent_attention_mfma: bad sizes");
    KVA_REQUIRE(rows_per_item == 16 || rows_per_item == 16 * LAT_WAVES, "latent_attention_mfma: items of 16 or %d rows", 16 * LAT_WAVES);
    KVA_REQUIRE(splits >= 1 && splits <= 65535 && (splits == 1 || (per_split > 0 && per_split % 32 == 0 && part_o && part_ml)),
                "latent_attention_mfma: key ranges need a length that is a multiple of 32 and a workspace");
    KVA_REQUIRE(window >= 0 && keep_first >= 0, "latent_attention_mfma: negative window or kept first positions");
    if (window == 0) keep_first = 0;
    if (num_items == 0) return KVA_OK;
    const LatArgs a{(bf16_t *)out, part_o, part_ml, (const bf16_t *)q, (const bf16_t *)cache, block_table,
                    item_entry, item_row0, entry_seat, entry_q_start, entry_start_pos, sinks, max_blocks, heads, page_size, window,
                    keep_first, splits, per_split, scale};
    dim3 grid(num_items, splits), block(LAT_WAVES * KVA_WAVE);
    bool done = false;
#define LAUNCH_ONE(NDT, NKS)                                                                                   \
    if (!done && rank == NDT * 16 && key_dim == NKS * 32) {                                                    \
        if (rows_per_item == 16)                                                                               \
            hipLaunchKernelGGL((latent_attention_split_kernel<NDT, NKS>), grid, block, 0, stream, a);          \
        else                                                                                                   \
            hipLaunchKernelGGL((latent_attention_rows_kernel<NDT, NKS>), grid, block, 0, stream, a);           \
        done = true;                                                                                           \
    }
    LAT_INSTANCES(LAUNCH_ONE)
#undef LAUNCH_ONE
    KVA_CHECK_LAUNCH("latent_attention_mfma");
    return KVA_OK;
}

extern "C" int kva_latent_attention_merge(void *out, const float *part_o, const float *part_ml, const float *sinks, int total_rows,
                                          int heads, int rank, int splits, hipStream_t stream) {
    KVA_REQUIRE(out && part_o && part_ml && total_rows >= 0 && heads > 0 && splits > 1, "latent_attention_merge: bad arguments");
    return latent_merge_launch(out, part_o, part_ml, sinks, total_rows, heads, rank, splits, stream);
}


// ---- grouped-query attention with the same options ---------------------------------------------
//
// The kernel above over the paged K / V^T arrays of ordinary attention (kv_layout.h), for what the
// tuned kernels of attention_mfma.hip do not take: chunks of positions that see only each other,
// a window that keeps a request's first
// positions visible, a sink per head, values of another size than the keys.  Rows of a tile are
// (token, query head of the kv head's group) pairs, row = token_in_entry * G + head_in_group; one
// wavefront per (item, kv head, key range).  D = 32 NKS key elements, DV = 16 NDT value elements.
template <int NDT, int NKS, int RT>
__global__ void __launch_bounds__(KVA_WAVE)
gqa_attention_rows_kernel(bf16_t *__restrict__ out, float *__restrict__ part_o, float *__restrict__ part_ml,
                          const bf16_t *__restrict__ q, int q_stride, const bf16_t *__restrict__ k_cache,
                          const bf16_t *__restrict__ v_cache, const int *__restrict__ block_table, int max_blocks,
                          const int *__restrict__ item_entry, const int *__restrict__ item_row0,
                          const int *__restrict__ entry_seat, const int *__restrict__ entry_q_start,
                          const int *__restrict__ entry_start_pos, int heads, int kv_heads, int page_size,
                          float scale, int window, int keep_first, int chunk, const float *__restrict__ sinks,
                          int splits, int per_split) {
    // RT tiles of 16 rows share every key and value fragment the wavefront loads (prompt portions:
    // half the loads a product with RT = 2)
    constexpr int DV = NDT * 16, D = NKS * 32;
    const int lane = threadIdx.x, r = lane & 15, g = lane >> 4;
    const int item = blockIdx.x, kvh = blockIdx.y / splits, split = blockIdx.y % splits;
    const int group = heads / kv_heads;
    const int e = item_entry[item], row0 = item_row0[item];
    const int q_start = entry_q_start[e], q_len = entry_q_start[e + 1] - q_start;
    const int start_pos = entry_start_pos[e];
    const int *bt = block_table + (size_t)entry_seat[e] * max_blocks;
    const int rows = q_len * group;
    if (row0 >= rows) return;
    const int last_row = min(row0 + 16 * RT - 1, rows - 1);
    const int item_hi = start_pos + last_row / group;
    const int pos_lo = start_pos + row0 / group;
    const int item_lo = kva_first_visible(pos_lo, window, chunk);
    const int hi_lo = kva_first_visible(item_hi, window, chunk);     // where the last row's window (or chunk) starts
    int my_pos[RT], my_lo[RT], my_head[RT];
    bool row_valid[RT];
    size_t my_token[RT];
    Frag8 qf[RT][NKS];
    f32x4 o[RT][NDT];
    float m[RT], l[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int row = min(row0 + 16 * rt + r, rows - 1);
        row_valid[rt] = row0 + 16 * rt + r < rows;
        my_pos[rt] = start_pos + row / group;
        my_head[rt] = kvh * group + row % group;
        my_lo[rt] = kva_first_visible(my_pos[rt], window, chunk);
        my_token[rt] = (size_t)q_start + row / group;
        const bf16_t *qrow = q + my_token[rt] * q_stride + (size_t)my_head[rt] * D + 8 * g;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) qf[rt][ks].u4 = *reinterpret_cast<const uint4 *>(qrow + 32 * ks);
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) o[rt][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
        m[rt] = -INFINITY;
        l[rt] = 0.f;
    }
    const float scale2 = scale * LAT_LOG2E;

    int k_begin = 0, k_end = item_hi + 1;
    if (splits > 1) {
        k_begin = split * per_split;
        k_end = min(k_end, k_begin + per_split);
    }
    if (keep_first == 0 && item_lo > k_begin) k_begin = min(item_lo & ~31, k_end);     // nothing in front is visible
    for (int kstart = k_begin & ~31; kstart < k_end; kstart += 32) {
        if (kstart + 32 <= item_lo && kstart >= keep_first) continue;
        int page[2];
        bool mapped[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const int key0 = kstart + 16 * t;
            const int p = key0 <= item_hi ? bt[key0 / page_size] : -1;
            mapped[t] = p >= 0;
            page[t] = p >= 0 ? p : 0;
        }
        // every load of the block is asked for before the first product
        Frag8 kf[2][NKS], vv[NDT];
        uint2 keep[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            const int key = kstart + 16 * t + r;
            // K pages are [D / 8][page_size][8]: chunk 4 ks + g of key `key`
            const bf16_t *kp = k_cache + ((size_t)page[t] * kv_heads + kvh) * page_size * D +
                               ((size_t)g * page_size + key % page_size) * 8;
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) kf[t][ks].u4 = *reinterpret_cast<const uint4 *>(kp + (size_t)ks * 4 * page_size * 8);
            // values: lane (element r of a tile, group g) takes keys 4 g .. 4 g + 3 of the 16-key tile
            const int key0 = kstart + 16 * t + 4 * g;
            int n = min(item_hi + 1, k_end) - key0;
            if (!mapped[t] || key0 + 4 <= k_begin) n = 0;
            keep[t] = keep_first_keys(make_uint2(~0u, ~0u), n);
            if (key0 < k_begin && n > 0) {
                const uint2 head = keep_first_keys(make_uint2(~0u, ~0u), k_begin - key0);
                keep[t].x &= ~head.x; keep[t].y &= ~head.y;
            }
            const bf16_t *vrow = v_cache + (((size_t)page[t] * kv_heads + kvh) * DV + r) * page_size + key0 % page_size;
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt) vv[dt].u2[t] = *reinterpret_cast<const uint2 *>(vrow + (size_t)dt * 16 * page_size);
        }
        __builtin_amdgcn_sched_barrier(0);
        // a block that every row of the item sees whole needs no mask (wave-uniform)
        const bool whole = mapped[0] && mapped[1] && kstart >= k_begin && kstart + 32 <= k_end && kstart + 31 <= pos_lo &&
                           (kstart >= hi_lo || kstart + 32 <= keep_first);
        Frag8 pf[RT];
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) {
            f32x4 s[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < NKS; ++ks)
                    s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][ks].v, qf[rt][ks].v, s[t], 0, 0, 0);
            }
            float sv[8], mx = -INFINITY;
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    float x = s[t][i] * scale2;
                    if (!whole) {
                        const int key = kstart + 16 * t + 4 * g + i;
                        const bool vis = row_valid[rt] && mapped[t] && key <= my_pos[rt] &&
                                         (key >= my_lo[rt] || key < keep_first) && key >= k_begin && key < k_end;
                        x = vis ? x : -INFINITY;
                    }
                    sv[t * 4 + i] = x;
                    mx = fmaxf(mx, x);
                }
            const float bm = quad_rows_max(mx);
            if (__builtin_amdgcn_ballot_w64(bm > m[rt]) != 0) {       // the maximum moved: re-base l and O
                const float m_new = fmaxf(m[rt], bm);
                const float corr = __builtin_amdgcn_exp2f(m[rt] - ((m_new == -INFINITY) ? 0.f : m_new));
                l[rt] *= corr;
#pragma unroll
                for (int dt = 0; dt < NDT; ++dt) {
                    o[rt][dt][0] *= corr; o[rt][dt][1] *= corr; o[rt][dt][2] *= corr; o[rt][dt][3] *= corr;
                }
                m[rt] = m_new;
            }
            const float ref = (m[rt] == -INFINITY) ? 0.f : m[rt];
#pragma unroll
            for (int j = 0; j < 8; j += 2) {
                const float p0 = __builtin_amdgcn_exp2f(sv[j] - ref), p1 = __builtin_amdgcn_exp2f(sv[j + 1] - ref);
                l[rt] += p0 + p1;
                pf[rt].p2[j / 2] = pack_bf16(p0, p1);
            }
        }
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            Frag8 v = vv[dt];
            v.u2[0].x &= keep[0].x; v.u2[0].y &= keep[0].y;
            v.u2[1].x &= keep[1].x; v.u2[1].y &= keep[1].y;
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) o[rt][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, pf[rt].v, o[rt][dt], 0, 0, 0);
        }
    }
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        float lsum = quad_rows_sum(l[rt]);
        if (!row_valid[rt]) continue;
        const size_t my_global = my_token[rt] * heads + my_head[rt];   // row of the output, of the partial results
        if (splits > 1) {
            float *po = part_o + (my_global * splits + split) * DV + 4 * g;
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt)
                *reinterpret_cast<float4 *>(po + 16 * dt) = make_float4(o[rt][dt][0], o[rt][dt][1], o[rt][dt][2], o[rt][dt][3]);
            if (g == 0) {
                part_ml[(my_global * splits + split) * 2] = m[rt];
                part_ml[(my_global * splits + split) * 2 + 1] = lsum;
            }
            continue;
        }
        float mul = 1.f;
        if (sinks) {
            const float sk = sinks[my_head[rt]] * LAT_LOG2E, m_new = fmaxf(m[rt], sk);
            const float corr = __builtin_amdgcn_exp2f(m[rt] - m_new);
            lsum = lsum * corr + __builtin_amdgcn_exp2f(sk - m_new);
            mul = corr;
        }
        mul /= lsum;
        bf16_t *orow = out + my_global * DV + 4 * g;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            Frag4 w;
            w.h[0] = float_to_bf16_bits(o[rt][dt][0] * mul); w.h[1] = float_to_bf16_bits(o[rt][dt][1] * mul);
            w.h[2] = float_to_bf16_bits(o[rt][dt][2] * mul); w.h[3] = float_to_bf16_bits(o[rt][dt][3] * mul);
            *reinterpret_cast<uint2 *>(orow + 16 * dt) = w.u2;
        }
    }
}

// (value size / 16, key size / 32) pairs with an instance
#define GQA_ROWS_INSTANCES(X) X(2, 1) X(4, 1) X(2, 2) X(4, 2) X(8, 2) X(6, 3) X(4, 4) X(8, 4) X(12, 6) X(16, 8)

extern "C" int kva_attention_rows_mfma_supported(int head_dim, int value_dim, int page_size) {
    if (page_size <= 0 || page_size % 16) return 0;
#define CHECK_ONE(NDT, NKS) if (value_dim == NDT * 16 && head_dim == NKS * 32) return 1;
    GQA_ROWS_INSTANCES(CHECK_ONE)
#undef CHECK_ONE
    return 0;
}

extern "C" int kva_attention_rows_mfma(void *out, float *part_o, float *part_ml, const void *q, int q_stride,
                                       const void *k_cache, const void *v_cache, const int *block_table,
                                       int max_blocks, const int *item_entry, const int *item_row0,
                                       const int *entry_seat, const int *entry_q_start, const int *entry_start_pos,
                                       int num_items, int total_rows, int heads, int kv_heads, int head_dim,
                                       int value_dim, int page_size, float scale, int window, int keep_first,
                                       int chunk, const float *sinks, int splits, int per_split, int row_tiles,
                                       hipStream_t stream) {
    KVA_REQUIRE(kva_attention_rows_mfma_supported(head_dim, value_dim, page_size),
                "attention_rows_mfma: no instance for keys of %d, values of %d, pages of %d", head_dim, value_dim, page_size);
    KVA_REQUIRE(num_items >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && max_blocks > 0 && total_rows >= 0,
                "attention_rows_mfma: bad sizes");
    KVA_REQUIRE(q_stride % 8 == 0 && q_stride >= heads * head_dim, "attention_rows_mfma: query row stride %d", q_stride);
    KVA_REQUIRE(splits >= 1 && (long long)splits * kv_heads <= 65535 &&
                    (splits == 1 || (per_split > 0 && per_split % 32 == 0 && part_o && part_ml)),
                "attention_rows_mfma: key ranges need a length that is a multiple of 32 and a workspace");
    KVA_REQUIRE(window >= 0 && keep_first >= 0 && chunk >= 0 && !(window > 0 && chunk > 0),
                "attention_rows_mfma: negative window, kept first positions or chunk, or a window together with chunks");
    KVA_REQUIRE(row_tiles == 1 || (row_tiles == 2 && value_dim <= 128 && head_dim <= 128),
                "attention_rows_mfma: one row tile an item, or two for heads up to 128");
    if (window == 0) keep_first = 0;
    if (num_items == 0) return KVA_OK;
    dim3 grid(num_items, kv_heads * splits), block(KVA_WAVE);
    bool done = false;
#define LAUNCH_ONE(NDT, NKS)                                                                                    \
    if (!done && value_dim == NDT * 16 && head_dim == NKS * 32) {                                               \
        auto kernel = gqa_attention_rows_kernel<NDT, NKS, 1>;                                                    \
        if constexpr (NDT <= 8 && NKS <= 4) {                                                                    \
            if (row_tiles == 2) kernel = gqa_attention_rows_kernel<NDT, NKS, 2>;                                 \
        }                                                                                                        \
        hipLaunchKernelGGL(kernel, grid, block, 0, stream, (bf16_t *)out, part_o,                                \
                           part_ml, (const bf16_t *)q, q_stride, (const bf16_t *)k_cache,                        \
                           (const bf16_t *)v_cache, block_table, max_blocks, item_entry, item_row0, entry_seat,  \
                           entry_q_start, entry_start_pos, heads, kv_heads, page_size, scale, window,            \
                           keep_first, chunk, sinks, splits, per_split);                                                \
        done = true;                                                                                             \
    }
    GQA_ROWS_INSTANCES(LAUNCH_ONE)
#undef LAUNCH_ONE
    KVA_CHECK_LAUNCH("attention_rows_mfma");
    if (splits > 1) return latent_merge_launch(out, part_o, part_ml, sinks, total_rows, heads, value_dim, splits, stream);
    return KVA_OK;
}
