// Attention over the paged cache whose heads' weights are mixed before they meet the values:
//
//   s_h(j)  = (q_h . k_j) * scale - slope_h (p - j)             j of the query's own chunk, j <= p
//   w_h(j)  = softmax over j
//   w'_h(j) = sum_g talk[h, g] w_g(j)                            talk float32 [H, H]
//   out_h   = sum_j w'_h(j) v_j                                  v of the head's own key/value head, h / (H / G)
//
// Position p sees the keys floor(p / chunk) * chunk .. p (chunk 0: all from 0 on), chunks counted from the
// request's first token; slopes may be null (no distance bias).  The mix needs every head's weight of a key,
// already divided by its sum, so maxima and sums come first and the weights after them.
// A cache page holds K as [G][page_size][D], then V as [G][D][page_size].
//
// Kernels:
//  * talking_sums_kernel + talking_prefill_kernel: bfloat16 on the matrix cores, heads of a multiple of 32 up to 128, up
//    to 32 heads, pages of a multiple of 16: requests of more than one token.  The first leaves every row's log of the
//    softmax's sum; in the second a workgroup takes 16 tokens of a request and ALL heads.
//  * talking_scores_kernel + talking_values_kernel: the same sizes, decoded tokens (any number of heads).
//  * talking_generic_kernel: any type and size.
#include "common.h"

LLE_DEFINE_ERROR_STRING()

struct TalkArgs {
    const void* q;     // [N, H, D]
    const void* kv;    // pages of one layer
    const int32_t* block_tables;
    const int32_t* seq_slots;
    const int32_t* cu_tokens;
    const int32_t* kv_lens;
    const int32_t* token_seq;
    void* out;         // [N, H, D]
    int H, G, D, P, max_pages, chunk;
    int P_log2;  // -1: the page size is no power of two
    int64_t page_stride;
    float scale;
    const float* slopes;  // [H] or null
    const float* talk;    // [H, H]
};

static int log2_or_minus_one(int n) {
    for (int i = 0; i < 31; ++i)
        if (n == 1 << i) return i;
    return -1;
}

// the page that key j lies in (pages of a power of two, the usual case, cost a shift instead of a division)
__device__ __forceinline__ int page_index(const TalkArgs& a, int j) { return a.P_log2 >= 0 ? j >> a.P_log2 : j / a.P; }

#define TK_KEYS 64

// scores of one tile of keys into LDS: s[h][j], -FLT_MAX past the row's last key
template <typename T>
__device__ __forceinline__ void talk_scores(const TalkArgs& a, const T* __restrict__ q, const int32_t* __restrict__ table,
                                            int j0, int pos, float* __restrict__ s) {
    const T* kv = (const T*)a.kv;
    const int group = a.H / a.G;
    for (int idx = threadIdx.x; idx < a.H * TK_KEYS; idx += blockDim.x) {
        const int h = idx / TK_KEYS, j = j0 + idx % TK_KEYS;
        float x = -FLT_MAX;
        if (j <= pos) {
            const int lp = j / a.P, off = j - lp * a.P;
            const T* k = kv + (int64_t)table[lp] * a.page_stride + ((int64_t)(h / group) * a.P + off) * a.D;
            const T* qh = q + (int64_t)h * a.D;
            float dot = 0.f;
            for (int e = 0; e < a.D; ++e) dot = fmaf(to_f32<T>(qh[e]), to_f32<T>(k[e]), dot);
            x = dot * a.scale;
            if (a.slopes) x -= a.slopes[h] * (float)(pos - j);
        }
        s[idx] = x;
    }
}

// any type and sizes: a workgroup per token; LDS holds s [H][TK_KEYS], w [H][TK_KEYS], acc [H][D], m [H], l [H]
template <typename T>
__global__ __launch_bounds__(256) void talking_generic_kernel(TalkArgs a) {
    extern __shared__ float lds[];
    float* s = lds;
    float* w = s + a.H * TK_KEYS;
    float* acc = w + a.H * TK_KEYS;
    float* m = acc + a.H * a.D;
    float* l = m + a.H;
    const int64_t tok = blockIdx.x;
    const int seq = a.token_seq[tok];
    const int q_start = a.cu_tokens[seq], q_len = a.cu_tokens[seq + 1] - q_start;
    const int pos = a.kv_lens[seq] - q_len + (int)(tok - q_start);
    const int lo = a.chunk > 0 ? pos / a.chunk * a.chunk : 0;
    const int32_t* table = a.block_tables + (int64_t)a.seq_slots[seq] * a.max_pages;
    const T* q = (const T*)a.q + tok * a.H * a.D;
    const T* kv = (const T*)a.kv;
    const int wave = threadIdx.x / LLE_WAVE, lane = threadIdx.x % LLE_WAVE, waves = blockDim.x / LLE_WAVE;
    const int group = a.H / a.G;
    for (int h = threadIdx.x; h < a.H; h += blockDim.x) {
        m[h] = -FLT_MAX;
        l[h] = 0.f;
    }
    for (int i = threadIdx.x; i < a.H * a.D; i += blockDim.x) acc[i] = 0.f;
    __syncthreads();
    for (int j0 = lo; j0 <= pos; j0 += TK_KEYS) {
        talk_scores<T>(a, q, table, j0, pos, s);
        __syncthreads();
        for (int h = wave; h < a.H; h += waves) {  // TK_KEYS lanes hold a head's tile
            const float x = s[h * TK_KEYS + lane];
            const float top = fmaxf(m[h], wave_max(x));
            const float sum = wave_sum(j0 + lane <= pos ? expf(x - top) : 0.f);
            if (lane == 0) {
                l[h] = l[h] * expf(m[h] - top) + sum;
                m[h] = top;
            }
        }
        __syncthreads();
    }
    for (int j0 = lo; j0 <= pos; j0 += TK_KEYS) {
        talk_scores<T>(a, q, table, j0, pos, s);
        __syncthreads();
        for (int idx = threadIdx.x; idx < a.H * TK_KEYS; idx += blockDim.x) {
            const int h = idx / TK_KEYS;
            s[idx] = j0 + idx % TK_KEYS <= pos ? expf(s[idx] - m[h]) / l[h] : 0.f;
        }
        __syncthreads();
        for (int idx = threadIdx.x; idx < a.H * TK_KEYS; idx += blockDim.x) {
            const int h = idx / TK_KEYS, j = idx % TK_KEYS;
            float x = 0.f;
            for (int g = 0; g < a.H; ++g) x = fmaf(a.talk[h * a.H + g], s[g * TK_KEYS + j], x);
            w[idx] = x;
        }
        __syncthreads();
        const int count = min(TK_KEYS, pos - j0 + 1);
        for (int i = threadIdx.x; i < a.H * a.D; i += blockDim.x) {
            const int h = i / a.D, e = i - h * a.D;
            const int64_t v_base = ((int64_t)a.G + h / group) * a.P * a.D + (int64_t)e * a.P;
            float x = acc[i];
            int lp = j0 / a.P, off = j0 - lp * a.P;
            const T* v = kv + (int64_t)table[lp] * a.page_stride + v_base;
            for (int j = 0; j < count; ++j) {
                x = fmaf(w[h * TK_KEYS + j], to_f32<T>(v[off]), x);
                if (++off == a.P && j + 1 < count) {
                    off = 0;
                    v = kv + (int64_t)table[++lp] * a.page_stride + v_base;
                }
            }
            acc[i] = x;
        }
        __syncthreads();
    }
    T* out = (T*)a.out + tok * a.H * a.D;
    for (int i = threadIdx.x; i < a.H * a.D; i += blockDim.x) out[i] = from_f32<T>(acc[i]);
}

// bytes of LDS that the generic kernel asks for (a caller refuses sizes that do not fit 160 KB)
extern "C" int lle_talking_generic_lds(int H, int D) { return (int)((2 * (int64_t)H * TK_KEYS + (int64_t)H * D + 2 * H) * sizeof(float)); }

extern "C" int lle_talking_generic(const void* q, const void* kv, const void* block_tables, const void* seq_slots,
                                   const void* cu_tokens, const void* kv_lens, const void* token_seq, void* out, int N, int H,
                                   int G, int D, int P, int64_t page_stride, int max_pages, int chunk, float scale,
                                   const void* slopes, const void* talk, int dtype, hipStream_t stream) {
    if (N <= 0) return 0;
    const int64_t smem = lle_talking_generic_lds(H, D);
    if (H <= 0 || G <= 0 || H % G != 0 || D <= 0 || P <= 0 || chunk < 0 || !talk || smem > 160 * 1024) return (int)hipErrorInvalidValue;
    const TalkArgs a{q, kv, (const int32_t*)block_tables, (const int32_t*)seq_slots, (const int32_t*)cu_tokens,
                     (const int32_t*)kv_lens, (const int32_t*)token_seq, out, H, G, D, P, max_pages, chunk, log2_or_minus_one(P), page_stride, scale,
                     (const float*)slopes, (const float*)talk};
    const void* fn = dtype == LLE_F32 ? (const void*)talking_generic_kernel<float> : (const void*)talking_generic_kernel<bf16_t>;
    if (smem > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
        if (e != hipSuccess) return (int)e;
    }
    if (dtype == LLE_F32) talking_generic_kernel<float><<<N, 256, smem, stream>>>(a);
    else talking_generic_kernel<bf16_t><<<N, 256, smem, stream>>>(a);
    LLE_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------
// matrix-core kernels (bfloat16)
// ---------------------------------------------------------------------------------
typedef bf16_t bf16x8 __attribute__((ext_vector_type(8)));
typedef bf16_t bf16x4 __attribute__((ext_vector_type(4)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x4 __attribute__((ext_vector_type(4)));
typedef _Float16 f16x2 __attribute__((ext_vector_type(2)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

#define NEG_BIG (-1.0e30f)
#define LOG2E 1.44269504088896340736f
// row r of tile x of a 32-key step stands for this key of the step: a lane's eight scores are consecutive keys then
#define KEY_OF_ROW(r, x) (8 * ((r) / 4) + 4 * (x) + (r) % 4)

// Decoded tokens, first launch: scores.  grid = (requests, G, key splits), four wavefronts; a wavefront takes every
// (4 x splits)-th tile of 16 keys.  ws_s [S][H][K] holds the base-2 scores from the 16-key tile on in which the chunk
// begins (NEG_BIG where the query does not see the key), ws_ml [S][H][K / 16] every tile's maximum and sum.
template <int DK>
__global__ __launch_bounds__(256) void talking_scores_kernel(TalkArgs a, float* __restrict__ ws_s, float2* __restrict__ ws_ml, int K) {
    constexpr int D = DK * 32;
    const int s = blockIdx.x, kvh = blockIdx.y;
    const int q_start = a.cu_tokens[s];
    if (a.cu_tokens[s + 1] - q_start != 1) return;
    const int pos = a.kv_lens[s] - 1;
    const int lo = a.chunk > 0 ? pos / a.chunk * a.chunk : 0, lo16 = lo & ~15;
    const int tiles = (pos - lo16) / 16 + 1;
    const int wave = threadIdx.x / LLE_WAVE, lane = threadIdx.x % LLE_WAVE, c = lane / 16, r16 = lane % 16;
    const int32_t* table = a.block_tables + (int64_t)a.seq_slots[s] * a.max_pages;
    const int group = a.H / a.G;
    const bf16_t* kv = (const bf16_t*)a.kv;
    for (int g0 = 0; g0 < group; g0 += 16) {  // 16 heads of the group at a time
        const int g = g0 + r16, h = kvh * group + g;
        const bool exists = g < group;
        bf16x8 qv[DK];
        const bf16_t* q = (const bf16_t*)a.q + ((int64_t)q_start * a.H + kvh * group + (exists ? g : g0)) * D;
#pragma unroll
        for (int ks = 0; ks < DK; ++ks) qv[ks] = *(const bf16x8*)(q + 32 * ks + 8 * c);
        const float slope = a.slopes && exists ? a.slopes[h] * LOG2E : 0.f;
        for (int tile = blockIdx.z * 4 + wave; tile < tiles; tile += 4 * gridDim.z) {
            const int j0 = lo16 + 16 * tile;
            const int lp = page_index(a, j0), off = j0 - lp * a.P;
            const bf16_t* k = kv + (int64_t)table[__builtin_amdgcn_readfirstlane(lp)] * a.page_stride +
                              ((int64_t)kvh * a.P + off + r16) * D + 8 * c;
            f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK; ++ks) sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(k + 32 * ks), qv[ks], sc, 0, 0, 0);
            float top = NEG_BIG;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int j = j0 + 4 * c + i;
                sc[i] = j < lo || j > pos ? NEG_BIG : fmaf(sc[i], a.scale * LOG2E, slope * (float)(j - pos));
                top = fmaxf(top, sc[i]);
            }
            top = fmaxf(top, __shfl_xor(top, 16, LLE_WAVE));
            top = fmaxf(top, __shfl_xor(top, 32, LLE_WAVE));
            float sum = 0.f;  // (every tile holds a key that the query sees: its maximum is a score)
#pragma unroll
            for (int i = 0; i < 4; ++i) sum += __builtin_amdgcn_exp2f(sc[i] - top);
            sum += __shfl_xor(sum, 16, LLE_WAVE);
            sum += __shfl_xor(sum, 32, LLE_WAVE);
            if (exists) {
                const int64_t row = (int64_t)s * a.H + h;
                *(f32x4*)(ws_s + row * K + 16 * tile + 4 * c) = sc;
                if (c == 0) ws_ml[row * (K / 16) + tile] = make_float2(top, sum);
            }
        }
    }
}

// Decoded tokens, second launch: weights, mix, values.  grid = (requests, G, blocks of 64 value elements), sixteen
// wavefronts.  1024 keys at a time: a thread makes one key's weights of all heads and mixes them for CNT query heads of
// the key/value head, the weights cross through LDS, and the values, asked for before that, are multiplied on the matrix
// cores: wavefront w takes elements 16 (w % 4) .. and keys 256 (w / 4) .. of them; the four shares meet in LDS.
#define TV_KEYS 1024
#define TV_ROW (TV_KEYS + 8)  // (rows of the weights in LDS: 16 bytes more, so that rows start in different banks)
template <int CNT>
__global__ __launch_bounds__(1024) void talking_values_kernel(TalkArgs a, const float* __restrict__ ws_s,
                                                              const float2* __restrict__ ws_ml, int K) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    bf16_t* s_w = (bf16_t*)lds;          // [CNT][TV_ROW], then the shares [4][CNT][64] in the same place
    float* s_m = lds + CNT * TV_ROW / 2;  // [H]
    float* s_t = s_m + a.H;               // [H][CNT]: talk / sum
    const int s = blockIdx.x, kvh = blockIdx.y;
    const int q_start = a.cu_tokens[s];
    if (a.cu_tokens[s + 1] - q_start != 1) return;
    const int pos = a.kv_lens[s] - 1;
    const int lo = a.chunk > 0 ? pos / a.chunk * a.chunk : 0, lo16 = lo & ~15;
    const int tiles = (pos - lo16) / 16 + 1;
    const int wave = threadIdx.x / LLE_WAVE, lane = threadIdx.x % LLE_WAVE, c = lane / 16, r16 = lane % 16;
    const int32_t* table = a.block_tables + (int64_t)a.seq_slots[s] * a.max_pages;
    const int group = a.H / a.G;
    const int e0 = blockIdx.z * 64 + (wave % 4) * 16, part = wave / 4;
    const bool has_values = e0 < a.D;  // (the same for the whole wavefront)
    const bf16_t* v_base = (const bf16_t*)a.kv + ((int64_t)a.G + kvh) * a.P * a.D + (int64_t)(has_values ? e0 + r16 : 0) * a.P;
    const float* s_row = ws_s + (int64_t)s * a.H * K;
    bf16x8 vv[8];
    auto load_v = [&](int b0) {
#pragma unroll
        for (int st = 0; st < 8; ++st) {  // keys past the last one read again: their weights are 0
            const int j = min(lo16 + b0 + 256 * part + 32 * st + 16 * (c / 2), lo16 + 16 * (tiles - 1));
            const int lp = page_index(a, j), off = j - lp * a.P;
            vv[st] = *(const bf16x8*)(v_base + (int64_t)table[lp] * a.page_stride + off + 8 * (c % 2));
        }
    };
    for (int g0 = 0; g0 < group; g0 += CNT) {
        const int count = min(CNT, group - g0);
        __syncthreads();
        for (int h = wave; h < a.H; h += 16) {
            const float2* ml = ws_ml + ((int64_t)s * a.H + h) * (K / 16);
            float top = NEG_BIG;
            for (int t = lane; t < tiles; t += LLE_WAVE) top = fmaxf(top, ml[t].x);
            top = wave_max(top);
            float sum = 0.f;
            for (int t = lane; t < tiles; t += LLE_WAVE) sum += ml[t].y * __builtin_amdgcn_exp2f(ml[t].x - top);
            sum = wave_sum(sum);
            if (lane == 0) s_m[h] = top;
            if (lane < CNT) s_t[h * CNT + lane] = lane < count ? a.talk[(kvh * group + g0 + lane) * a.H + h] / sum : 0.f;
        }
        __syncthreads();
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int b0 = 0; b0 < 16 * tiles; b0 += TV_KEYS) {
            const int key = b0 + threadIdx.x;
            float w[CNT];
#pragma unroll
            for (int i = 0; i < CNT; ++i) w[i] = 0.f;
            if (key < 16 * tiles) {
#pragma unroll 8
                for (int g = 0; g < a.H; ++g) {
                    const float p = __builtin_amdgcn_exp2f(s_row[(int64_t)g * K + key] - s_m[g]);
#pragma unroll
                    for (int i = 0; i < CNT; ++i) w[i] = fmaf(s_t[g * CNT + i], p, w[i]);  // (the same for all threads)
                }
            }
            load_v(b0);
            __syncthreads();  // (the keys before have been multiplied)
#pragma unroll
            for (int i = 0; i < CNT; ++i) s_w[i * TV_ROW + threadIdx.x] = (bf16_t)w[i];
            __syncthreads();
#pragma unroll
            for (int st = 0; st < 8; ++st) {
                const bf16x8 p = *(const bf16x8*)(s_w + (r16 % CNT) * TV_ROW + 256 * part + 32 * st + 8 * c);
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv[st], p, acc, 0, 0, 0);
            }
        }
        __syncthreads();
        float* s_o = lds;  // [4][CNT][64]
        if (r16 < CNT) *(f32x4*)(s_o + (part * CNT + r16) * 64 + (wave % 4) * 16 + 4 * c) = acc;
        __syncthreads();
        for (int i = threadIdx.x; i < count * 64; i += blockDim.x) {
            const int e = blockIdx.z * 64 + i % 64;
            if (e < a.D) {
                float o = 0.f;
#pragma unroll
                for (int p = 0; p < 4; ++p) o += s_o[p * CNT * 64 + i];
                ((bf16_t*)a.out)[((int64_t)q_start * a.H + kvh * group + g0 + i / 64) * a.D + e] = (bf16_t)o;
            }
        }
    }
}

// The tiles of 16 tokens in the order of their work, largest first: a tile's keys begin at its chunk's first, so the last
// tiles of all chunks come first.  `count` indices, some of them past the last tile (tile_order_count).
__host__ __device__ __forceinline__ int tile_order_count(int tiles, int chunk) {
    const int per = chunk > 0 ? (chunk + 15) / 16 : tiles;
    return per >= tiles ? tiles : (tiles + per - 1) / per * per;
}
__device__ __forceinline__ int tile_in_order(int k, int tiles, int chunk) {
    const int per = chunk > 0 ? (chunk + 15) / 16 : tiles;
    if (per >= tiles) return tiles - 1 - k;
    const int chunks = (tiles + per - 1) / per;
    return k % chunks * per + per - 1 - k / chunks;
}

// A barrier that waits for this wavefront's LDS traffic only: loads from memory stay on their way across it.
__device__ __forceinline__ void lds_barrier() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// Portions, first launch: the base-2 log of every row's sum, ws [N][H].  grid = (blocks of 16 tokens, G, requests), four
// wavefronts that take every fourth 32-key step; a wavefront makes the scores of TS_HEADS (a divisor of the group) of the
// key/value head's query heads with the keys in its registers, the others in further rounds.
#define TS_WAVES 4
template <int DK, int TS_HEADS>
__global__ __launch_bounds__(TS_WAVES* LLE_WAVE) void talking_sums_kernel(TalkArgs a, float* __restrict__ ws) {
    constexpr int D = DK * 32;
    __shared__ float s_m[TS_WAVES][TS_HEADS][16], s_l[TS_WAVES][TS_HEADS][16];
    const int s = blockIdx.z, kvh = blockIdx.y;
    const int q_start = a.cu_tokens[s], q_len = a.cu_tokens[s + 1] - q_start;
    if (q_len <= 1) return;
    const int tiles = (q_len + 15) / 16, order = tile_order_count(tiles, a.chunk);
    // (launches that are resident at once come two workgroups to a CU, halves of the launch side by side: the second half
    // takes its tiles the other way round)
    const int at = blockIdx.y < gridDim.y / 2 ? (int)blockIdx.x : order - 1 - (int)blockIdx.x;
    if (at < 0 || at >= order) return;
    const int t0 = tile_in_order(at, tiles, a.chunk) * 16;
    if (t0 >= q_len) return;
    const int past = a.kv_lens[s] - q_len;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / LLE_WAVE), lane = threadIdx.x % LLE_WAVE;
    const int c = lane / 16, r16 = lane % 16;
    const int32_t* table = a.block_tables + (int64_t)a.seq_slots[s] * a.max_pages;
    const int group = a.H / a.G, P = a.P;
    const bf16_t* kv = (const bf16_t*)a.kv;
    const int last = min(q_len, t0 + 16) - 1;
    const bool exists = t0 + r16 <= last;
    const int pos = exists ? past + t0 + r16 : -1;
    const int lo = exists && a.chunk > 0 ? pos / a.chunk * a.chunk : 0;
    const int key_lo = a.chunk > 0 ? (past + t0) / a.chunk * a.chunk : 0, key_hi = past + last;
    const int open_lo = a.chunk > 0 ? key_hi / a.chunk * a.chunk : 0, open_hi = past + t0;  // keys that every row sees
    const int first_step = key_lo / 32, end_step = key_hi / 32 + 1;
    const int half_lo = key_lo / 16, half_hi = key_hi / 16;
    const float scale = a.scale * LOG2E;
    bf16x8 kreg[2][DK];
    auto page_of = [&](int step) {
        const int j = min(max(2 * step + r16 / 8, half_lo), half_hi) * 16;
        return table[page_index(a, j)];
    };
    auto load_k = [&](int step, int page) {
        const int j = min(max(2 * step + r16 / 8, half_lo), half_hi) * 16;
        const bf16_t* k = kv + (int64_t)page * a.page_stride + ((int64_t)kvh * P + (j - page_index(a, j) * P)) * D + 8 * c;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int ks = 0; ks < DK; ++ks) kreg[x][ks] = *(const bf16x8*)(k + (int64_t)(KEY_OF_ROW(r16, x) % 16) * D + 32 * ks);
    };
    for (int g0 = 0; g0 < group; g0 += TS_HEADS) {
        bf16x8 qv[TS_HEADS][DK];
        float slope[TS_HEADS], m[TS_HEADS], l[TS_HEADS];
#pragma unroll
        for (int i = 0; i < TS_HEADS; ++i) {
            const int h = kvh * group + g0 + i;
            const bf16_t* q = (const bf16_t*)a.q + ((int64_t)(q_start + min(t0 + r16, last)) * a.H + h) * D + 8 * c;
#pragma unroll
            for (int ks = 0; ks < DK; ++ks) qv[i][ks] = *(const bf16x8*)(q + 32 * ks);
            slope[i] = a.slopes ? a.slopes[h] * LOG2E : 0.f;
            m[i] = NEG_BIG;
            l[i] = 0.f;
        }
        int page = page_of(first_step + wave);
        load_k(first_step + wave, page);
        page = page_of(first_step + wave + TS_WAVES);
        for (int step = first_step + wave; step < end_step; step += TS_WAVES) {
            f32x4 sc[TS_HEADS][2];
#pragma unroll
            for (int i = 0; i < TS_HEADS; ++i) {
                sc[i][0] = sc[i][1] = f32x4{0.f, 0.f, 0.f, 0.f};
            }
            // (products that wait for one another stand apart)
#pragma unroll
            for (int ks = 0; ks < DK; ++ks)
#pragma unroll
                for (int i = 0; i < TS_HEADS; ++i)
#pragma unroll
                    for (int t = 0; t < 2; ++t)
                        sc[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kreg[t][ks], qv[i][ks], sc[i][t], 0, 0, 0);
            load_k(step + TS_WAVES, page);  // (past the last step: keys that are there)
            page = page_of(step + 2 * TS_WAVES);
            const bool open = 32 * step >= open_lo && 32 * step + 31 <= open_hi;  // (the same for all lanes)
            const float d0 = (float)(32 * step + 8 * c - pos);
#pragma unroll
            for (int i = 0; i < TS_HEADS; ++i) {
                float x[8], top = m[i];
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = fmaf(sc[i][e / 4][e % 4], scale, slope[i] * (d0 + (float)e));
                if (!open) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        const int j = 32 * step + 8 * c + e;
                        if (j < lo || j > pos) x[e] = NEG_BIG;
                    }
                }
#pragma unroll
                for (int e = 0; e < 8; ++e) top = fmaxf(top, x[e]);
                const float base = top <= NEG_BIG ? 0.f : top;
                float sum = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) sum += __builtin_amdgcn_exp2f(x[e] - base);
                l[i] = l[i] * __builtin_amdgcn_exp2f(m[i] - base) + sum;
                m[i] = top;
            }
        }
        __syncthreads();  // (the round before has been read)
#pragma unroll
        for (int i = 0; i < TS_HEADS; ++i) {
            float top = fmaxf(m[i], __shfl_xor(m[i], 16, LLE_WAVE));
            top = fmaxf(top, __shfl_xor(top, 32, LLE_WAVE));
            const float base = top <= NEG_BIG ? 0.f : top;
            float sum = l[i] * __builtin_amdgcn_exp2f(m[i] - base);
            sum += __shfl_xor(sum, 16, LLE_WAVE);
            sum += __shfl_xor(sum, 32, LLE_WAVE);
            if (c == 0) {
                s_m[wave][i][r16] = top;
                s_l[wave][i][r16] = sum;
            }
        }
        __syncthreads();
        if (threadIdx.x < TS_HEADS * 16) {
            const int i = threadIdx.x / 16, r = threadIdx.x % 16;
            if (t0 + r <= last) {
                float top = s_m[0][i][r];
#pragma unroll
                for (int w = 1; w < TS_WAVES; ++w) top = fmaxf(top, s_m[w][i][r]);
                float sum = 0.f;  // (a row sees a key: itself)
#pragma unroll
                for (int w = 0; w < TS_WAVES; ++w) sum += s_l[w][i][r] * __builtin_amdgcn_exp2f(s_m[w][i][r] - top);
                ws[(int64_t)(q_start + t0 + r) * a.H + kvh * group + g0 + i] = top + log2f(sum);
            }
        }
    }
}

// Portions, second launch.  grid = (output splits, blocks of 16 tokens, requests), eight wavefronts.  A wavefront makes the
// scores of HW heads for XT of a step's two 16-key tiles (all of the model's heads over the eight wavefronts), one query
// token a lane column, so that with ONE key/value head for the HW heads nobody reads a key twice.  Three things happen in
// step i, each to another 32 keys, with one barrier a step between them:
//   keys i      scores, weights (divided by their sum already, so between 0 and 1) into LDS in half precision (11 bits of
//               mantissa, three more than the mixed weights keep), [key][token][head];
//   keys i - 1  mixed on the matrix cores ([4 tokens x 4 keys] x heads times heads x 16 heads of this workgroup's
//               split; talk in half precision holds a bfloat16 number as it is), summed in 32-bit, [token][head][key] into
//               LDS as bfloat16;
//   keys i - 2  O^T += V^T W^T: a wavefront takes BH heads of one key/value head and the value elements of its share (the
//               wavefronts that have the same heads share the elements, so nobody reads a value twice).
// Both LDS buffers are there twice.  A split computes all scores and the sums of 8 OW output heads: OW bounds the
// accumulators.  LDS rows of 64 bytes are cut into four 16-byte pieces whose order is swizzled so that neither the writes nor
// the reads of the two exchanges meet in a bank.
#define TALK_P_BYTES (512 * 64)      // 32 keys x 16 tokens, rows of 32 heads
#define TALK_W_BYTES (16 * 16 * 64)  // 16 tokens x 16 heads, rows of 32 keys
__device__ __forceinline__ int talk_p_at(int key, int q, int piece) {  // byte offset of a 16-byte piece of a weight row
    return (key * 16 + q) * 64 + ((piece ^ (q >> 2) ^ key) & 3) * 16;
}
__device__ __forceinline__ int talk_w_at(int q, int h, int piece) {  // of a mixed-weight row (32 keys)
    const int row = h ^ q;
    return (q * 16 + row) * 64 + ((piece ^ (row >> 2)) & 3) * 16;
}

// (ONE: a load under a condition makes the compiler wait for every load on its way where the paths meet again, so the usual
// case has none; loads past the last step ask for keys that are there.)
template <int DK, int HW, int XT, int OW, int BH, bool ONE>
__global__ __launch_bounds__(512) void talking_prefill_kernel(TalkArgs a, const float* __restrict__ sums) {
    constexpr int D = DK * 32;
    constexpr int P_BYTES = TALK_P_BYTES, W_BYTES = TALK_W_BYTES;
    constexpr int BUNDLES = 4 * XT;                   // of HW heads: eight wavefronts, or four for either key tile
    constexpr int WB = BH / OW, TN = 2 * DK / WB;     // wavefronts that share BH output heads, and their tiles of value elements
    static_assert(BH % OW == 0 && 2 * DK % WB == 0, "the value elements are dealt to the wavefronts in equal shares");
    extern __shared__ __attribute__((aligned(16))) char smem[];
    char* s_p = smem;
    char* s_w = smem + 2 * P_BYTES;
    const int s = blockIdx.z, out0 = blockIdx.x * 8 * OW;
    const int q_start = a.cu_tokens[s], q_len = a.cu_tokens[s + 1] - q_start;
    if (q_len <= 1) return;
    const int tiles = (q_len + 15) / 16;
    if ((int)blockIdx.y >= tile_order_count(tiles, a.chunk)) return;
    const int t0 = tile_in_order(blockIdx.y, tiles, a.chunk) * 16;
    if (t0 >= q_len) return;
    const int past = a.kv_lens[s] - q_len;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / LLE_WAVE), lane = threadIdx.x % LLE_WAVE;
    const int c = lane / 16, r16 = lane % 16;
    const int32_t* table = a.block_tables + (int64_t)a.seq_slots[s] * a.max_pages;
    const int group = a.H / a.G, P = a.P;
    const bf16_t* kv = (const bf16_t*)a.kv;
    const int last = min(q_len, t0 + 16) - 1;
    const bool exists = t0 + r16 <= last;
    const int pos = exists ? past + t0 + r16 : -1;
    const int lo = exists && a.chunk > 0 ? pos / a.chunk * a.chunk : 0;
    const int key_lo = a.chunk > 0 ? (past + t0) / a.chunk * a.chunk : 0, key_hi = past + last;  // of all rows
    const int open_lo = a.chunk > 0 ? key_hi / a.chunk * a.chunk : 0, open_hi = exists ? past + t0 : -1;
    const int first_step = key_lo / 32, steps = key_hi / 32 + 1 - first_step;
    const int half_lo = key_lo / 16, half_hi = key_hi / 16;  // 16-key halves that hold keys: others may have no page
    const int h0 = wave % BUNDLES * HW, x0 = XT == 1 ? wave / BUNDLES : 0;  // (x0: the wavefront's first key tile)
    const int heads_here = max(0, min(HW, a.H - h0));  // (the same for the whole wavefront)
    const bool all_rows = last - t0 == 15;

    // weights of heads that do not exist stay zero
    for (int i = threadIdx.x; i < 2 * P_BYTES / 16; i += 512) ((uint4*)s_p)[i] = make_uint4(0, 0, 0, 0);

    bf16x8 qv[HW][DK];
    float slope[HW], sum[HW];
#pragma unroll
    for (int i = 0; i < HW; ++i) {
        const int h = min(h0 + i, a.H - 1);
        const int64_t tok = q_start + min(t0 + r16, last);
        const bf16_t* q = (const bf16_t*)a.q + (tok * a.H + h) * D + 8 * c;
#pragma unroll
        for (int ks = 0; ks < DK; ++ks) qv[i][ks] = *(const bf16x8*)(q + 32 * ks);
        slope[i] = a.slopes ? a.slopes[h] * LOG2E : 0.f;
        sum[i] = sums[tok * a.H + h];
    }
    const float scale = a.scale * LOG2E;

    // output heads and value elements of this wavefront (heads of a bundle are all there or none is)
    const int oh_local = wave / WB * BH, oh0 = out0 + oh_local, v_tile0 = wave % WB * TN;
    const bool has_outs = oh0 < a.H;

    // a step's two 16-key halves lie in one page each; a lane's keys lie in half r16 / 8, its values' keys in half c / 2
    const int k_half = r16 / 8, v_half = c / 2;
    auto key_of = [&](int i, int half) { return min(max(2 * (first_step + i) + half, half_lo), half_hi) * 16; };
    auto page_of = [&](int i, int half) { return table[page_index(a, key_of(i, half))]; };
    bf16x8 kreg[XT][DK], vreg[TN];
    auto load_k = [&](int i, int page, int kvh) {
        const int j = key_of(i, k_half);
        const bf16_t* k = kv + (int64_t)page * a.page_stride + ((int64_t)kvh * P + (j - page_index(a, j) * P)) * D + 8 * c;
#pragma unroll
        for (int x = 0; x < XT; ++x)
#pragma unroll
            for (int ks = 0; ks < DK; ++ks) kreg[x][ks] = *(const bf16x8*)(k + (int64_t)(KEY_OF_ROW(r16, x0 + x) % 16) * D + 32 * ks);
    };
    auto load_v = [&](int i, int page, int kvh) {
        const int j = key_of(i, v_half);
        const bf16_t* v = kv + (int64_t)page * a.page_stride + ((int64_t)a.G + kvh) * P * D + (int64_t)(v_tile0 * 16 + r16) * P + (j - page_index(a, j) * P) + 8 * (c % 2);
#pragma unroll
        for (int n = 0; n < TN; ++n) vreg[n] = *(const bf16x8*)(v + (int64_t)16 * n * P);
    };

    // talk's rows of this split's heads: element e of lane (c, r16) is talk[out0 + r16][8 c + e]
    f16x8 talk;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        const int g = 8 * c + e, h = out0 + r16;
        talk[e] = (_Float16)(r16 < 8 * OW && h < a.H && g < a.H ? a.talk[h * a.H + g] : 0.f);
    }
    const int first_kvh = min(h0, a.H - 1) / group, first_vkv = min(oh0, a.H - 1) / group;
    f32x4 o[BH][TN];
#pragma unroll
    for (int i = 0; i < BH; ++i)
#pragma unroll
        for (int n = 0; n < TN; ++n) o[i][n] = f32x4{0.f, 0.f, 0.f, 0.f};

    // a page is looked up one step before its keys or values are asked for, these one step before they are used
    int k_page = page_of(0, k_half), k_page_now = k_page, v_page = page_of(0, v_half);
    load_k(0, k_page, first_kvh);
    k_page = page_of(1, k_half);
    __syncthreads();  // (the zeros are there)
    for (int i = 0; i < steps + 2; ++i) {
        if (i < steps && heads_here > 0) {
            const int step = first_step + i;
            _Float16 p[4 * XT][HW];
            [[maybe_unused]] int kvh = first_kvh;
            const bool open = all_rows && 32 * step >= open_lo && 32 * step + 31 <= past + t0;  // (the same for all lanes)
            const int j0 = 32 * step + 8 * c + 4 * x0;
            const float d0 = (float)(j0 - pos);
            // SG heads at a time: products that wait for one another stand apart, and their sums fit the registers
            constexpr int SG = ONE ? (HW * XT > 4 ? HW / 2 : HW) : 1;
#pragma unroll
            for (int n0 = 0; n0 < HW; n0 += SG) {
                f32x4 sc[SG][XT];
                if constexpr (!ONE) {
                    const int own = min(h0 + n0, a.H - 1) / group;
                    if (own != kvh) load_k(i, k_page_now, kvh = own);
                }
#pragma unroll
                for (int ks = 0; ks < DK; ++ks)
#pragma unroll
                    for (int n = 0; n < SG; ++n)
#pragma unroll
                        for (int t = 0; t < XT; ++t)
                            sc[n][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                                kreg[t][ks], qv[n0 + n][ks], ks == 0 ? f32x4{0.f, 0.f, 0.f, 0.f} : sc[n][t], 0, 0, 0);
#pragma unroll
                for (int n = 0; n < SG; ++n) {
                    float x[4 * XT];
#pragma unroll
                    for (int e = 0; e < 4 * XT; ++e)
                        x[e] = fmaf(sc[n][e / 4][e % 4], scale, fmaf(slope[n0 + n], d0 + (float)e, -sum[n0 + n]));
                    if (!open) {
#pragma unroll
                        for (int e = 0; e < 4 * XT; ++e)
                            if (j0 + e < lo || j0 + e > pos) x[e] = NEG_BIG;
                    }
                    // (heads that do not exist leave zeros)
#pragma unroll
                    for (int e = 0; e < 4 * XT; ++e)
                        p[e][n0 + n] = n0 + n < heads_here ? (_Float16)__builtin_amdgcn_exp2f(x[e]) : (_Float16)0.f;
                }
            }
            char* buf = s_p + (i & 1) * P_BYTES;
#pragma unroll
            for (int e = 0; e < 4 * XT; ++e) {
                char* at = buf + talk_p_at(8 * c + 4 * x0 + e, r16, h0 / 8) + (h0 % 8) * 2;
                if constexpr (HW == 1) *(_Float16*)at = p[e][0];
                else if constexpr (HW == 2) *(f16x2*)at = f16x2{p[e][0], p[e][1]};
                else *(f16x4*)at = f16x4{p[e][0], p[e][1], p[e][2], p[e][3]};
            }
        }
        load_k(i + 1, k_page, first_kvh);
        k_page_now = k_page;
        k_page = page_of(i + 2, k_half);
        if (i >= 1 && i - 1 < steps) {
            // 32 tiles of (4 tokens x 4 keys), four a wavefront: row r of a tile is token 4 qa + r / 4, key 4 kq + r % 4
            const char* from = s_p + ((i - 1) & 1) * P_BYTES;
            char* to = s_w + ((i - 1) & 1) * W_BYTES;
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const int tile = wave * 4 + t, qa = tile % 4, kq = tile / 4;
                const f16x8 p = *(const f16x8*)(from + talk_p_at(4 * kq + r16 % 4, 4 * qa + r16 / 4, c));
                const f32x4 w = __builtin_amdgcn_mfma_f32_16x16x32_f16(p, talk, f32x4{0.f, 0.f, 0.f, 0.f}, 0, 0, 0);
                // lane (c, r16): head r16 of the split, token 4 qa + c, keys 4 kq .. + 3
                *(bf16x4*)(to + talk_w_at(4 * qa + c, r16, kq / 2) + (kq % 2) * 8) = bf16x4{(bf16_t)w[0], (bf16_t)w[1], (bf16_t)w[2], (bf16_t)w[3]};
            }
        }
        if (i >= 2 && has_outs) {
            const char* from = s_w + (i & 1) * W_BYTES;
            bf16x8 w[BH];
#pragma unroll
            for (int n = 0; n < BH; ++n) w[n] = *(const bf16x8*)(from + talk_w_at(r16, oh_local + n, c));
#pragma unroll
            for (int n = 0; n < BH; ++n)
#pragma unroll
                for (int m = 0; m < TN; ++m) o[n][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vreg[m], w[n], o[n][m], 0, 0, 0);
        }
        load_v(i - 1, v_page, first_vkv);  // used in the next step
        v_page = page_of(i, v_half);
        lds_barrier();
    }
    if (!exists || !has_outs) return;
#pragma unroll
    for (int i = 0; i < BH; ++i) {
        bf16_t* dst = (bf16_t*)a.out + ((int64_t)(q_start + t0 + r16) * a.H + oh0 + i) * D + 16 * v_tile0 + 4 * c;
#pragma unroll
        for (int n = 0; n < TN; ++n)
            *(bf16x4*)(dst + 16 * n) = bf16x4{(bf16_t)o[i][n][0], (bf16_t)o[i][n][1], (bf16_t)o[i][n][2], (bf16_t)o[i][n][3]};
    }
}

template <int DK, int HW, int XT, int OW, int BH, bool ONE>
static int talk_prefill_launch(const TalkArgs& a, int S, int max_q_len, const float* sums, hipStream_t stream) {
    const size_t smem = 2 * (TALK_P_BYTES + TALK_W_BYTES);
    if (smem > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute((const void*)talking_prefill_kernel<DK, HW, XT, OW, BH, ONE>,
                                           hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
        if (e != hipSuccess) return (int)e;
    }
    const int splits = (a.H + 8 * OW - 1) / (8 * OW);
    talking_prefill_kernel<DK, HW, XT, OW, BH, ONE><<<dim3(splits, tile_order_count((max_q_len + 15) / 16, a.chunk), S), 512, smem, stream>>>(a, sums);
    return (int)hipGetLastError();
}

// Which form of the kernel takes a model's heads: how many there are, and how many neighbours share a key/value head.  (More
// than 16 heads: one output head a wavefront, four splits.  Two of them need more registers than two wavefronts a SIMD have,
// and what spills costs more than the scores made twice as often: 202 against 113 us for 2048 tokens, 32 heads.)
template <int DK>
static int talk_prefill(const TalkArgs& a, int S, int max_q_len, int out_heads, float* sums, hipStream_t stream) {
    const int group = a.H / a.G;
    const dim3 grid(tile_order_count((max_q_len + 15) / 16, a.chunk), a.G, S);
    if (group % 4 == 0) talking_sums_kernel<DK, 4><<<grid, TS_WAVES * LLE_WAVE, 0, stream>>>(a, sums);
    else if (group % 2 == 0) talking_sums_kernel<DK, 2><<<grid, TS_WAVES * LLE_WAVE, 0, stream>>>(a, sums);
    else talking_sums_kernel<DK, 1><<<grid, TS_WAVES * LLE_WAVE, 0, stream>>>(a, sums);
    const hipError_t e = hipGetLastError();
    if (e != hipSuccess) return (int)e;
#define LLE_TALK(HW, XT, OW, BH, ONE) return talk_prefill_launch<DK, HW, XT, OW, BH, ONE>(a, S, max_q_len, sums, stream)
    if (group % 4 == 0) {
        constexpr int BH1 = DK % 2 == 0 ? 4 : 2;  // (four heads over four wavefronts: an even number of element blocks)
        if (a.H <= 8) LLE_TALK(2, 1, 1, BH1, true);
        if (a.H <= 16) {
            if (out_heads == 1) LLE_TALK(4, 1, 1, BH1, true);
            LLE_TALK(4, 1, 2, 4, true);
        }
        LLE_TALK(4, 2, 1, BH1, true);
    }
    if (group % 2 == 0) {
        if (a.H <= 8) LLE_TALK(2, 1, 1, 2, true);
        if (a.H <= 16) {
            if (out_heads == 1) LLE_TALK(2, 2, 1, 2, true);
            LLE_TALK(2, 2, 2, 2, true);
        }
        LLE_TALK(4, 2, 1, 2, false);
    }
    if (a.H <= 8) LLE_TALK(1, 2, 1, 1, true);
    if (a.H <= 16) LLE_TALK(2, 2, 1, 1, false);
    LLE_TALK(4, 2, 1, 1, false);
#undef LLE_TALK
}

template <int DK>
static int talk_launch(const TalkArgs& a, int S, int run_decode, int splits, int K, float* ws_s, float2* ws_ml, int run_prefill,
                       int max_q_len, int out_heads, float* ws_sums, hipStream_t stream) {
    if (run_decode) {
        talking_scores_kernel<DK><<<dim3(S, a.G, splits), 256, 0, stream>>>(a, ws_s, ws_ml, K);
        hipError_t e = hipGetLastError();
        if (e != hipSuccess) return (int)e;
        const int group = a.H / a.G;
        const dim3 grid(S, a.G, (a.D + 63) / 64);
        auto values = [&](auto kernel, int cnt) {
            const size_t smem = (size_t)cnt * TV_ROW * sizeof(bf16_t) + (size_t)a.H * (1 + cnt) * sizeof(float);
            if (smem > 64 * 1024) return hipErrorInvalidValue;
            kernel<<<grid, 1024, smem, stream>>>(a, (const float*)ws_s, (const float2*)ws_ml, K);
            return hipGetLastError();
        };
        if (group == 1) e = values(talking_values_kernel<1>, 1);
        else if (group == 2) e = values(talking_values_kernel<2>, 2);
        else if (group <= 4) e = values(talking_values_kernel<4>, 4);
        else if (group <= 8) e = values(talking_values_kernel<8>, 8);
        else e = values(talking_values_kernel<16>, 16);
        if (e != hipSuccess) return (int)e;
    }
    if (run_prefill) {
        return talk_prefill<DK>(a, S, max_q_len, out_heads, ws_sums, stream);
    }
    return 0;
}

// bfloat16, D 32, 64, 96 or 128, pages of a multiple of 16 keys; with run_prefill up to 32 heads.  run_decode: the batch
// holds requests of one token (ws_s float32 [S H K], ws_ml float32 [S H K / 8]; K a multiple of 16, at least 15 more than
// the keys that a query sees); run_prefill: it holds longer ones.  ws_sums float32
// [N H].  out_heads: output heads a wavefront sums up where both forms are there (9 to 16 heads), 1 or 2.
extern "C" int lle_talking_mfma(const void* q, const void* kv, const void* block_tables, const void* seq_slots,
                                const void* cu_tokens, const void* kv_lens, const void* token_seq, void* out, int S, int H, int G,
                                int D, int P, int64_t page_stride, int max_pages, int chunk, float scale, const void* slopes,
                                const void* talk, int run_decode, int splits, int K, void* ws_s, void* ws_ml, int run_prefill,
                                int max_q_len, int out_heads, void* ws_sums, hipStream_t stream) {
    if (S <= 0) return 0;
    if (H <= 0 || G <= 0 || H % G != 0 || D % 32 != 0 || D <= 0 || D > 128 || P % 16 != 0 || P <= 0 || chunk < 0 || !talk ||
        S > 65535 || G > 65535)
        return (int)hipErrorInvalidValue;
    if (run_decode && (!ws_s || !ws_ml || K % 16 != 0 || K < 16 || splits < 1 || splits > 65535)) return (int)hipErrorInvalidValue;
    if (run_prefill && (H > 32 || max_q_len < 2 || !ws_sums || tile_order_count((max_q_len + 15) / 16, chunk) > 65535)) return (int)hipErrorInvalidValue;
    const TalkArgs a{q, kv, (const int32_t*)block_tables, (const int32_t*)seq_slots, (const int32_t*)cu_tokens,
                     (const int32_t*)kv_lens, (const int32_t*)token_seq, out, H, G, D, P, max_pages, chunk, log2_or_minus_one(P), page_stride, scale,
                     (const float*)slopes, (const float*)talk};
    switch (D / 32) {
        case 1: return talk_launch<1>(a, S, run_decode, splits, K, (float*)ws_s, (float2*)ws_ml, run_prefill, max_q_len, out_heads, (float*)ws_sums, stream);
        case 2: return talk_launch<2>(a, S, run_decode, splits, K, (float*)ws_s, (float2*)ws_ml, run_prefill, max_q_len, out_heads, (float*)ws_sums, stream);
        case 3: return talk_launch<3>(a, S, run_decode, splits, K, (float*)ws_s, (float2*)ws_ml, run_prefill, max_q_len, out_heads, (float*)ws_sums, stream);
        case 4: return talk_launch<4>(a, S, run_decode, splits, K, (float*)ws_s, (float2*)ws_ml, run_prefill, max_q_len, out_heads, (float*)ws_sums, stream);
    }
    return (int)hipErrorInvalidValue;
}
