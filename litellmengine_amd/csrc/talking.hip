// Attention over the paged cache whose heads' weights are mixed before they meet the values:
//
//   s_h(j)  = (q_h . k_j) * scale - slope_h (p - j)             j of the query's own chunk, j <= p
//   w_h(j)  = softmax over j
//   w'_h(j) = sum_g talk[h, g] w_g(j)                            talk float32 [H, H]
//   out_h   = sum_j w'_h(j) v_j                                  v of the head's own key/value head, h / (H / G)
//
// Position p sees the keys floor(p / chunk) * chunk .. p (chunk 0: all from 0 on), chunks counted from the
// request's first token; slopes may be null (no distance bias).  The mix needs every head's weight of a key,
// already divided by its sum, so scores are made twice: once for the rows' maxima and sums, once for the weights.
// A cache page holds K as [G][page_size][D], then V as [G][D][page_size].
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
    int64_t page_stride;
    float scale;
    const float* slopes;  // [H] or null
    const float* talk;    // [H, H]
};

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
                     (const int32_t*)kv_lens, (const int32_t*)token_seq, out, H, G, D, P, max_pages, chunk, page_stride, scale,
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
