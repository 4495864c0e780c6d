// RMSNorm fused with the residual add (and, for the first norm of a model, with the embedding).
// Reference counterparts: rms_norm_forward_kernel (src/layers/rms_norm.cu:97-141)
// and add_fp32_kernel (src/ops/add.cu:16-27), two launches there.
//
//   h = hidden[row] (+ delta[row])          32-bit sum, the residual stream
//   out[r] = h * rsqrt(mean(h^2) + eps) * w
// With `rows == nullptr` row r is r and h is written back to `hidden`; with a
// row list (the output head: only the wanted rows) nothing is written back.
#include "common.h"

LLE_DEFINE_ERROR_STRING()

template <typename T>
__global__ __launch_bounds__(1024) void add_rmsnorm_kernel(float* __restrict__ hidden, const T* __restrict__ delta,
                                                            const int32_t* __restrict__ rows,
                                                            const void* __restrict__ weight, int weight_dtype,
                                                            T* __restrict__ out, int H, float eps) {
    __shared__ float red[16];
    const int64_t r = blockIdx.x;
    const int64_t row = rows ? (int64_t)rows[r] : r;
    float* h = hidden + row * H;
    const T* dl = delta ? delta + row * H : nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = h[i];
        if (dl) v += to_f32<T>(dl[i]);
        if (!rows && dl) h[i] = v;
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps);
    T* o = out + r * H;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = h[i];
        if (rows && dl) v += to_f32<T>(dl[i]);
        o[i] = from_f32<T>(v * inv * load_as_f32(weight, i, weight_dtype));
    }
}

// four consecutive elements of either type as 32-bit floats
template <typename T> struct Quad;
template <> struct Quad<float> {
    static __device__ __forceinline__ float4 load(const float* p) { return *(const float4*)p; }
    static __device__ __forceinline__ void store(float* p, float4 v) { *(float4*)p = v; }
};
template <> struct Quad<bf16_t> {
    typedef bf16_t vec __attribute__((ext_vector_type(4)));
    static __device__ __forceinline__ float4 load(const bf16_t* p) {
        const vec v = *(const vec*)p;
        return make_float4((float)v[0], (float)v[1], (float)v[2], (float)v[3]);
    }
    static __device__ __forceinline__ void store(bf16_t* p, float4 v) {
        *(vec*)p = vec{(bf16_t)v.x, (bf16_t)v.y, (bf16_t)v.z, (bf16_t)v.w};
    }
};

__device__ __forceinline__ float4 load_weight4(const void* w, int64_t i, int dtype) {
    return dtype == LLE_F32 ? Quad<float>::load((const float*)w + i) : Quad<bf16_t>::load((const bf16_t*)w + i);
}

// The same sums in one pass for rows of up to 256 * 4 * NORM_CHUNKS elements (a multiple of 4):
// every thread keeps its part of the row in registers between the sum and the scaling.
#define NORM_CHUNKS 8
// `delta` may come as `slices` partial sums of type TD, `slice_stride` elements apart (a product
// over slices of K leaves them so): they are added in slice order.
template <typename T, typename TD = T, bool SLICED = false>
__global__ __launch_bounds__(256) void add_rmsnorm_vec_kernel(float* __restrict__ hidden, const TD* __restrict__ delta,
                                                              const int32_t* __restrict__ rows,
                                                              const void* __restrict__ weight, int weight_dtype,
                                                              T* __restrict__ out, int H, float eps, int slices = 1,
                                                              int64_t slice_stride = 0) {
    __shared__ float red[16];
    const int64_t r = blockIdx.x;
    const int64_t row = rows ? (int64_t)rows[r] : r;
    float* h = hidden + row * H;
    const TD* dl = delta ? delta + row * H : nullptr;
    float4 v[NORM_CHUNKS], wv[NORM_CHUNKS];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NORM_CHUNKS; ++k) {  // the weights do not wait for the sum
        const int i = (k * 256 + threadIdx.x) * 4;
        if (i < H) wv[k] = load_weight4(weight, i, weight_dtype);
    }
    if constexpr (SLICED) {
        // all of a row's loads of one kind are asked for together (a load that waits for the one before
        // it pays the memory's latency once more): the row and the first slice, then slice by slice
        float4 d[NORM_CHUNKS];
    #pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                v[k] = *(const float4*)(h + i);
                if (dl) d[k] = Quad<TD>::load(dl + i);
            }
        }
        if (dl) {
    #pragma unroll 2
            for (int sl = 1; sl < slices; ++sl) {
                float4 e[NORM_CHUNKS];
    #pragma unroll
                for (int k = 0; k < NORM_CHUNKS; ++k) {
                    const int i = (k * 256 + threadIdx.x) * 4;
                    if (i < H) e[k] = Quad<TD>::load(dl + sl * slice_stride + i);
                }
    #pragma unroll
                for (int k = 0; k < NORM_CHUNKS; ++k) {
                    const int i = (k * 256 + threadIdx.x) * 4;
                    if (i < H) {
                        d[k].x += e[k].x;
                        d[k].y += e[k].y;
                        d[k].z += e[k].z;
                        d[k].w += e[k].w;
                    }
                }
            }
        }
    #pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                float4 x = v[k];
                if (dl) {
                    x.x += d[k].x;
                    x.y += d[k].y;
                    x.z += d[k].z;
                    x.w += d[k].w;
                    if (!rows) *(float4*)(h + i) = x;
                }
                v[k] = x;
                ss += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
            }
        }
    } else {
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                float4 x = *(const float4*)(h + i);
                if (dl) {
                    const float4 d = Quad<TD>::load(dl + i);
                    x.x += d.x;
                    x.y += d.y;
                    x.z += d.z;
                    x.w += d.w;
                    if (!rows) *(float4*)(h + i) = x;
                }
                v[k] = x;
                ss += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
            }
        }
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps);
    T* o = out + r * H;
#pragma unroll
    for (int k = 0; k < NORM_CHUNKS; ++k) {
        const int i = (k * 256 + threadIdx.x) * 4;
        if (i < H) {
            const float4 w = wv[k];
            Quad<T>::store(o + i, make_float4(v[k].x * inv * w.x, v[k].y * inv * w.y, v[k].z * inv * w.z,
                                              v[k].w * inv * w.w));
        }
    }
}

// hidden += sums[0] + sums[1] + ... (float32 [slices][N][H], rows of hidden and of a slice alike), then
// the norm as lle_add_rmsnorm; H a multiple of 4 up to 256 * 4 * NORM_CHUNKS
// The first rows of the residual stream and their first norm in one launch: hidden[n] =
// table[id(n)] as 32-bit (the embedding, src/layers/embedding.cu:75-87), out[n] its RMSNorm.
// An id below zero stands for feedback[seq_slots[token_seq[n]]] (the token that the step before
// picked for the row's request and left on the device), as in the embedding kernel itself.
// VEC: rows of a multiple of 4 and at most 256 * 4 * NORM_CHUNKS elements, kept in registers.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void embedding_rmsnorm_kernel(const int32_t* __restrict__ ids,
                                                                const T* __restrict__ table,
                                                                float* __restrict__ hidden,
                                                                const void* __restrict__ weight, int weight_dtype,
                                                                T* __restrict__ out, int H, float eps,
                                                                const int32_t* __restrict__ feedback,
                                                                const int32_t* __restrict__ token_seq,
                                                                const int32_t* __restrict__ seq_slots) {
    __shared__ float red[16];
    const int64_t n = blockIdx.x;
    int id = ids[n];
    if (id < 0) id = feedback ? feedback[seq_slots[token_seq[n]]] : 0;
    const T* row = table + (int64_t)id * H;
    float* h = hidden + n * H;
    T* o = out + n * H;
    float ss = 0.f;
    if constexpr (VEC) {
        float4 v[NORM_CHUNKS], wv[NORM_CHUNKS];
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                wv[k] = load_weight4(weight, i, weight_dtype);
                v[k] = Quad<T>::load(row + i);
            }
        }
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                *(float4*)(h + i) = v[k];
                ss += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
            }
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)H + eps);
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                const float4 w = wv[k];
                Quad<T>::store(o + i, make_float4(v[k].x * inv * w.x, v[k].y * inv * w.y, v[k].z * inv * w.z,
                                                  v[k].w * inv * w.w));
            }
        }
    } else {
        for (int i = threadIdx.x; i < H; i += blockDim.x) {
            const float v = to_f32<T>(row[i]);
            h[i] = v;
            ss += v * v;
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)H + eps);
        // (each thread reads back the elements that it wrote itself)
        for (int i = threadIdx.x; i < H; i += blockDim.x)
            o[i] = from_f32<T>(h[i] * inv * load_as_f32(weight, i, weight_dtype));
    }
}

// ids int32 [N], table [V, H] and out [N, H] of `dtype`, hidden float32 [N, H]; `feedback`,
// `token_seq` [N] and `seq_slots`: all three or none.  The host has checked the ids.
extern "C" int lle_embedding_rmsnorm(const void* ids, const void* table, void* hidden, const void* weight,
                                     int weight_dtype, void* out, int N, int H, float eps, int dtype,
                                     const void* feedback, const void* token_seq, const void* seq_slots,
                                     hipStream_t stream) {
    if (N <= 0 || H <= 0) return 0;
    if ((feedback != nullptr) != (token_seq != nullptr) || (feedback != nullptr) != (seq_slots != nullptr))
        return (int)hipErrorInvalidValue;
    const bool vec = H % 4 == 0 && H <= 256 * 4 * NORM_CHUNKS;
#define LLE_EMBED_NORM(T, VEC)                                                                                  \
    embedding_rmsnorm_kernel<T, VEC><<<N, 256, 0, stream>>>(                                                    \
        (const int32_t*)ids, (const T*)table, (float*)hidden, weight, weight_dtype, (T*)out, H, eps,            \
        (const int32_t*)feedback, (const int32_t*)token_seq, (const int32_t*)seq_slots)
    if (dtype == LLE_F32) {
        if (vec) LLE_EMBED_NORM(float, true); else LLE_EMBED_NORM(float, false);
    } else if (dtype == LLE_BF16) {
        if (vec) LLE_EMBED_NORM(bf16_t, true); else LLE_EMBED_NORM(bf16_t, false);
    } else {
        return (int)hipErrorInvalidValue;
    }
#undef LLE_EMBED_NORM
    LLE_RETURN_LAUNCH_STATUS();
}

extern "C" int lle_add_rmsnorm_sums(void* hidden, const void* sums, int slices, int64_t slice_stride, const void* rows,
                                    const void* weight, int weight_dtype, void* out, int R, int H, float eps, int dtype,
                                    hipStream_t stream) {
    if (R <= 0) return 0;
    if (H % 4 != 0 || H > 256 * 4 * NORM_CHUNKS || slices < 1 || !sums) return (int)hipErrorInvalidValue;
    if (dtype == LLE_F32)
        add_rmsnorm_vec_kernel<float, float, true><<<R, 256, 0, stream>>>((float*)hidden, (const float*)sums,
                                                                     (const int32_t*)rows, weight, weight_dtype,
                                                                     (float*)out, H, eps, slices, slice_stride);
    else
        add_rmsnorm_vec_kernel<bf16_t, float, true><<<R, 256, 0, stream>>>((float*)hidden, (const float*)sums,
                                                                      (const int32_t*)rows, weight, weight_dtype,
                                                                      (bf16_t*)out, H, eps, slices, slice_stride);
    LLE_RETURN_LAUNCH_STATUS();
}

extern "C" int lle_add_rmsnorm(void* hidden, const void* delta, const void* rows, const void* weight,
                               int weight_dtype, void* out, int R, int H, float eps, int dtype,
                               hipStream_t stream) {
    if (R <= 0) return 0;
    if (H % 4 == 0 && H <= 256 * 4 * NORM_CHUNKS) {
        if (dtype == LLE_F32)
            add_rmsnorm_vec_kernel<float><<<R, 256, 0, stream>>>((float*)hidden, (const float*)delta,
                                                                  (const int32_t*)rows, weight, weight_dtype,
                                                                  (float*)out, H, eps);
        else
            add_rmsnorm_vec_kernel<bf16_t><<<R, 256, 0, stream>>>((float*)hidden, (const bf16_t*)delta,
                                                                   (const int32_t*)rows, weight, weight_dtype,
                                                                   (bf16_t*)out, H, eps);
        LLE_RETURN_LAUNCH_STATUS();
    }
    int threads = 256;
    if (H > 2048) threads = 512;
    if (H > 8192) threads = 1024;
    if (dtype == LLE_F32)
        add_rmsnorm_kernel<float><<<R, threads, 0, stream>>>((float*)hidden, (const float*)delta,
                                                              (const int32_t*)rows, weight, weight_dtype,
                                                              (float*)out, H, eps);
    else
        add_rmsnorm_kernel<bf16_t><<<R, threads, 0, stream>>>((float*)hidden, (const bf16_t*)delta,
                                                               (const int32_t*)rows, weight, weight_dtype,
                                                               (bf16_t*)out, H, eps);
    LLE_RETURN_LAUNCH_STATUS();
}

// plain RMSNorm of activation rows x [R, H] of type T (no residual): out = norm(x) * w, in the type TO
template <typename T, typename TO = T>
__global__ __launch_bounds__(256) void rmsnorm_kernel(const T* __restrict__ x, const void* __restrict__ weight,
                                                       int weight_dtype, TO* __restrict__ out, int H, float eps) {
    __shared__ float red[16];
    const int64_t r = blockIdx.x;
    const T* xr = x + r * H;
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        const float v = to_f32<T>(xr[i]);
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps);
    TO* o = out + r * H;
    for (int i = threadIdx.x; i < H; i += blockDim.x)
        o[i] = from_f32<TO>(to_f32<T>(xr[i]) * inv * load_as_f32(weight, i, weight_dtype));
}

extern "C" int lle_rmsnorm(const void* x, const void* weight, int weight_dtype, void* out, int R, int H, float eps,
                           int dtype, hipStream_t stream) {
    if (R <= 0) return 0;
    if (dtype == LLE_F32)
        rmsnorm_kernel<float><<<R, 256, 0, stream>>>((const float*)x, weight, weight_dtype, (float*)out, H, eps);
    else
        rmsnorm_kernel<bf16_t><<<R, 256, 0, stream>>>((const bf16_t*)x, weight, weight_dtype, (bf16_t*)out, H, eps);
    LLE_RETURN_LAUNCH_STATUS();
}

// float32 rows in, bfloat16 rows out: the norm of a product's 32-bit result, handed on in the activation type
extern "C" int lle_rmsnorm_f32_to_bf16(const void* x, const void* weight, int weight_dtype, void* out, int R, int H, float eps,
                                       hipStream_t stream) {
    if (R <= 0) return 0;
    rmsnorm_kernel<float, bf16_t><<<R, 256, 0, stream>>>((const float*)x, weight, weight_dtype, (bf16_t*)out, H, eps);
    LLE_RETURN_LAUNCH_STATUS();
}

// For arrangements that norm a sublayer's OUTPUT: hidden[r] += norm(y[r] (+ extra[r])) * w, in 32-bit and in
// place, and the new row of `hidden` leaves in the activation type TO as well (the next sublayer reads it).
// `y` and `extra` hold float32 or bfloat16, each said by its own code.
template <typename TO>
__global__ __launch_bounds__(1024) void rmsnorm_add_kernel(float* __restrict__ hidden, const void* __restrict__ y,
                                                            int y_dtype, const void* __restrict__ extra,
                                                            int extra_dtype, const void* __restrict__ weight,
                                                            int weight_dtype, TO* __restrict__ out, int H, float eps) {
    __shared__ float red[16];
    const int64_t r = blockIdx.x;
    const int64_t at = r * H;
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = load_as_f32(y, at + i, y_dtype);
        if (extra) v += load_as_f32(extra, at + i, extra_dtype);
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps);
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = load_as_f32(y, at + i, y_dtype);
        if (extra) v += load_as_f32(extra, at + i, extra_dtype);
        const float h = hidden[at + i] + v * inv * load_as_f32(weight, i, weight_dtype);
        hidden[at + i] = h;
        if (out) out[at + i] = from_f32<TO>(h);
    }
}

// `out` may be null (float32 callers read `hidden` itself)
extern "C" int lle_rmsnorm_add(void* hidden, const void* y, int y_dtype, const void* extra, int extra_dtype,
                               const void* weight, int weight_dtype, void* out, int R, int H, float eps,
                               int out_dtype, hipStream_t stream) {
    if (R <= 0) return 0;
    const int threads = H > 8192 ? 1024 : H > 2048 ? 512 : 256;
    if (out_dtype == LLE_F32)
        rmsnorm_add_kernel<float><<<R, threads, 0, stream>>>((float*)hidden, y, y_dtype, extra, extra_dtype, weight,
                                                              weight_dtype, (float*)out, H, eps);
    else
        rmsnorm_add_kernel<bf16_t><<<R, threads, 0, stream>>>((float*)hidden, y, y_dtype, extra, extra_dtype, weight,
                                                               weight_dtype, (bf16_t*)out, H, eps);
    LLE_RETURN_LAUNCH_STATUS();
}

// For arrangements whose sublayers run side by side on one norm's result and whose sum enters the stream
// times constants: hidden[r] += mult_a * a[r] (+ mult_b * b[r]) in 32-bit and in place, then out[r] = norm(hidden[r]) * w.
// `a`, `b` hold float32 or bfloat16, each said by its own code.  With `rows` only those rows are read, row
// rows[r] gives out[r], and `hidden` is left alone.  The new row waits in registers between the sum of
// squares and the scaling (rows up to 256 x 4 x SA_CHUNKS wide and a multiple of 4; a plain loop otherwise).
#define SA_CHUNKS 8
template <typename TO>
__global__ __launch_bounds__(256) void scaled_add_rmsnorm_kernel(float* __restrict__ hidden, const void* __restrict__ a,
                                                                  int a_dtype, const void* __restrict__ b, int b_dtype,
                                                                  float mult_a, float mult_b, const int32_t* __restrict__ rows,
                                                                  const void* __restrict__ weight, int weight_dtype,
                                                                  TO* __restrict__ out, int H, float eps) {
    __shared__ float red[16];
    const int64_t r = rows ? rows[blockIdx.x] : blockIdx.x;
    const int64_t at = r * H, to = (int64_t)blockIdx.x * H;
    float ss = 0.f;
    if (H % 4 == 0 && H <= 256 * 4 * SA_CHUNKS) {
        float4 keep[SA_CHUNKS];
#pragma unroll
        for (int c = 0; c < SA_CHUNKS; ++c) {
            const int i = (c * 256 + threadIdx.x) * 4;
            if (i < H) {
                float4 v = *(const float4*)(hidden + at + i);
                const float4 x = load_weight4(a, at + i, a_dtype);
                float4 d = make_float4(mult_a * x.x, mult_a * x.y, mult_a * x.z, mult_a * x.w);
                if (b) {
                    const float4 y = load_weight4(b, at + i, b_dtype);
                    d = make_float4(fmaf(mult_b, y.x, d.x), fmaf(mult_b, y.y, d.y), fmaf(mult_b, y.z, d.z), fmaf(mult_b, y.w, d.w));
                }
                v = make_float4(v.x + d.x, v.y + d.y, v.z + d.z, v.w + d.w);
                ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
                keep[c] = v;
                if (!rows) *(float4*)(hidden + at + i) = keep[c];
            }
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)H + eps);
#pragma unroll
        for (int c = 0; c < SA_CHUNKS; ++c) {
            const int i = (c * 256 + threadIdx.x) * 4;
            if (i < H) {
                const float4 w = load_weight4(weight, i, weight_dtype);
                Quad<TO>::store(out + to + i, make_float4(keep[c].x * inv * w.x, keep[c].y * inv * w.y, keep[c].z * inv * w.z,
                                                          keep[c].w * inv * w.w));
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float d = mult_a * load_as_f32(a, at + i, a_dtype);
        if (b) d = fmaf(mult_b, load_as_f32(b, at + i, b_dtype), d);
        const float v = hidden[at + i] + d;
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps);
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float d = mult_a * load_as_f32(a, at + i, a_dtype);
        if (b) d = fmaf(mult_b, load_as_f32(b, at + i, b_dtype), d);
        const float v = hidden[at + i] + d;
        if (!rows) hidden[at + i] = v;
        out[to + i] = from_f32<TO>(v * inv * load_as_f32(weight, i, weight_dtype));
    }
}

// R = number of rows of `out` (all rows of `hidden`, or the length of `rows`)
extern "C" int lle_scaled_add_rmsnorm(void* hidden, const void* a, int a_dtype, const void* b, int b_dtype, float mult_a,
                                      float mult_b, const void* rows, const void* weight, int weight_dtype, void* out, int R, int H,
                                      float eps, int out_dtype, hipStream_t stream) {
    if (R <= 0) return 0;
    if (out_dtype == LLE_F32)
        scaled_add_rmsnorm_kernel<float><<<R, 256, 0, stream>>>((float*)hidden, a, a_dtype, b, b_dtype, mult_a, mult_b,
                                                                 (const int32_t*)rows, weight, weight_dtype, (float*)out, H, eps);
    else
        scaled_add_rmsnorm_kernel<bf16_t><<<R, 256, 0, stream>>>((float*)hidden, a, a_dtype, b, b_dtype, mult_a, mult_b,
                                                                  (const int32_t*)rows, weight, weight_dtype, (bf16_t*)out, H,
                                                                  eps);
    LLE_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------
// Two norms around one add, for arrangements with a norm after a sublayer and a norm before the next:
//   hidden += RMSNorm(y [+ extra]) * w_out        (32-bit, in place)
//   out     = RMSNorm(hidden) * w_next            (the new row's norm, in the activation type)
// One workgroup a row; a thread keeps its share of the row (up to NR_PER elements) in registers from
// the first sum to the last store, so y, extra and hidden are read once.  Rows wider than
// NR_PER * threads take the plain loops.
// ---------------------------------------------------------------------------------
#define NR_PER 8

template <typename TO>
__global__ __launch_bounds__(1024) void rmsnorm_add_rmsnorm_kernel(
    float* __restrict__ hidden, const void* __restrict__ y, int y_dtype, const void* __restrict__ extra, int extra_dtype,
    const void* __restrict__ w_out, const void* __restrict__ w_next, int weight_dtype, TO* __restrict__ out, int H,
    float eps_out, float eps_next) {
    __shared__ float red[16];
    const int64_t at = (int64_t)blockIdx.x * H;
    if (H <= NR_PER * (int)blockDim.x) {
        float v[NR_PER];
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NR_PER; ++j) {
            const int i = threadIdx.x + j * blockDim.x;
            v[j] = 0.f;
            if (i < H) {
                v[j] = load_as_f32(y, at + i, y_dtype);
                if (extra) v[j] += load_as_f32(extra, at + i, extra_dtype);
            }
            ss += v[j] * v[j];
        }
        const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps_out);
        ss = 0.f;
#pragma unroll
        for (int j = 0; j < NR_PER; ++j) {
            const int i = threadIdx.x + j * blockDim.x;
            if (i < H) {
                v[j] = hidden[at + i] + v[j] * inv * load_as_f32(w_out, i, weight_dtype);
                hidden[at + i] = v[j];
                ss += v[j] * v[j];
            }
        }
        const float inv2 = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps_next);
#pragma unroll
        for (int j = 0; j < NR_PER; ++j) {
            const int i = threadIdx.x + j * blockDim.x;
            if (i < H) out[at + i] = from_f32<TO>(v[j] * inv2 * load_as_f32(w_next, i, weight_dtype));
        }
        return;
    }
    float ss = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = load_as_f32(y, at + i, y_dtype);
        if (extra) v += load_as_f32(extra, at + i, extra_dtype);
        ss += v * v;
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps_out);
    ss = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        float v = load_as_f32(y, at + i, y_dtype);
        if (extra) v += load_as_f32(extra, at + i, extra_dtype);
        const float h = hidden[at + i] + v * inv * load_as_f32(w_out, i, weight_dtype);
        hidden[at + i] = h;
        ss += h * h;
    }
    const float inv2 = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps_next);
    for (int i = threadIdx.x; i < H; i += blockDim.x)  // (every thread reads back what it wrote itself)
        out[at + i] = from_f32<TO>(hidden[at + i] * inv2 * load_as_f32(w_next, i, weight_dtype));
}

// both weights have the same type
extern "C" int lle_rmsnorm_add_rmsnorm(void* hidden, const void* y, int y_dtype, const void* extra, int extra_dtype,
                                       const void* w_out, const void* w_next, int weight_dtype, void* out, int R, int H,
                                       float eps_out, float eps_next, int out_dtype, hipStream_t stream) {
    if (R <= 0) return 0;
    const int threads = H > 4096 ? 1024 : H > 2048 ? 512 : 256;
    if (out_dtype == LLE_F32)
        rmsnorm_add_rmsnorm_kernel<float><<<R, threads, 0, stream>>>((float*)hidden, y, y_dtype, extra, extra_dtype, w_out,
                                                                      w_next, weight_dtype, (float*)out, H, eps_out, eps_next);
    else
        rmsnorm_add_rmsnorm_kernel<bf16_t><<<R, threads, 0, stream>>>((float*)hidden, y, y_dtype, extra, extra_dtype, w_out,
                                                                       w_next, weight_dtype, (bf16_t*)out, H, eps_out, eps_next);
    LLE_RETURN_LAUNCH_STATUS();
}

// Between two blocks something enters the stream: hidden[n] += a[n] (+ b[n]) (+ vec) (+ table[id(n)] * scale), all in
// 32-bit and in place, then out[n] = norm(hidden[n]) * w, one launch.  `a` (float32 or bfloat16, null: nothing is left
// to be added) may come as `slices` partial sums, `slice_stride` elements apart, added in slice order; `b` (or null)
// is another summand of a's kind with a type of its own; `vec` float32 [H] or null; `table` [V, H] or null: the
// embedding's rows once more, ids as in the embedding kernel.  With `rows` only those rows are read, row rows[r] gives
// row r of the result, and `hidden` is left alone.  The new row waits in registers where rows are no wider
// than 256 x 4 x NORM_CHUNKS and a multiple of 4 (a plain loop otherwise).
struct InjectArgs {
    float* hidden;
    const void* a;
    int a_dtype, slices;
    int64_t slice_stride;
    const void* b;
    int b_dtype;
    const float* vec;
    const int32_t* ids;
    const void* table;
    int table_dtype;
    float scale;
    const int32_t *feedback, *token_seq, *seq_slots;
    const int32_t* rows;
    const void* weight;
    int weight_dtype;
    void* out;
    int H;
    float eps;
};

__device__ __forceinline__ float4 load_quad(const void* p, int64_t i, int dtype) {
    return dtype == LLE_F32 ? Quad<float>::load((const float*)p + i) : Quad<bf16_t>::load((const bf16_t*)p + i);
}
__device__ __forceinline__ void add_quad(float4& v, float4 d) {
    v.x += d.x;
    v.y += d.y;
    v.z += d.z;
    v.w += d.w;
}

template <typename TO>
__global__ __launch_bounds__(256) void inject_rmsnorm_kernel(InjectArgs x) {
    __shared__ float red[16];
    const int64_t n = x.rows ? x.rows[blockIdx.x] : blockIdx.x, at = n * x.H, to = (int64_t)blockIdx.x * x.H;
    const int H = x.H;
    int64_t row = 0;
    if (x.table) {
        int id = x.ids[n];
        if (id < 0) id = x.feedback ? x.feedback[x.seq_slots[x.token_seq[n]]] : 0;
        row = (int64_t)id * H;
    }
    TO* out = (TO*)x.out;
    float ss = 0.f;
    if (H % 4 == 0 && H <= 256 * 4 * NORM_CHUNKS) {
        float4 keep[NORM_CHUNKS], wv[NORM_CHUNKS];
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                wv[k] = load_weight4(x.weight, i, x.weight_dtype);
                float4 v = *(const float4*)(x.hidden + at + i);
                if (x.a) {
                    float4 d = load_quad(x.a, at + i, x.a_dtype);
                    for (int s = 1; s < x.slices; ++s) add_quad(d, load_quad(x.a, s * x.slice_stride + at + i, x.a_dtype));
                    if (x.b) add_quad(d, load_quad(x.b, at + i, x.b_dtype));
                    add_quad(v, d);
                }
                if (x.table) {
                    const float4 e = load_quad(x.table, row + i, x.table_dtype);
                    add_quad(v, make_float4(e.x * x.scale, e.y * x.scale, e.z * x.scale, e.w * x.scale));
                }
                if (x.vec) add_quad(v, Quad<float>::load(x.vec + i));
                if (!x.rows) *(float4*)(x.hidden + at + i) = v;
                keep[k] = v;
                ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
            }
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)H + x.eps);
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H)
                Quad<TO>::store(out + to + i, make_float4(keep[k].x * inv * wv[k].x, keep[k].y * inv * wv[k].y,
                                                          keep[k].z * inv * wv[k].z, keep[k].w * inv * wv[k].w));
        }
        return;
    }
    auto sum_at = [&](int i) {
        float v = x.hidden[at + i];
        if (x.a) {
            float d = load_as_f32(x.a, at + i, x.a_dtype);
            for (int s = 1; s < x.slices; ++s) d += load_as_f32(x.a, s * x.slice_stride + at + i, x.a_dtype);
            if (x.b) d += load_as_f32(x.b, at + i, x.b_dtype);
            v += d;
        }
        if (x.table) v += load_as_f32(x.table, row + i, x.table_dtype) * x.scale;
        if (x.vec) v += x.vec[i];
        return v;
    };
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        const float v = sum_at(i);
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + x.eps);
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
        const float v = sum_at(i);
        if (!x.rows) x.hidden[at + i] = v;
        out[to + i] = from_f32<TO>(v * inv * load_as_f32(x.weight, i, x.weight_dtype));
    }
}

extern "C" int lle_inject_rmsnorm(void* hidden, const void* a, int a_dtype, int slices, int64_t slice_stride, const void* b,
                                  int b_dtype, const void* vec, const void* ids, const void* table, int table_dtype,
                                  float scale, const void* feedback, const void* token_seq, const void* seq_slots,
                                  const void* rows, const void* weight, int weight_dtype, void* out, int N, int H, float eps,
                                  int out_dtype, hipStream_t stream) {
    if (N <= 0 || H <= 0) return 0;
    if (slices < 1 || (b && !a) || (table && !ids) || (feedback != nullptr) != (token_seq != nullptr) ||
        (feedback != nullptr) != (seq_slots != nullptr))
        return (int)hipErrorInvalidValue;
    const InjectArgs x{(float*)hidden, a, a_dtype, slices, slice_stride, b, b_dtype, (const float*)vec, (const int32_t*)ids,
                       table, table_dtype, scale, (const int32_t*)feedback, (const int32_t*)token_seq,
                       (const int32_t*)seq_slots, (const int32_t*)rows, weight, weight_dtype, out, H, eps};
    if (out_dtype == LLE_F32) inject_rmsnorm_kernel<float><<<N, 256, 0, stream>>>(x);
    else inject_rmsnorm_kernel<bf16_t><<<N, 256, 0, stream>>>(x);
    LLE_RETURN_LAUNCH_STATUS();
}

// The first rows of the residual stream where they are made of more than the embedding table:
//   h[n] = RMSNorm(table[id(n)] * scale (+ pos[position n])) * w0 (w0 null: without that norm)
// and, with `weight`, the first block's norm of the new row in the same launch: out[n] = RMSNorm(h[n]) * weight.  All in
// 32-bit; h is float32.  Ids as in the embedding kernel; the host has checked ids and positions (a position past the
// table would read its last row).  A thread keeps its share of the row in registers (rows up to 256 x 4 x NORM_CHUNKS and a
// multiple of 4; others are read back from `hidden`, each element by the thread that wrote it).
struct EmbedArgs {
    const int32_t* ids;
    const void* table;
    int table_dtype;
    float scale;
    const int32_t *feedback, *token_seq, *seq_slots;
    const void* pos;
    int pos_dtype, pos_rows;
    const int32_t* positions;
    const void* w0;
    int w0_dtype;
    float eps0;
    float* hidden;
    const void* weight;
    int weight_dtype;
    float eps;
    void* out;
    int H;
};

template <typename TO>
__global__ __launch_bounds__(256) void embedding_norm_kernel(EmbedArgs x) {
    __shared__ float red[16];
    const int64_t n = blockIdx.x;
    const int H = x.H;
    int id = x.ids[n];
    if (id < 0) id = x.feedback ? x.feedback[x.seq_slots[x.token_seq[n]]] : 0;
    const int64_t row = (int64_t)id * H;
    const int64_t prow = x.pos ? (int64_t)min(max(x.positions[n], 0), x.pos_rows - 1) * H : 0;
    float* h = x.hidden + n * H;
    auto made = [&](int i) {
        float v = load_as_f32(x.table, row + i, x.table_dtype) * x.scale;
        if (x.pos) v += load_as_f32(x.pos, prow + i, x.pos_dtype);
        return v;
    };
    const bool fits = H % 4 == 0 && H <= 256 * 4 * NORM_CHUNKS;
    float4 keep[NORM_CHUNKS];
    float ss = 0.f;
    const auto squares = [](float4 v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; };
    const auto times = [](float4 v, float f, float4 w) { return make_float4(v.x * f * w.x, v.y * f * w.y, v.z * f * w.z, v.w * f * w.w); };
    if (fits) {
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                const float4 e = load_quad(x.table, row + i, x.table_dtype);
                keep[k] = make_float4(e.x * x.scale, e.y * x.scale, e.z * x.scale, e.w * x.scale);
                if (x.pos) add_quad(keep[k], load_quad(x.pos, prow + i, x.pos_dtype));
                ss += squares(keep[k]);
            }
        }
    } else {
        for (int i = threadIdx.x; i < H; i += blockDim.x) {
            const float v = made(i);
            h[i] = v;
            ss += v * v;
        }
    }
    const float inv0 = x.w0 ? 1.0f / sqrtf(block_sum(ss, red) / (float)H + x.eps0) : 1.0f;
    ss = 0.f;
    if (fits) {
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) {
                if (x.w0) keep[k] = times(keep[k], inv0, load_quad(x.w0, i, x.w0_dtype));
                *(float4*)(h + i) = keep[k];
                ss += squares(keep[k]);
            }
        }
    } else {
        for (int i = threadIdx.x; i < H; i += blockDim.x) {
            float v = h[i];
            if (x.w0) v *= inv0 * load_as_f32(x.w0, i, x.w0_dtype);
            h[i] = v;
            ss += v * v;
        }
    }
    if (!x.weight) return;  // (the same for every thread)
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)H + x.eps);
    TO* out = (TO*)x.out + n * H;
    if (fits) {
#pragma unroll
        for (int k = 0; k < NORM_CHUNKS; ++k) {
            const int i = (k * 256 + threadIdx.x) * 4;
            if (i < H) Quad<TO>::store(out + i, times(keep[k], inv, load_quad(x.weight, i, x.weight_dtype)));
        }
    } else {
        for (int i = threadIdx.x; i < H; i += blockDim.x) out[i] = from_f32<TO>(h[i] * inv * load_as_f32(x.weight, i, x.weight_dtype));
    }
}

extern "C" int lle_embedding_norm(const void* ids, const void* table, int table_dtype, float scale, const void* feedback,
                                  const void* token_seq, const void* seq_slots, const void* pos, int pos_dtype, int pos_rows,
                                  const void* positions, const void* w0, int w0_dtype, float eps0, void* hidden,
                                  const void* weight, int weight_dtype, float eps, void* out, int N, int H, int out_dtype,
                                  hipStream_t stream) {
    if (N <= 0 || H <= 0) return 0;
    if ((feedback != nullptr) != (token_seq != nullptr) || (feedback != nullptr) != (seq_slots != nullptr) ||
        (pos && (!positions || pos_rows <= 0)) || (weight && !out))
        return (int)hipErrorInvalidValue;
    const EmbedArgs x{(const int32_t*)ids, table, table_dtype, scale, (const int32_t*)feedback, (const int32_t*)token_seq,
                      (const int32_t*)seq_slots, pos, pos_dtype, pos_rows, (const int32_t*)positions, w0, w0_dtype, eps0,
                      (float*)hidden, weight, weight_dtype, eps, out, H};
    if (out_dtype == LLE_F32) embedding_norm_kernel<float><<<N, 256, 0, stream>>>(x);
    else embedding_norm_kernel<bf16_t><<<N, 256, 0, stream>>>(x);
    LLE_RETURN_LAUNCH_STATUS();
}
