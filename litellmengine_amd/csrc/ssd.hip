// The state-space recurrence of Mamba-2: a matrix state per head with one decay per token and head.
//
//   c = silu(conv(u) + b)               per channel over time, J taps, the request's last J - 1 rows kept     ssd_conv
//   x, B, C = c's parts                 x [H vdim], B and C [G N]; head h reads group h / (H / G)
//   dt = softplus(d + dt_bias),  a = -exp(A_log) dt                 one of each per token and head            ssd_scan
//   S <- exp(a_t) S + dt_t B_t x_t^T;   y_t = S^T C_t + D x_t       S [N, vdim] float32, per head
//   out = norm(y * silu(z)) * w         the root mean square over each of `groups` equal parts of a row       ssd_gate_norm
//
// The state lies transposed in its row, [head][value j][state n].  Everything that enters the recurrence is 32-bit in
// every mode; u, z and out have the activation type.
//
// A request with few tokens in a step (SSD_WALK at most: decoded tokens, short portions) is walked token by token from
// its state.  A longer one is cut into chunks of SSD_CHUNK tokens that are worked on side by side.  With l_t the sum of
// a over the chunk's tokens up to t,
//   pass 1  every chunk's own contribution to the state, sum_s exp(l_last - l_s) dt_s B_s x_s^T, and exp(l_last)
//   carry   a short walk over the chunks leaves every chunk's entry state, and the request's state behind the last
//   pass 2  y_t = exp(l_t) S_entry^T C_t + sum_(s <= t) exp(l_t - l_s) (C_t . B_s) dt_s x_s + D x_t
// All exponents are at most zero.  The sums l are kept as two floats, so that the difference of two neighbours deep in
// a chunk is as exact as if it had been added up on its own.  The products are taken on the 32-bit matrix instruction.
#include "common.h"

LLE_DEFINE_ERROR_STRING()

#define SSD_CHUNK 64
#define SSD_WALK 32
typedef float ssd_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float ssd_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float ssd_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// ---------------------------------------------------------------------------------
// Convolution and silu.  The channels are the columns col0 .. col0 + CC - 1 of u; a thread walks `run` tokens of one
// channel with its taps and the last J - 1 inputs in registers; where the request changes inside a run the window is
// filled anew.  `state` rows hold the last J - 1 inputs of earlier steps, oldest first (float32); zeros at admission
// stand for the zeros before a request's start.  ADVANCE (steps of single tokens only): the kept rows move on by the
// token in the same launch.  grid = (runs, blocks of 256 channels)
// ---------------------------------------------------------------------------------
struct SsdConvArgs {
    const void* u;
    int cols, col0;
    const float* taps;  // [CC, J]
    const float* bias;  // [CC] or null
    float* state;
    int64_t state_stride;
    const int32_t *token_seq, *cu_tokens, *seq_slots;
    float* out;  // [N, CC]
    int N, CC, J, run;
    // steps of single tokens: workgroups behind the convolution's make the step sizes' product, dt = x dt_w^T
    const void* x;     // [N, K] or null
    const void* dt_w;  // [H, K]
    float* dt;         // [N, H]
    int K, H, conv_blocks;
};

// dt[n, h] = sum_k x[n, k] dt_w[h, k] in 32-bit: a wavefront has one head and up to SSD_DT_TOKENS tokens
#define SSD_DT_TOKENS 4
template <typename T>
__device__ __forceinline__ void ssd_step_products(const SsdConvArgs& a, int block) {
    const int wave = block * 4 + threadIdx.x / LLE_WAVE, lane = threadIdx.x % LLE_WAVE;
    const int h = wave % a.H, n0 = wave / a.H * SSD_DT_TOKENS;
    if (n0 >= a.N) return;
    const T* w = (const T*)a.dt_w + (int64_t)h * a.K;
    const T* x = (const T*)a.x;
    float acc[SSD_DT_TOKENS];
#pragma unroll
    for (int t = 0; t < SSD_DT_TOKENS; ++t) acc[t] = 0.f;
#pragma unroll 4
    for (int k = lane; k < a.K; k += LLE_WAVE) {
        const float wv = to_f32<T>(w[k]);
#pragma unroll
        for (int t = 0; t < SSD_DT_TOKENS; ++t) acc[t] = fmaf(to_f32<T>(x[(int64_t)min(n0 + t, a.N - 1) * a.K + k]), wv, acc[t]);
    }
#pragma unroll
    for (int t = 0; t < SSD_DT_TOKENS; ++t) {
        const float sum = wave_sum(acc[t]);
        if (lane == 0 && n0 + t < a.N) a.dt[(int64_t)(n0 + t) * a.H + h] = sum;
    }
}

template <typename T, int J, bool ADVANCE>
__global__ __launch_bounds__(256) void ssd_conv_run_kernel(SsdConvArgs a) {
    constexpr int W = J > 1 ? J - 1 : 1;
    if (ADVANCE && (int)blockIdx.y >= a.conv_blocks) {
        ssd_step_products<T>(a, (blockIdx.y - a.conv_blocks) * gridDim.x + blockIdx.x);
        return;
    }
    const int ch = blockIdx.y * 256 + threadIdx.x;
    if (ch >= a.CC) return;
    const int n0 = blockIdx.x * a.run, n1 = min(a.N, n0 + a.run);
    const T* u = (const T*)a.u + a.col0 + ch;
    float tp[J], win[W];
#pragma unroll
    for (int j = 0; j < J; ++j) tp[j] = a.taps[(int64_t)ch * J + j];
#pragma unroll
    for (int m = 0; m < W; ++m) win[m] = 0.f;
    const float bias = a.bias ? a.bias[ch] : 0.f;
    int seq_before = -1;
    for (int n = n0; n < n1; ++n) {
        const int seq = a.token_seq[n];
        float* kept = J > 1 ? a.state + (int64_t)a.seq_slots[seq] * a.state_stride : nullptr;
        if (J > 1 && seq != seq_before) {  // (the same for the whole wavefront) the J - 1 inputs ahead of this token
            const int before = n - a.cu_tokens[seq];
#pragma unroll
            for (int m = 0; m < W; ++m) {
                const int back = J - 1 - m;
                win[m] = back <= before ? to_f32<T>(u[(int64_t)(n - back) * a.cols]) : kept[(int64_t)(J - 1 - (back - before)) * a.CC + ch];
            }
        }
        seq_before = seq;
        const float x = to_f32<T>(u[(int64_t)n * a.cols]);
        float acc = bias;
        if (J > 1) {
#pragma unroll
            for (int m = 0; m < W; ++m) acc = fmaf(tp[m], win[m], acc);
#pragma unroll
            for (int m = 0; m + 1 < W; ++m) win[m] = win[m + 1];
            win[W - 1] = x;
            if (ADVANCE) {
#pragma unroll
                for (int m = 0; m < W; ++m) kept[(int64_t)m * a.CC + ch] = win[m];
            }
        }
        a.out[(int64_t)n * a.CC + ch] = ssd_silu(fmaf(tp[J - 1], x, acc));
    }
}

// any number of taps: a thread a channel and token
template <typename T>
__global__ __launch_bounds__(256) void ssd_conv_kernel(SsdConvArgs a) {
    const int64_t n = blockIdx.x;
    const int ch = blockIdx.y * 256 + threadIdx.x;
    if (ch >= a.CC) return;
    const T* u = (const T*)a.u + a.col0 + ch;
    const int seq = a.token_seq[n], before = (int)(n - a.cu_tokens[seq]);
    const float* kept = a.state + (int64_t)a.seq_slots[seq] * a.state_stride;
    float acc = a.bias ? a.bias[ch] : 0.f;
    for (int j = 0; j < a.J; ++j) {
        const int back = a.J - 1 - j;
        const float x = back <= before ? to_f32<T>(u[(n - back) * a.cols]) : kept[(int64_t)(a.J - 1 - (back - before)) * a.CC + ch];
        acc = fmaf(a.taps[(int64_t)ch * a.J + j], x, acc);
    }
    a.out[n * a.CC + ch] = ssd_silu(acc);
}

// state row of every request <- the last J - 1 of (what it held, then the request's inputs of this step)
template <typename T>
__global__ __launch_bounds__(256) void ssd_conv_state_kernel(SsdConvArgs a) {
    const int s = blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
    if (ch >= a.CC) return;
    const int q0 = a.cu_tokens[s], len = a.cu_tokens[s + 1] - q0, kept = a.J - 1;
    if (len <= 0) return;
    float* row = a.state + (int64_t)a.seq_slots[s] * a.state_stride + ch;
    const T* u = (const T*)a.u + a.col0 + ch;
    for (int m = 0; m < kept; ++m) {  // (row m takes what lies `len` rows further on: never a row written before it)
        const int from = m + len - kept;  // index among this step's inputs, below zero: a kept row
        row[(int64_t)m * a.CC] = from >= 0 ? to_f32<T>(u[(int64_t)(q0 + from) * a.cols]) : row[(int64_t)(m + len) * a.CC];
    }
}

template <typename T>
static bool ssd_conv_runs(SsdConvArgs a, bool advance, hipStream_t stream) {
    const int blocks = (a.CC + 255) / 256;
    int run = (int)((int64_t)a.N * blocks / 2048);  // runs that load taps and windows seldom, and fill the chip
    a.run = run < 1 ? 1 : run > 16 ? 16 : run;
    dim3 grid((a.N + a.run - 1) / a.run, blocks);
    a.conv_blocks = blocks;
    if (advance && a.x) {
        const int waves = a.H * ((a.N + SSD_DT_TOKENS - 1) / SSD_DT_TOKENS);
        grid.y += ((waves + 3) / 4 + grid.x - 1) / grid.x;
    }
#define SSD_CONV_CASE(JJ)                                                             \
    case JJ:                                                                          \
        if (advance) ssd_conv_run_kernel<T, JJ, true><<<grid, 256, 0, stream>>>(a);   \
        else ssd_conv_run_kernel<T, JJ, false><<<grid, 256, 0, stream>>>(a);          \
        return true;
    switch (a.J) {
        SSD_CONV_CASE(1) SSD_CONV_CASE(2) SSD_CONV_CASE(3) SSD_CONV_CASE(4)
        SSD_CONV_CASE(5) SSD_CONV_CASE(6) SSD_CONV_CASE(7) SSD_CONV_CASE(8)
    }
#undef SSD_CONV_CASE
    return false;
}

// u [N, cols] in `dtype`; taps float32 [CC, J], bias float32 [CC] or null; state rows of state_stride floats whose first
// (J - 1) CC hold the kept rows; out float32 [N, CC].  The state is advanced: by this launch where every request of the
// step has one token (`single` != 0), else by one behind it.  With `single` and J <= 8 the launch also makes dt = x dt_w^T
// (x [N, K] and dt_w [H, K] in `dtype`, dt float32 [N, H]) where x is given.
extern "C" int lle_ssd_conv(const void* u, int cols, int col0, const void* taps, int J, const void* bias, void* state,
                            int64_t state_stride, const void* token_seq, const void* cu_tokens, const void* seq_slots, void* out,
                            int N, int S, int CC, int single, const void* x, const void* dt_w, void* dt, int K, int H, int dtype,
                            hipStream_t stream) {
    if (N <= 0 || CC <= 0) return 0;
    if (J < 1 || (J > 1 && !state) || col0 < 0 || col0 + CC > cols || (CC + 255) / 256 > 65535 || S <= 0) return (int)hipErrorInvalidValue;
    if (x && (!single || J > 8 || !dt_w || !dt || K <= 0 || H <= 0)) return (int)hipErrorInvalidValue;
    const SsdConvArgs a{u, cols, col0, (const float*)taps, (const float*)bias, (float*)state, state_stride, (const int32_t*)token_seq,
                        (const int32_t*)cu_tokens, (const int32_t*)seq_slots, (float*)out, N, CC, J, 1, x, dt_w, (float*)dt, K, H, 0};
    const bool advance = single && J <= 8;
    const bool done = dtype == LLE_F32 ? ssd_conv_runs<float>(a, advance, stream) : ssd_conv_runs<bf16_t>(a, advance, stream);
    const int blocks = (CC + 255) / 256;
    if (!done) {
        if (dtype == LLE_F32) ssd_conv_kernel<float><<<dim3(N, blocks), 256, 0, stream>>>(a);
        else ssd_conv_kernel<bf16_t><<<dim3(N, blocks), 256, 0, stream>>>(a);
    }
    if (J > 1 && !advance) {
        if (dtype == LLE_F32) ssd_conv_state_kernel<float><<<dim3(S, blocks), 256, 0, stream>>>(a);
        else ssd_conv_state_kernel<bf16_t><<<dim3(S, blocks), 256, 0, stream>>>(a);
    }
    LLE_RETURN_LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------------
// The recurrence.
// ---------------------------------------------------------------------------------
struct SsdArgs {
    const float* c;  // [N, CC]: x [H vdim], B [G N], C [G N]
    int CC;
    const float* dt_in;  // rows of dt_cols floats: a head's step size before its bias
    int dt_cols;
    const float *dt_bias, *a_log, *D;  // [H]
    float* state;                      // rows of state_stride floats: [H][vdim][N]
    int64_t state_stride;
    const int32_t *seq_slots, *cu_tokens;
    float* y;  // [N, H vdim]
    int H, G, vdim, n;
    int heads_a_group;   // pass 2: heads of one group that a workgroup takes one after the other
    int pieces;          // chunks of the longest request
    float* part;         // [chunk slots][H][vdim n]: a chunk's own contribution, then its entry state
    float* part_decay;   // [chunk slots][H]
    bool state_wide;     // the state rows start at multiples of 16 bytes
};

// where a request's chunks lie in `part`: requests one after the other, never two in one slot
__device__ __forceinline__ int64_t ssd_slot(int q0, int s) { return (int64_t)(q0 / SSD_CHUNK) + s; }

template <int CTRL>
__device__ __forceinline__ float ssd_lanes(float x) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, false));
}
// the sum over the 16 lanes of a row, in every one of them
__device__ __forceinline__ float ssd_row_sum(float x) {
    x += ssd_lanes<0xB1>(x);
    x += ssd_lanes<0x4E>(x);
    x += ssd_lanes<0x141>(x);
    x += ssd_lanes<0x140>(x);
    return x;
}

// Requests of at most SSD_WALK tokens.  grid = (requests, heads, blocks of 16 value channels), 256 threads: thread
// (jl, ig) = (tid / 16, tid % 16) owns the state channels [ig KI, (ig + 1) KI) of column j = block 16 + jl; the sixteen
// threads of a column are neighbours in a wavefront and add their shares of S^T C up through the lanes' cross-bar.  The
// tokens pass through LDS SSD_TC at a time.
#define SSD_TC 8
template <int KI>
__global__ __launch_bounds__(256) void ssd_walk_kernel(SsdArgs a) {
    constexpr int KN = KI * 16;
    __shared__ __attribute__((aligned(16))) float s_B[SSD_TC][KN], s_C[SSD_TC][KN];
    __shared__ float s_x[SSD_TC][16], s_g[SSD_TC], s_dt[SSD_TC];
    const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, jl = tid / 16, ig = tid % 16;
    const int n = a.n, vdim = a.vdim, j0 = blockIdx.z * 16, j = j0 + jl;
    const int q0 = a.cu_tokens[s], q1 = a.cu_tokens[s + 1];
    if (q1 <= q0 || q1 - q0 > SSD_WALK) return;
    const int grp = h / (a.H / a.G), inner = a.H * vdim;
    float* col = a.state + (int64_t)a.seq_slots[s] * a.state_stride + ((int64_t)h * vdim + j) * n + ig * KI;
    const bool live = j < vdim;
    float S[KI];
    if (KI % 4 == 0 && n == KN && a.state_wide) {  // (rows of a multiple of 64 channels: 16 bytes a load)
#pragma unroll
        for (int i = 0; i + 3 < KI; i += 4) {
            const float4 v = live ? *(const float4*)(col + i) : float4{0.f, 0.f, 0.f, 0.f};
            S[i] = v.x, S[i + 1] = v.y, S[i + 2] = v.z, S[i + 3] = v.w;
        }
    } else {
#pragma unroll
        for (int i = 0; i < KI; ++i) S[i] = (live && ig * KI + i < n) ? col[i] : 0.f;
    }
    const float rate = expf(a.a_log[h]), dt_bias = a.dt_bias[h], D = a.D[h];
    for (int c0 = q0; c0 < q1; c0 += SSD_TC) {
        const int nt = min(SSD_TC, q1 - c0);
        if (c0 > q0) __syncthreads();  // (the chunk before has been read)
        for (int e = tid; e < SSD_TC * KN; e += 256) {
            const int t = e / KN, i = e - t * KN;
            const bool there = t < nt && i < n;
            const float* row = a.c + (int64_t)(c0 + t) * a.CC + inner + grp * n + i;
            s_B[t][i] = there ? row[0] : 0.f;
            s_C[t][i] = there ? row[a.G * n] : 0.f;
        }
        if (tid < SSD_TC * 16) {
            const int t = tid / 16, e = tid % 16;
            s_x[t][e] = (t < nt && j0 + e < vdim) ? a.c[(int64_t)(c0 + t) * a.CC + h * vdim + j0 + e] : 0.f;
        } else if (tid >= 192 && tid - 192 < nt) {
            const float dt = ssd_softplus(a.dt_in[(int64_t)(c0 + tid - 192) * a.dt_cols + h] + dt_bias);
            s_dt[tid - 192] = dt;
            s_g[tid - 192] = expf(-rate * dt);
        }
        __syncthreads();
#pragma unroll
        for (int t = 0; t < SSD_TC; ++t) {
            if (t < nt) {
                const float g = s_g[t], x = s_x[t][jl], xdt = x * s_dt[t];
                const float *B = &s_B[t][ig * KI], *C = &s_C[t][ig * KI];
                float o = 0.f;
#pragma unroll
                for (int i = 0; i < KI; ++i) {
                    S[i] = fmaf(B[i], xdt, g * S[i]);
                    o = fmaf(S[i], C[i], o);
                }
                o = ssd_row_sum(o);
                if (ig == 0 && live) a.y[(int64_t)(c0 + t) * inner + h * vdim + j] = fmaf(D, x, o);
            }
        }
    }
    if (!live) return;
    if (KI % 4 == 0 && n == KN && a.state_wide) {
#pragma unroll
        for (int i = 0; i + 3 < KI; i += 4) *(float4*)(col + i) = float4{S[i], S[i + 1], S[i + 2], S[i + 3]};
    } else {
#pragma unroll
        for (int i = 0; i < KI; ++i)
            if (ig * KI + i < n) col[i] = S[i];
    }
}

// One wavefront: step sizes of a chunk's tokens (a token a lane; past the last one: 0) and the sums l of the logarithms
// of their decays up to each token, as two floats (the second is what the first has rounded away).
__device__ __forceinline__ void ssd_chunk_steps(const SsdArgs& a, int h, int t0, int nt, float& dt, float& l_hi, float& l_lo) {
    const int lane = threadIdx.x % LLE_WAVE;
    dt = lane < nt ? ssd_softplus(a.dt_in[(int64_t)(t0 + lane) * a.dt_cols + h] + a.dt_bias[h]) : 0.f;
    double l = -(double)expf(a.a_log[h]) * (double)dt;
#pragma unroll
    for (int o = 1; o < LLE_WAVE; o <<= 1) {
        const double before = __shfl_up(l, o, LLE_WAVE);
        if (lane >= o) l += before;
    }
    l_hi = (float)l;
    l_lo = (float)(l - (double)l_hi);
}

// Pass 1.  grid = (requests x pieces, heads), 256 threads.  B and x (times its factor) of the chunk wait in LDS; the
// contribution, [vdim, n] as the state lies, is taken in 16 x 16 tiles, four tokens an instruction: a lane (c, r) gives
// token 4 k + c of row (column) r.  Row strides of 16 modulo 64 words spread the four tokens over the banks.
template <int JT>  // tiles of value channels that a wavefront keeps side by side
__global__ __launch_bounds__(256) void ssd_chunk_state_kernel(SsdArgs a) {
    extern __shared__ float lds[];
    const int s = blockIdx.x / a.pieces, piece = blockIdx.x % a.pieces, h = blockIdx.y;
    const int q0 = a.cu_tokens[s], len = a.cu_tokens[s + 1] - q0;
    if (len <= SSD_WALK || piece * SSD_CHUNK >= len) return;
    const int t0 = q0 + piece * SSD_CHUNK, nt = min(SSD_CHUNK, len - piece * SSD_CHUNK);
    const int n = a.n, vdim = a.vdim, grp = h / (a.H / a.G), inner = a.H * vdim;
    const int BS = (n + 63) / 64 * 64 + 16, XS = (vdim + 63) / 64 * 64 + 16;
    float* s_B = lds;                    // [SSD_CHUNK][BS]
    float* s_x = s_B + SSD_CHUNK * BS;   // [SSD_CHUNK][XS]
    float* s_f = s_x + SSD_CHUNK * XS;   // [SSD_CHUNK] exp(l_last - l_s) dt_s
    const int tid = threadIdx.x, wave = tid / LLE_WAVE, lane = tid % LLE_WAVE, c = lane / 16, r = lane % 16;
    const int64_t slot = ssd_slot(q0, s) + piece;
    if (wave == 0) {
        float dt, hi, lo;
        ssd_chunk_steps(a, h, t0, nt, dt, hi, lo);
        const float hi_last = __shfl(hi, LLE_WAVE - 1, LLE_WAVE), lo_last = __shfl(lo, LLE_WAVE - 1, LLE_WAVE);
        s_f[lane] = expf((hi_last - hi) + (lo_last - lo)) * dt;
        if (lane == 0) a.part_decay[slot * a.H + h] = expf(hi_last);
    }
    const int np = BS - 16, vp = XS - 16;
    const float* rows = a.c + (int64_t)t0 * a.CC;
    const int bcol = inner + grp * n;
    const bool wide = n % 4 == 0 && vdim % 4 == 0 && a.CC % 4 == 0 && bcol % 4 == 0;
    if (wide) {
        for (int e = tid; e < SSD_CHUNK * np / 4; e += 256) {
            const int t = e / (np / 4), i = (e - t * (np / 4)) * 4;
            *(float4*)(s_B + t * BS + i) = (t < nt && i < n) ? *(const float4*)(rows + (int64_t)t * a.CC + bcol + i) : float4{0.f, 0.f, 0.f, 0.f};
        }
    } else {
        for (int e = tid; e < SSD_CHUNK * np; e += 256) {
            const int t = e / np, i = e - t * np;
            s_B[t * BS + i] = (t < nt && i < n) ? rows[(int64_t)t * a.CC + bcol + i] : 0.f;
        }
    }
    __syncthreads();
    if (wide) {
        for (int e = tid; e < SSD_CHUNK * vp / 4; e += 256) {
            const int t = e / (vp / 4), i = (e - t * (vp / 4)) * 4;
            float4 v = float4{0.f, 0.f, 0.f, 0.f};
            if (t < nt && i < vdim) {
                v = *(const float4*)(rows + (int64_t)t * a.CC + h * vdim + i);
                const float f = s_f[t];
                v = float4{v.x * f, v.y * f, v.z * f, v.w * f};
            }
            *(float4*)(s_x + t * XS + i) = v;
        }
    } else {
        for (int e = tid; e < SSD_CHUNK * vp; e += 256) {
            const int t = e / vp, i = e - t * vp;
            s_x[t * XS + i] = (t < nt && i < vdim) ? rows[(int64_t)t * a.CC + h * vdim + i] * s_f[t] : 0.f;
        }
    }
    __syncthreads();
    float* out = a.part + (slot * a.H + h) * (int64_t)vdim * n;
    const int j_tiles = (vdim + 15) / 16, n_tiles = (n + 15) / 16;
    for (int nt0 = wave; nt0 < n_tiles; nt0 += 4) {
        for (int jt0 = 0; jt0 < j_tiles; jt0 += JT) {
            ssd_f32x4 acc[JT];
#pragma unroll
            for (int q = 0; q < JT; ++q) acc[q] = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
            for (int k = 0; k < SSD_CHUNK; k += 4) {
                const float b = s_B[(k + c) * BS + nt0 * 16 + r];
#pragma unroll
                for (int q = 0; q < JT; ++q) {
                    const int jt = min(jt0 + q, j_tiles - 1);
                    acc[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_x[(k + c) * XS + jt * 16 + r], b, acc[q], 0, 0, 0);
                }
            }
#pragma unroll
            for (int q = 0; q < JT; ++q) {
                const int j = (jt0 + q) * 16 + 4 * c, col = nt0 * 16 + r;
                if (col < n) {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (jt0 + q < j_tiles && j + e < vdim) out[(int64_t)(j + e) * n + col] = acc[q][e];
                }
            }
        }
    }
}

// grid = (requests, heads, blocks of 256 state elements): a thread walks one element through the chunks and leaves every
// chunk's entry state in the place of its contribution, the state behind the last chunk in the request's row
__global__ __launch_bounds__(256) void ssd_carry_kernel(SsdArgs a) {
    const int s = blockIdx.x, h = blockIdx.y, elems = a.vdim * a.n;
    const int e = blockIdx.z * 256 + threadIdx.x;
    const int q0 = a.cu_tokens[s], len = a.cu_tokens[s + 1] - q0;
    if (e >= elems || len <= SSD_WALK) return;
    const int live = (len + SSD_CHUNK - 1) / SSD_CHUNK;
    const int64_t slot0 = ssd_slot(q0, s), stride = (int64_t)a.H * elems;
    float* base = a.part + (slot0 * a.H + h) * elems + e;
    const float* decay = a.part_decay + slot0 * a.H + h;
    float* own = a.state + (int64_t)a.seq_slots[s] * a.state_stride + (int64_t)h * elems + e;
    float S = *own;
    for (int p0 = 0; p0 < live; p0 += 8) {
        float A[8], B[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) {  // (asked for together)
            const int p = min(p0 + k, live - 1);
            B[k] = base[p * stride];
            A[k] = decay[(int64_t)p * a.H];
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) {
            if (p0 + k < live) {
                base[(p0 + k) * stride] = S;
                S = fmaf(A[k], S, B[k]);
            }
        }
    }
    *own = S;
}

// four consecutive elements of a row of `n`, zeros past its end
template <bool WIDE>
__device__ __forceinline__ ssd_f32x4 ssd_quad(const float* row, int i, int n) {
    ssd_f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (WIDE) {  // (n a multiple of 4, rows aligned)
        if (i < n) v = *(const ssd_f32x4*)(row + i);
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (i + e < n) v[e] = row[i + e];
    }
    return v;
}

// Pass 2.  grid = (requests x pieces, heads / heads_a_group), 256 threads; wavefront w has the chunk's tokens
// 16 w .. 16 w + 15, and the products C_t . B_s of its rows stay in registers for all heads that the workgroup takes.
// A lane (c, r) loads four neighbouring elements of a contraction of row r; element e is slot c of instruction e:
//   M^T = B C^T: the result leaves the lane with token t = r and keys s = 4 c .. 4 c + 3 of a tile: the second operand of
//   Y^T += (x dt)^T M^T (contraction over s), whose first operand comes from LDS, and of
//   Y^T += S C^T (contraction over n) with the entry state's rows straight from memory.
// LDS: x dt [SSD_CHUNK][XS], XS = 4 modulo 64 words: the rows 4 c + e of an instruction lie in different banks.
template <int NQ, bool WIDE>
__global__ __launch_bounds__(256) void ssd_chunk_out_kernel(SsdArgs a) {
    extern __shared__ float lds[];
    __shared__ float s_dt[SSD_CHUNK];
    const int s = blockIdx.x / a.pieces, piece = blockIdx.x % a.pieces, h0 = blockIdx.y * a.heads_a_group;
    const int q0 = a.cu_tokens[s], len = a.cu_tokens[s + 1] - q0;
    if (len <= SSD_WALK || piece * SSD_CHUNK >= len) return;
    const int t0 = q0 + piece * SSD_CHUNK, nt = min(SSD_CHUNK, len - piece * SSD_CHUNK);
    const int n = a.n, vdim = a.vdim, grp = h0 / (a.H / a.G), inner = a.H * vdim;
    const int XS = (vdim + 63) / 64 * 64 + 4, vp = XS - 4;
    float* s_x = lds;
    const int tid = threadIdx.x, wave = tid / LLE_WAVE, lane = tid % LLE_WAVE, c = lane / 16, r = lane % 16;
    const int64_t slot = ssd_slot(q0, s) + piece;
    const float* rows = a.c + (int64_t)t0 * a.CC;
    const int tok = wave * 16 + r;  // this lane's token of the chunk
    ssd_f32x4 C[NQ], cb[4];
    {
        const float* crow = rows + (int64_t)min(tok, nt - 1) * a.CC + inner + (a.G + grp) * n;
#pragma unroll
        for (int q = 0; q < NQ; ++q) C[q] = ssd_quad<WIDE>(crow, 16 * q + 4 * c, n);
    }
#pragma unroll
    for (int st = 0; st < 4; ++st) {
        cb[st] = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
        if (st <= wave) {
            const float* brow = rows + (int64_t)min(st * 16 + r, nt - 1) * a.CC + inner + grp * n;
#pragma unroll
            for (int q = 0; q < NQ; ++q) {
                const ssd_f32x4 b = ssd_quad<WIDE>(brow, 16 * q + 4 * c, n);
#pragma unroll
                for (int e = 0; e < 4; ++e) cb[st] = __builtin_amdgcn_mfma_f32_16x16x4f32(b[e], C[q][e], cb[st], 0, 0, 0);
            }
        }
    }
    for (int hh = 0; hh < a.heads_a_group; ++hh) {
        const int h = h0 + hh;
        // the entry state's first rows are asked for now, the later ones while the rows before them are multiplied
        const float* S = a.part + (slot * a.H + h) * (int64_t)vdim * n;
        ssd_f32x4 sv[NQ];
#pragma unroll
        for (int q = 0; q < NQ; ++q) sv[q] = ssd_quad<WIDE>(S + (int64_t)min(r, vdim - 1) * n, 16 * q + 4 * c, n);
        float dt, hi, lo;  // of token `lane` of the chunk (every wavefront makes them for itself)
        ssd_chunk_steps(a, h, t0, nt, dt, hi, lo);
        if (hh > 0) __syncthreads();  // (the head before has been read)
        if (wave == 0) s_dt[lane] = dt;
        __syncthreads();
        if (WIDE) {
            for (int e = tid; e < SSD_CHUNK * vp / 4; e += 256) {
                const int t = e / (vp / 4), i = (e - t * (vp / 4)) * 4;
                ssd_f32x4 v = {0.f, 0.f, 0.f, 0.f};
                if (t < nt && i < vdim) v = *(const ssd_f32x4*)(rows + (int64_t)t * a.CC + h * vdim + i) * s_dt[t];
                *(ssd_f32x4*)(s_x + t * XS + i) = v;
            }
        } else {
            for (int e = tid; e < SSD_CHUNK * vp; e += 256) {
                const int t = e / vp, i = e - t * vp;
                s_x[t * XS + i] = (t < nt && i < vdim) ? rows[(int64_t)t * a.CC + h * vdim + i] * s_dt[t] : 0.f;
            }
        }
        __syncthreads();
        const float hi_t = __shfl(hi, tok, LLE_WAVE), lo_t = __shfl(lo, tok, LLE_WAVE);
        ssd_f32x4 m[4];
#pragma unroll
        for (int st = 0; st < 4; ++st) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = st * 16 + 4 * c + e;
                const float hi_s = __shfl(hi, key, LLE_WAVE), lo_s = __shfl(lo, key, LLE_WAVE);
                // (later keys weigh nothing; their exponent would be above zero)
                m[st][e] = key <= tok ? cb[st][e] * expf((hi_t - hi_s) + (lo_t - lo_s)) : 0.f;
            }
        }
        const float entry = expf(hi_t), D = a.D[h];
        for (int jt = 0; jt * 16 < vdim; ++jt) {
            // (two chains of sums: a product waits for the one before it in its own chain only)
            ssd_f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = acc;
#pragma unroll
            for (int q = 0; q < NQ; ++q) {
#pragma unroll
                for (int e = 0; e < 4; e += 2) {
                    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[q][e], C[q][e], acc, 0, 0, 0);
                    acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[q][e + 1], C[q][e + 1], acc2, 0, 0, 0);
                }
            }
            const float* next = S + (int64_t)min((jt + 1) * 16 + r, vdim - 1) * n;
#pragma unroll
            for (int q = 0; q < NQ; ++q) sv[q] = ssd_quad<WIDE>(next, 16 * q + 4 * c, n);
            acc = (acc + acc2) * entry;
            acc2 = ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int st = 0; st < 4; ++st) {
                if (st <= wave) {  // (the same for the whole wavefront)
#pragma unroll
                    for (int e = 0; e < 4; e += 2) {
                        const float* x2 = s_x + (st * 16 + 4 * c + e) * XS + jt * 16 + r;
                        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x2[0], m[st][e], acc, 0, 0, 0);
                        acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x2[XS], m[st][e + 1], acc2, 0, 0, 0);
                    }
                }
            }
            acc += acc2;
            if (tok < nt) {
                const int j = jt * 16 + 4 * c;
                const float* x = rows + (int64_t)tok * a.CC + h * vdim;
                float* y = a.y + (int64_t)(t0 + tok) * inner + h * vdim;
                if (WIDE) {
                    if (j < vdim) *(ssd_f32x4*)(y + j) = *(const ssd_f32x4*)(x + j) * D + acc;
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (j + e < vdim) y[j + e] = fmaf(D, x[j + e], acc[e]);
                }
            }
        }
    }
}

extern "C" int lle_ssd_max_dim(void) { return 256; }
extern "C" int lle_ssd_chunk(void) { return SSD_CHUNK; }
extern "C" int lle_ssd_walk(void) { return SSD_WALK; }

// c float32 [N, CC], CC = H vdim + 2 G n; dt_in float32 rows of dt_cols; dt_bias, a_log, D float32 [H]; state rows of
// state_stride floats that begin with [H][vdim][n]; y float32 [N, H vdim].  `walk`: some request has at most SSD_WALK
// tokens; `pieces` > 0: chunks of the longest request (0: no request has more), with `part` float32
// [(N / SSD_CHUNK + S) H vdim n] and `part_decay` [(N / SSD_CHUNK + S) H].  heads_a_group divides H / G.
extern "C" int lle_ssd_scan(const void* c, int CC, const void* dt_in, int dt_cols, const void* dt_bias, const void* a_log,
                            const void* D, void* state, int64_t state_stride, const void* seq_slots, const void* cu_tokens, void* y,
                            int S, int H, int G, int vdim, int n, int walk, int pieces, int heads_a_group, void* part,
                            void* part_decay, hipStream_t stream) {
    if (S <= 0 || H <= 0) return 0;
    if (G <= 0 || H % G || vdim <= 0 || vdim > 256 || n <= 0 || n > 256 || H > 65535 || CC != H * vdim + 2 * G * n || dt_cols < H ||
        pieces < 0 || heads_a_group <= 0 || (H / G) % heads_a_group || (int64_t)S * (pieces > 0 ? pieces : 1) > 0x7fffffff ||
        (pieces > 0 && (!part || !part_decay)))
        return (int)hipErrorInvalidValue;
    const SsdArgs a{(const float*)c, CC, (const float*)dt_in, dt_cols, (const float*)dt_bias, (const float*)a_log, (const float*)D,
                    (float*)state, state_stride, (const int32_t*)seq_slots, (const int32_t*)cu_tokens, (float*)y, H, G, vdim, n,
                    heads_a_group, pieces, (float*)part, (float*)part_decay, (uintptr_t)state % 16 == 0 && state_stride % 4 == 0};
    if (walk) {
        const dim3 grid(S, H, (vdim + 15) / 16);
        if (n <= 16) ssd_walk_kernel<1><<<grid, 256, 0, stream>>>(a);
        else if (n <= 32) ssd_walk_kernel<2><<<grid, 256, 0, stream>>>(a);
        else if (n <= 64) ssd_walk_kernel<4><<<grid, 256, 0, stream>>>(a);
        else if (n <= 128) ssd_walk_kernel<8><<<grid, 256, 0, stream>>>(a);
        else ssd_walk_kernel<16><<<grid, 256, 0, stream>>>(a);
        const hipError_t e = hipGetLastError();
        if (e != hipSuccess || pieces == 0) return (int)e;
    }
    if (pieces == 0) return 0;
    {
        const int BS = (n + 63) / 64 * 64 + 16, XS = (vdim + 63) / 64 * 64 + 16;
        const size_t lds = ((size_t)SSD_CHUNK * (BS + XS) + SSD_CHUNK) * sizeof(float);
        auto go = [&](auto kernel) {
            if (lds > 64 * 1024) {
                const hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
                if (e != hipSuccess) return e;
            }
            kernel<<<dim3(S * pieces, H), 256, lds, stream>>>(a);
            return hipGetLastError();
        };
        const hipError_t e = vdim <= 16 ? go(ssd_chunk_state_kernel<1>) : vdim <= 32 ? go(ssd_chunk_state_kernel<2>) : go(ssd_chunk_state_kernel<4>);
        if (e != hipSuccess) return (int)e;
    }
    ssd_carry_kernel<<<dim3(S, H, (vdim * n + 255) / 256), 256, 0, stream>>>(a);
    hipError_t e = hipGetLastError();
    if (e != hipSuccess) return (int)e;
    const size_t lds = (size_t)SSD_CHUNK * ((vdim + 63) / 64 * 64 + 4) * sizeof(float);
    const bool wide = n % 4 == 0 && vdim % 4 == 0;  // (then CC and every column offset are multiples of 4 too)
    const dim3 grid(S * pieces, H / heads_a_group);
    auto go = [&](auto narrow_k, auto wide_k) {
        const void* k = wide ? (const void*)wide_k : (const void*)narrow_k;
        if (lds > 64 * 1024) {
            const hipError_t e2 = hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e2 != hipSuccess) return (int)e2;
        }
        if (wide) wide_k<<<grid, 256, lds, stream>>>(a);
        else narrow_k<<<grid, 256, lds, stream>>>(a);
        return (int)hipGetLastError();
    };
#define SSD_OUT_CASE(NQ) \
    if (n <= 16 * NQ) return go(ssd_chunk_out_kernel<NQ, false>, ssd_chunk_out_kernel<NQ, true>);
    SSD_OUT_CASE(1)
    SSD_OUT_CASE(2)
    SSD_OUT_CASE(3)
    SSD_OUT_CASE(4)
    SSD_OUT_CASE(6)
    SSD_OUT_CASE(8)
    SSD_OUT_CASE(12)
    SSD_OUT_CASE(16)
#undef SSD_OUT_CASE
    return (int)hipErrorInvalidValue;
}

// ---------------------------------------------------------------------------------
// out[n, :] = (y silu(z)) / rms(its part) * w: a row is cut into `groups` equal parts, each divided by its own root mean
// square.  z: the columns z0 .. of u.  A workgroup of 256 threads a (token, part); a thread keeps its share of the part in
// registers, in pieces of V elements (parts up to 256 x SSD_PER; wider ones are made twice).
// ---------------------------------------------------------------------------------
#define SSD_PER 32
template <typename T, int V>
__global__ __launch_bounds__(256) void ssd_gate_norm_kernel(const float* __restrict__ y, const T* __restrict__ u, int cols, int z0,
                                                             const float* __restrict__ w, float eps, T* __restrict__ out, int inner,
                                                             int width) {
    __shared__ float red[16];
    const int64_t n = blockIdx.x;
    const int p0 = blockIdx.y * width;
    const float* yr = y + n * inner + p0;
    const T* zr = u + n * cols + z0 + p0;
    T* dst = out + n * inner + p0;
    typedef T piece_t __attribute__((ext_vector_type(V)));
    typedef float fpiece_t __attribute__((ext_vector_type(V)));
    float keep[SSD_PER], ss = 0.f;
    const bool fits = width <= 256 * SSD_PER;
    if (fits) {
#pragma unroll
        for (int k = 0; k < SSD_PER; k += V) {
            const int i = (k / V * 256 + threadIdx.x) * V;
            if (k * 256 >= width) break;  // (the same for every thread)
            if (i < width) {  // (V divides the width and every offset)
                const fpiece_t yv = *(const fpiece_t*)(yr + i);
                const piece_t zv = *(const piece_t*)(zr + i);
#pragma unroll
                for (int e = 0; e < V; ++e) {
                    const float z = to_f32<T>(zv[e]);
                    keep[k + e] = yv[e] * z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.44269504088896340736f));
                    ss = fmaf(keep[k + e], keep[k + e], ss);
                }
            }
        }
    } else {
        for (int i = threadIdx.x; i < width; i += 256) {
            const float v = yr[i] * ssd_silu(to_f32<T>(zr[i]));
            ss = fmaf(v, v, ss);
        }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)width + eps);
    if (fits) {
#pragma unroll
        for (int k = 0; k < SSD_PER; k += V) {
            const int i = (k / V * 256 + threadIdx.x) * V;
            if (k * 256 >= width) break;
            if (i < width) {
                const fpiece_t wv = *(const fpiece_t*)(w + p0 + i);
                piece_t o;
#pragma unroll
                for (int e = 0; e < V; ++e) o[e] = from_f32<T>(keep[k + e] * inv * wv[e]);
                *(piece_t*)(dst + i) = o;
            }
        }
    } else {
        for (int i = threadIdx.x; i < width; i += 256)
            dst[i] = from_f32<T>(yr[i] * ssd_silu(to_f32<T>(zr[i])) * inv * w[p0 + i]);
    }
}

extern "C" int lle_ssd_gate_norm(const void* y, const void* u, int cols, int z0, const void* w, float eps, void* out, int N, int inner,
                                 int groups, int dtype, hipStream_t stream) {
    if (N <= 0 || inner <= 0) return 0;
    if (groups <= 0 || inner % groups || groups > 65535 || z0 < 0 || z0 + inner > cols) return (int)hipErrorInvalidValue;
    const dim3 grid(N, groups);
    const bool wide = (inner / groups) % 4 == 0 && cols % 4 == 0 && z0 % 4 == 0;
#define SSD_GATE(T, V)                                                                                                         \
    ssd_gate_norm_kernel<T, V><<<grid, 256, 0, stream>>>((const float*)y, (const T*)u, cols, z0, (const float*)w, eps, (T*)out, inner, \
                                                         inner / groups)
    if (dtype == LLE_F32) {
        if (wide) SSD_GATE(float, 4); else SSD_GATE(float, 1);
    } else {
        if (wide) SSD_GATE(bf16_t, 4); else SSD_GATE(bf16_t, 1);
    }
#undef SSD_GATE
    LLE_RETURN_LAUNCH_STATUS();
}
