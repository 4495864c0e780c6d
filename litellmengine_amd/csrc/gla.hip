// Gated linear attention: a recurrence with a matrix state per head whose rows decay each at a rate of its own,
// made from the data.
//
//   decay_t = sigmoid(z_t)^(1 / tau),  z_t = a2 low_t + b       per head and key channel, 32-bit        gla_decay
//   S[i][j] <- decay_t[i] S[i][j] + k_t[i] v_t[j]                                                       gla_scan
//   o_t[j]   = sum_i q_scale q_t[i] S[i][j]                     (the read-out sees the token's own write)
//   y_t      = o_t / rms(o_t) * norm_w * silu(g_t)              per head, eps inside the root, norm_w [vdim] for all heads
//
// The state is float32 [head][key i][value j] per request slot.  A row of `u` holds q [H dim], k [H dim], v [H vdim]
// and g [H vdim] of a token as the projection left them.  A thread owns one value channel j of one head and a
// quarter of the key channels of S[:, j] in registers; q, k and the decays of a few tokens are staged in LDS,
// where every thread reads the same word at a time (a broadcast).
//
// The state is linear in what came before: S_out = diag(A) S_in + B, A the product of a stretch's decays.  A long
// portion is therefore cut into pieces that are walked side by side:
//   pass 1  every piece but a request's last, from a zero state: A, and B = sum_t (k_t times the decays behind t) v_t^T, a
//           product on the 32-bit matrix instruction (products of decays never grow, so nothing is ever divided)
//   carry   a short walk over the pieces leaves every piece's entry state
//   pass 2  every piece again from its entry state, with outputs; the last writes the state back
// A step of single tokens, or of short portions, is one launch from the state itself.
#include "common.h"

LLE_DEFINE_ERROR_STRING()

// decay[n][c] = exp(log(sigmoid(z)) / tau), z = sum_r low[n][r] a2[r][c] + b[c]; low float32 [N, R], a2 float32 [R, C].
// grid = (blocks of 256 channels, runs of GD_TOKENS tokens): a thread reads its column of a2 once for the run.
#define GD_TOKENS 8
__device__ __forceinline__ float gla_decay_of(float z, float inv_tau) {
    // log2(sigmoid(z)) = min(z, 0) log2 e - log2(1 + x), x = e^-|z|: no overflow at either end; a small x takes the
    // first terms of the series (1 + x would round them away)
    const float x = __builtin_amdgcn_exp2f(-fabsf(z) * 1.44269504088896340736f);
    const float series = x * (1.f - x * (0.5f - x * 0.33333333333f)) * 1.44269504088896340736f;
    const float log2_1px = x < 0.01f ? series : __builtin_amdgcn_logf(1.0f + x);
    return __builtin_amdgcn_exp2f((fminf(z, 0.f) * 1.44269504088896340736f - log2_1px) * inv_tau);
}

__global__ __launch_bounds__(256) void gla_decay_kernel(const float* __restrict__ low, const float* __restrict__ a2,
                                                         const float* __restrict__ b, float* __restrict__ decay, int N,
                                                         int R, int C, float inv_tau) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    const int n0 = blockIdx.y * GD_TOKENS;
    if (c >= C) return;
    float z[GD_TOKENS];
#pragma unroll
    for (int t = 0; t < GD_TOKENS; ++t) z[t] = b[c];
#pragma unroll 8
    for (int r = 0; r < R; ++r) {
        const float w = a2[(int64_t)r * C + c];
#pragma unroll
        for (int t = 0; t < GD_TOKENS; ++t) z[t] = fmaf(low[(int64_t)min(n0 + t, N - 1) * R + r], w, z[t]);  // (the same for all lanes)
    }
#pragma unroll
    for (int t = 0; t < GD_TOKENS; ++t)
        if (n0 + t < N) decay[(int64_t)(n0 + t) * C + c] = gla_decay_of(z[t], inv_tau);
}

extern "C" int lle_gla_decay(const void* low, const void* a2, const void* b, void* decay, int N, int R, int C, float tau,
                             hipStream_t stream) {
    if (N <= 0 || C <= 0) return 0;
    if (R <= 0 || !(tau > 0.f)) return (int)hipErrorInvalidValue;
    const int64_t runs = ((int64_t)N + GD_TOKENS - 1) / GD_TOKENS;
    if (runs > 65535) return (int)hipErrorInvalidValue;
    gla_decay_kernel<<<dim3((C + 255) / 256, (int)runs), 256, 0, stream>>>((const float*)low, (const float*)a2, (const float*)b,
                                                                           (float*)decay, N, R, C, 1.0f / tau);
    LLE_RETURN_LAUNCH_STATUS();
}

struct GlaArgs {
    const void* u;  // [N, cols], activation type
    int cols;
    const float* decay;  // [N, H dim]
    float q_scale;
    const float* norm_w;  // [vdim]
    float eps;
    float* state;  // [slots, state_stride]
    int64_t state_stride;
    const int32_t* seq_slots;
    const int32_t* cu_tokens;
    void* out;  // [N, H vdim], activation type
    int H, dim, vdim;
    int jt_log2;  // log2 of a group's threads: 64, 128 or 256, at least vdim
    int pieces, piece_len;
    float* part;  // [S, pieces, H, dim * vdim + dim]: B (then the entry state) and A of every piece
};

#define GLA_FROM_STATE 0  // one walk over a request's tokens
#define GLA_FROM_ENTRY 1  // pass 2
#define GLA_TC 8          // tokens staged at a time
#define GLA_IG 4          // groups of threads that share a value channel's key channels

// grid = (requests x pieces, heads).  KD >= dim (a multiple of 16) key channels are kept; a workgroup is GLA_IG groups
// of `jt` threads: thread (ig, j) owns value channel j and the key channels [ig KD / GLA_IG, (ig + 1) KD / GLA_IG).
// The groups' shares of o_t meet in LDS (dynamic: [GLA_IG][GLA_TC][jt]).
// MAXT: the most threads of a workgroup (wide heads take 512 where these are enough: twice the registers a thread).
template <int KD, typename T, int MODE, int MAXT>
__global__ __launch_bounds__(MAXT) void gla_scan_kernel(GlaArgs a) {
    constexpr int KI = KD / GLA_IG;
    static_assert(KD % GLA_IG == 0, "the key channels are dealt to the groups in equal shares");
    __shared__ float s_q[GLA_TC][KD], s_k[GLA_TC][KD], s_w[GLA_TC][KD];
    __shared__ float s_inv[GLA_TC];
    extern __shared__ float s_o[];
    const int dim = a.dim, vdim = a.vdim, HK = a.H * dim, HV = a.H * vdim, jt = 1 << a.jt_log2;
    const int s = blockIdx.x / a.pieces, piece = blockIdx.x % a.pieces;
    const int h = blockIdx.y;
    const int tid = threadIdx.x;
    const int j = tid & (jt - 1), ig = tid >> a.jt_log2, i0 = ig * KI;
    const int q0 = a.cu_tokens[s], q1 = a.cu_tokens[s + 1];
    const int live = (q1 - q0 + a.piece_len - 1) / a.piece_len;  // pieces of this request that hold tokens
    if (piece >= live) return;
    const int t0 = q0 + piece * a.piece_len, t1 = min(q1, t0 + a.piece_len);
    float* srow = a.state + (int64_t)a.seq_slots[s] * a.state_stride + (int64_t)h * dim * vdim;
    float* prow = a.part ? a.part + ((int64_t)(s * a.pieces + piece) * a.H + h) * (dim * vdim + dim) : nullptr;
    const T* u = (const T*)a.u;

    float S[KI];
#pragma unroll
    for (int ii = 0; ii < KI; ++ii) {
        const int i = i0 + ii;
        float x = 0.f;
        if (MODE == GLA_FROM_STATE && i < dim && j < vdim) x = srow[i * vdim + j];
        if (MODE == GLA_FROM_ENTRY && i < dim && j < vdim) x = prow[i * vdim + j];
        S[ii] = x;
    }
    for (int c0 = t0; c0 < t1; c0 += GLA_TC) {
        const int nt = min(GLA_TC, t1 - c0);
        __syncthreads();  // (the chunk before has been read)
        for (int idx = tid; idx < GLA_TC * KD; idx += blockDim.x) {
            const int t = idx / KD, i = idx - t * KD;
            // past the chunk's last token: nothing is written and nothing decays
            float qq = 0.f, kk = 0.f, ww = 1.0f;
            if (t < nt && i < dim) {
                const T* row = u + (int64_t)(c0 + t) * a.cols + h * dim + i;
                qq = to_f32<T>(row[0]) * a.q_scale;
                kk = to_f32<T>(row[HK]);
                ww = a.decay[(int64_t)(c0 + t) * HK + h * dim + i];
            }
            s_q[t][i] = qq;
            s_k[t][i] = kk;
            s_w[t][i] = ww;
        }
        float vv[GLA_TC];
#pragma unroll
        for (int t = 0; t < GLA_TC; ++t)
            vv[t] = (t < nt && j < vdim) ? to_f32<T>(u[(int64_t)(c0 + t) * a.cols + 2 * HK + h * vdim + j]) : 0.f;
        __syncthreads();
#pragma unroll
        for (int t = 0; t < GLA_TC; ++t) {
            // (the branch also keeps a token's operands from being read long before its turn: all of a chunk's at
            // once do not fit the registers)
            if (t < nt) {
                float o = 0.f;
#pragma unroll
                for (int ii = 0; ii < KI; ++ii) {
                    const int i = i0 + ii;
                    S[ii] = fmaf(s_w[t][i], S[ii], s_k[t][i] * vv[t]);
                    o = fmaf(s_q[t][i], S[ii], o);
                }
                s_o[(ig * GLA_TC + t) * jt + j] = o;
            }
        }
        __syncthreads();
        // the groups' shares are added up, and every token's head is divided by its own root mean square:
        // a wavefront per token
        const int wave = tid / LLE_WAVE, lane = tid % LLE_WAVE, waves = blockDim.x / LLE_WAVE;
        for (int t = wave; t < nt; t += waves) {
            float ss = 0.f;
            for (int e = lane; e < vdim; e += LLE_WAVE) {
                float o = s_o[t * jt + e];
#pragma unroll
                for (int g2 = 1; g2 < GLA_IG; ++g2) o += s_o[(g2 * GLA_TC + t) * jt + e];
                s_o[t * jt + e] = o;
                ss += o * o;
            }
            ss = wave_sum(ss);
            if (lane == 0) s_inv[t] = 1.0f / sqrtf(ss / (float)vdim + a.eps);
        }
        __syncthreads();
        for (int t = ig; t < nt; t += GLA_IG) {
            if (j < vdim) {
                const float gate = to_f32<T>(u[(int64_t)(c0 + t) * a.cols + 2 * HK + HV + h * vdim + j]);
                const float y = s_o[t * jt + j] * s_inv[t] * a.norm_w[j] * (gate / (1.0f + expf(-gate)));
                ((T*)a.out)[(int64_t)(c0 + t) * HV + h * vdim + j] = from_f32<T>(y);
            }
        }
    }
    if (piece != live - 1) return;
    if (j < vdim) {
#pragma unroll
        for (int ii = 0; ii < KI; ++ii)
            if (i0 + ii < dim) srow[(i0 + ii) * vdim + j] = S[ii];
    }
}

// Pass 1: grid = (requests x pieces, heads), 256 threads; every piece but a request's last is whole.  The decays behind a
// token are multiplied up in four groups of tokens side by side (a thread has sixteen tokens of a channel, NI channels one
// after the other, everything asked for at once); k times them (float32) and v wait in LDS, and B [dim, vdim] = sum over the
// tokens is taken in 16 x 16 tiles, four tokens an instruction.
// LDS: k [tokens][KS], v [tokens][VS] (row strides of 16 modulo 64: the operands' rows lie in different banks), the
// groups' products [4][dim].
#define GLA_PIECE 64
#define GLA_QUARTER (GLA_PIECE / 4)
typedef float gla_f32x4 __attribute__((ext_vector_type(4)));
template <typename T, int NI>
__global__ __launch_bounds__(256) void gla_piece_kernel(GlaArgs a) {
    extern __shared__ float lds[];
    const int dim = a.dim, vdim = a.vdim, HK = a.H * dim;
    const int KS = (dim + 63) / 64 * 64 + 16, VS = (vdim + 63) / 64 * 64 + 16;
    const int s = blockIdx.x / a.pieces, piece = blockIdx.x % a.pieces, h = blockIdx.y;
    const int q0 = a.cu_tokens[s], q1 = a.cu_tokens[s + 1];
    const int live = (q1 - q0 + GLA_PIECE - 1) / GLA_PIECE;
    if (piece >= live - 1) return;  // nobody comes after the last piece
    const int t0 = q0 + piece * GLA_PIECE;
    float* s_k = lds;
    float* s_v = s_k + GLA_PIECE * KS;
    float* s_g = s_v + GLA_PIECE * VS;
    float* prow = a.part + ((int64_t)(s * a.pieces + piece) * a.H + h) * (dim * vdim + dim);
    const T* u = (const T*)a.u;
    const int wave = threadIdx.x / LLE_WAVE, lane = threadIdx.x % LLE_WAVE, c = lane / 16, r = lane % 16;
    // wavefront g has the tokens g 16 .. g 16 + 15; lane + 64 n is its channel
    const int g = wave, first = t0 + g * GLA_QUARTER;
    float w[NI][GLA_QUARTER], k[NI][GLA_QUARTER];
#pragma unroll
    for (int n = 0; n < NI; ++n) {
        const int i = min(lane + LLE_WAVE * n, dim - 1);
#pragma unroll
        for (int t = 0; t < GLA_QUARTER; ++t) {
            w[n][t] = a.decay[(int64_t)(first + t) * HK + h * dim + i];
            k[n][t] = to_f32<T>(u[(int64_t)(first + t) * a.cols + HK + h * dim + i]);
        }
    }
    for (int j = lane; j < VS - 16; j += LLE_WAVE) {
        float v[GLA_QUARTER];
#pragma unroll
        for (int t = 0; t < GLA_QUARTER; ++t) v[t] = to_f32<T>(u[(int64_t)(first + t) * a.cols + 2 * HK + h * vdim + min(j, vdim - 1)]);
#pragma unroll
        for (int t = 0; t < GLA_QUARTER; ++t) s_v[(g * GLA_QUARTER + t) * VS + j] = j < vdim ? v[t] : 0.f;
    }
#pragma unroll
    for (int n = 0; n < NI; ++n) {
        const int i = lane + LLE_WAVE * n;
        float p = 1.f;
#pragma unroll
        for (int t = 0; t < GLA_QUARTER; ++t) p *= w[n][t];
        if (i < dim) s_g[g * dim + i] = p;
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < NI; ++n) {
        const int i = lane + LLE_WAVE * n;
        float run = 1.f;
        if (i < dim)
            for (int later = g + 1; later < 4; ++later) run *= s_g[later * dim + i];
#pragma unroll
        for (int t = GLA_QUARTER - 1; t >= 0; --t) {
            // (channels past the last one fill the last tile of sixteen with zeros)
            if (i < KS - 16) s_k[(g * GLA_QUARTER + t) * KS + i] = i < dim ? k[n][t] * run : 0.f;
            run *= w[n][t];
        }
        if (g == 0 && i < dim) prow[dim * vdim + i] = run;
    }
    __syncthreads();
    const int row_tiles = (dim + 15) / 16, col_tiles = (vdim + 15) / 16;
    for (int tile = wave; tile < row_tiles * col_tiles; tile += 4) {
        const int i0 = tile / col_tiles * 16, j0 = (tile - tile / col_tiles * col_tiles) * 16;
        gla_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < GLA_PIECE; t += 4)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(s_k[(t + c) * KS + i0 + r], s_v[(t + c) * VS + j0 + r], acc, 0, 0, 0);
#pragma unroll
        for (int n = 0; n < 4; ++n)
            if (i0 + 4 * c + n < dim && j0 + r < vdim) prow[(i0 + 4 * c + n) * vdim + j0 + r] = acc[n];
    }
}

// grid = (requests, heads, blocks of 256 state elements): a thread walks one element S[i][j] through the
// pieces and leaves every piece's entry state in the place of its B (eight pieces' A and B are asked
// for together: one after the other, each would wait for the memory on its own)
__global__ __launch_bounds__(256) void gla_carry_kernel(GlaArgs a) {
    const int s = blockIdx.x, h = blockIdx.y;
    const int elems = a.dim * a.vdim;
    const int e = blockIdx.z * blockDim.x + threadIdx.x;
    if (e >= elems) return;
    const int i = e / a.vdim;
    const int q0 = a.cu_tokens[s], q1 = a.cu_tokens[s + 1];
    const int live = (q1 - q0 + a.piece_len - 1) / a.piece_len;
    const int64_t stride = (int64_t)a.H * (elems + a.dim);
    float* base = a.part + ((int64_t)s * a.pieces * a.H + h) * (elems + a.dim);
    float S = a.state[(int64_t)a.seq_slots[s] * a.state_stride + (int64_t)h * elems + e];
    for (int p0 = 0; p0 < live; p0 += 8) {
        float A[8], B[8];
#pragma unroll
        for (int n = 0; n < 8; ++n) {
            const int p = min(p0 + n, live - 1);
            B[n] = base[p * stride + e];
            A[n] = base[p * stride + elems + i];
        }
#pragma unroll
        for (int n = 0; n < 8; ++n) {
            if (p0 + n < live) {
                base[(p0 + n) * stride + e] = S;
                S = A[n] * S + B[n];  // (the last piece has left no A and B; what S becomes there is not used)
            }
        }
    }
}

template <int KD, typename T, int MAXT>
static int gla_launch_of(const GlaArgs& a, int S, hipStream_t stream) {
    const int threads = GLA_IG << a.jt_log2;
    const size_t smem = (size_t)GLA_TC * threads * sizeof(float);
    const dim3 grid(S * a.pieces, a.H);
    if (a.pieces == 1) {
        gla_scan_kernel<KD, T, GLA_FROM_STATE, MAXT><<<grid, threads, smem, stream>>>(a);
        return (int)hipGetLastError();
    }
    const int KS = (a.dim + 63) / 64 * 64 + 16, VS = (a.vdim + 63) / 64 * 64 + 16;
    const size_t piece_smem = ((size_t)GLA_PIECE * (KS + VS) + 4 * a.dim) * sizeof(float);
    auto piece = [&](auto kernel) {
        if (piece_smem > 64 * 1024) {
            const hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)piece_smem);
            if (e != hipSuccess) return e;
        }
        kernel<<<grid, 256, piece_smem, stream>>>(a);
        return hipGetLastError();
    };
    hipError_t e = a.dim <= 64 ? piece(gla_piece_kernel<T, 1>) : a.dim <= 128 ? piece(gla_piece_kernel<T, 2>) : piece(gla_piece_kernel<T, 4>);
    if (e != hipSuccess) return (int)e;
    gla_carry_kernel<<<dim3(S, a.H, (a.dim * a.vdim + 255) / 256), 256, 0, stream>>>(a);
    e = hipGetLastError();
    if (e != hipSuccess) return (int)e;
    gla_scan_kernel<KD, T, GLA_FROM_ENTRY, MAXT><<<grid, threads, smem, stream>>>(a);
    return (int)hipGetLastError();
}

template <int KD, typename T>
static int gla_launch(const GlaArgs& a, int S, hipStream_t stream) {
    if constexpr (KD >= 96) {
        if (GLA_IG << a.jt_log2 <= 512) return gla_launch_of<KD, T, 512>(a, S, stream);
    }
    return gla_launch_of<KD, T, 1024>(a, S, stream);
}

extern "C" int lle_gla_max_dim(void) { return 256; }
extern "C" int lle_gla_piece(void) { return GLA_PIECE; }

// u [N, cols] in `dtype`: q, k, v, g in this order; decay float32 [N, H dim]; state float32 rows of `state_stride` floats
// that begin with H dim vdim of the matrix state.  `pieces` > 1 needs `part`, float32 [S pieces H (dim vdim + dim)]; every
// request has at most pieces * piece_len tokens: 64 of them in a piece, where there are several.
extern "C" int lle_gla_scan(const void* u, int cols, const void* decay, float q_scale, const void* norm_w, float eps, void* state,
                            int64_t state_stride, const void* seq_slots, const void* cu_tokens, void* out, int S, int H, int dim,
                            int vdim, int pieces, int piece_len, void* part, int dtype, hipStream_t stream) {
    if (S <= 0 || H <= 0) return 0;
    if (dim <= 0 || dim > 256 || vdim <= 0 || vdim > 256 || pieces < 1 || piece_len < 1 ||
        (pieces > 1 && (part == nullptr || piece_len != GLA_PIECE)) ||
        H > 65535 || (int64_t)S * pieces > 0x7fffffff || cols < 2 * H * (dim + vdim))
        return (int)hipErrorInvalidValue;
    // a group has as many threads as there are value channels
    const int jt_log2 = vdim <= 64 ? 6 : vdim <= 128 ? 7 : 8;
    const GlaArgs a{u, cols, (const float*)decay, q_scale, (const float*)norm_w, eps, (float*)state, state_stride,
                    (const int32_t*)seq_slots, (const int32_t*)cu_tokens, out, H, dim, vdim, jt_log2, pieces, piece_len,
                    (float*)part};
#define GLA_CASE(KD)                                                                    \
    if (dim <= KD)                                                                      \
        return dtype == LLE_F32 ? gla_launch<KD, float>(a, S, stream) : gla_launch<KD, bf16_t>(a, S, stream);
    GLA_CASE(16)
    GLA_CASE(32)
    GLA_CASE(48)
    GLA_CASE(64)
    GLA_CASE(96)
    GLA_CASE(128)
    GLA_CASE(192)
    GLA_CASE(256)
#undef GLA_CASE
    return (int)hipErrorInvalidValue;
}
