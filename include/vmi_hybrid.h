/* C-ABI of libvmi_hybrid.so — the layers of decoders that mix recurrences, linear attention and softmax attention (vllmini_amd/hybrid_ops.py
 * is its only caller).  One library for every step shape: a packed batch of T tokens that belong to B sequences ("entries"), each
 * with a portion of q_len >= 1 new tokens behind ctx tokens already held in the paged cache / the state slots.
 *
 * Element types (`dtype`): VMI_HY_BF16 — activations and weights in bfloat16 on v_mfma_f32_16x16x32_bf16, fp32 accumulation;
 * VMI_HY_F32 — the same kernels in float32 on v_mfma_f32_16x16x4_f32 (no reduced-precision products).  In both the residual
 * stream, norms, positions and angles, attention scores and weights, the recurrence's gates, decays and state are float32.
 *
 * Sizes: every row length handed over is a multiple of 32 elements (the loader pads heads, blocks and ranks with zero weights);
 * the true lengths that enter an average (norms) are arguments.
 *
 * Weights come as MFMA tiles: [group][N / 16][K / 32][64][8] with tile[s][t][kc * 16 + r][e] = w[16 s + r][32 t + 8 kc + e].
 *
 * Plain pointers and sizes, nothing retained, never synchronises; every entry returns 0 or a VMI_HY_E_* code and
 * vmi_hybrid_last_error() names the reason (thread-local). */
#ifndef VMI_HYBRID_H
#define VMI_HYBRID_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define VMI_HY_API __attribute__((visibility("default")))
#define VMI_HYBRID_ABI_VERSION 2

enum { VMI_HY_OK = 0, VMI_HY_E_ARG = 1, VMI_HY_E_SHAPE = 2, VMI_HY_E_HIP = 3 };
enum { VMI_HY_BF16 = 0, VMI_HY_F32 = 1 };

/* what a linear layer reads and what it does with the product */
enum {
  VMI_HY_X_ROWS = 0,    /* x: [M, K] of the element type */
  VMI_HY_X_NORM = 1,    /* x: float32 [M, K]; layer norm (`rms`: RMS norm) over the first norm_n columns with norm_w (float32 [K]), no bias */
  VMI_HY_X_CONCAT = 2,  /* x, x2: float32 [M, K / 2] each, side by side */
};
enum {
  VMI_HY_E_STORE = 0,     /* y (element type) = acc + bias */
  VMI_HY_E_RESIDUAL = 1,  /* y (float32) += acc */
  VMI_HY_E_FLOAT = 2,     /* y (float32) = acc * scale, columns below n_out only */
  VMI_HY_E_GLU = 3,       /* columns interleaved (gate, up): y (element type, N / 2 columns) = the gated unit of `scale` (its limit), glu_alpha, glu_up */
  VMI_HY_E_GATED = 4,     /* y (element type) = acc * sigmoid(gate[row * ldg + group]) */
  VMI_HY_E_STORE_GLU = 5, /* columns below n_split (a multiple of 16): y (element type) = acc; the others, interleaved: y2 = the gated unit */
};

typedef struct {
  const void* x;
  const void* x2;
  const int32_t* rows;   /* X_NORM: row m reads x[rows[m]] (NULL: x[m]) */
  const float* norm_w;
  const void* w;
  const float* bias;
  const void* gate;
  void* y;
  void* y2;
  int64_t ldx, ldy, ldg, ldy2;
  int64_t x_gstride, y_gstride;   /* elements from one group to the next */
  int32_t M, N, K, groups;
  int32_t norm_n, n_out, n_split, rms;
  float eps, scale, glu_alpha, glu_up;   /* gated unit: g = min(g, limit), u = clamp(u, limit): g sigmoid(alpha g) (u + glu_up) */
  int32_t x_kind, epilogue, dtype, device;
} vmi_hy_linear_args;
VMI_HY_API int vmi_hy_linear(const vmi_hy_linear_args* a, void* stream);

/* x[t, 0:width) = table[ids[t]] * scale (bfloat16 table of row length ld), zeros up to ld; float32 out */
VMI_HY_API int vmi_hy_embed(const int64_t* ids, const void* table, float* x, int32_t T, int32_t width, int32_t ld, int32_t vocab,
                            float scale, int32_t device, void* stream);

/* optional x += add (element type [T, ld]); then out (element type [T, ld]) = layer norm (`rms`: RMS norm) of x (float32 [T, ld]);
 * out may be NULL */
VMI_HY_API int vmi_hy_add_norm(float* x, const void* add, int64_t ld_add, const float* norm_w, void* out, int32_t T, int32_t n,
                               int32_t ld, float eps, int32_t rms, int32_t dtype, int32_t device, void* stream);

/* x (float32 [T, ld]) += scale * (RMS norm of a with wa + RMS norm of b with wb) + add; a, b, add element type [T, ..], add may be
 * NULL; norms over n columns */
VMI_HY_API int vmi_hy_merge(float* x, const void* a, int64_t ld_a, const void* b, int64_t ld_b, const void* add, int64_t ld_add,
                            const float* wa, const float* wb, int32_t T, int32_t n, int32_t ld, float eps, float scale, int32_t dtype,
                            int32_t device, void* stream);

/* out[t, j] = gated unit (limit, alpha, up) of in[t, 2 j], in[t, 2 j + 1]; n output columns */
VMI_HY_API int vmi_hy_glu(const void* in, int64_t ld_in, void* out, int64_t ld_out, int32_t T, int32_t n, float limit, float alpha,
                          float up, int32_t dtype, int32_t device, void* stream);

/* out [T, 2 n] = (x | x2) in the element type, x and x2 float32 [T, n] */
VMI_HY_API int vmi_hy_concat(const float* x, const float* x2, void* out, int32_t T, int32_t n, int32_t dtype, int32_t device,
                             void* stream);

/* index of the largest of each row's first V values (first maximum on ties) */
VMI_HY_API int vmi_hy_argmax(const float* logits, int64_t ld, int32_t rows, int32_t V, int64_t* out, int32_t device, void* stream);

/* The step's layout, shared by the kernels below (all device pointers). */
typedef struct {
  const int32_t* tok_seq;    /* [T] entry of the token, -1: padding row */
  const int32_t* tok_pos;    /* [T] position in its sequence */
  const int32_t* tok_slot;   /* [T] cache row of the token (page * page_size + offset), -1: none */
  const int32_t* q_start;    /* [B] first token of the entry's portion */
  const int32_t* q_len;      /* [B] */
  const int32_t* ctx;        /* [B] tokens before the portion */
  const int32_t* state_slot; /* [B] */
  const int32_t* flip;       /* [B] which half of the convolution tail holds the inputs before the portion (0 / 1) */
  const int32_t* table;      /* [B, table_ld] pages */
  const int32_t* chunks;     /* [n_chunks][2]: (entry, first row inside its portion) of every run of up to 16 rows */
  const int32_t* chunk_start;/* [B] first chunk of the entry */
  int32_t T, B, table_ld, page_size, n_chunks;
} vmi_hy_step;

/* The recurrent block between its input and output projections: causal convolution, block-diagonal gates, the gated linear
 * recurrence, and the product with gelu(y).  yx [T, ldx]: columns [0, width) = y before its activation, [width, 2 width) = the
 * convolution's input.  Rows are processed in tiles of 64 (16 when `single`: every portion is one token); sequences that span
 * tiles need `spans` != 0 and the scratch: float32 [2][T][width] and [ceil(T / 64)][width]. */
typedef struct {
  const void* yx;
  void* out;              /* [T, ldo] element type */
  const float* conv_w;    /* [taps][width] */
  const float* conv_b;    /* [width] */
  const void* gates;      /* element type, tiles of ra then ri: [2][blocks][bw / 16][bw / 32][64][8] */
  const float* gate_b;    /* [2][width] */
  const float* decay;     /* [width]: -8 softplus(lam) */
  float* state;           /* [slots][width] */
  void* tail;             /* [slots][2][taps - 1][width] element type */
  float* scratch;
  float* carry;
  int64_t ldx, ldo;
  int32_t width, blocks, taps, single, spans, dtype, device;
} vmi_hy_rglru_args;
VMI_HY_API int vmi_hy_rglru(const vmi_hy_rglru_args* a, const vmi_hy_step* s, void* stream);

/* Latent attention, what follows the projections: proj [T, ldp] = per head [dim | rot], then [rank | rot], then gates.
 * Writes the token's cache row [rank | rot] (RMS norm of the latent, rotated shared key) and the rotated query parts into
 * q [T, heads, rank + rot] at offset rank.  rot_n / rank_n: the true sizes; freq float64 [rot_n / 2]. */
typedef struct {
  const void* proj;
  void* q;
  void* cache;            /* [pages][page_size][rank + rot] element type */
  const float* norm_w;    /* [rank] */
  const double* freq;
  int64_t ldp;
  int32_t heads, dim, rot, rank, rot_n, rank_n;
  float eps;
  int32_t dtype, device;
} vmi_hy_latent_prep_args;
VMI_HY_API int vmi_hy_latent_prep(const vmi_hy_latent_prep_args* a, const vmi_hy_step* s, void* stream);

/* out [T, heads, rank] = softmax(scale * q . k) . latent over the visible cache rows (causal).  Query rows of an entry are
 * (token, head) pairs, head fastest, cut into tiles of 16 * row_tiles: tiles [n_tiles][2] = (entry, first row), entry -1: none.  splits > 1: the
 * keys of a tile are dealt to that many workgroups, partial float32 [splits][T * heads][rank + 2]. */
typedef struct {
  const void* q;
  const void* cache;
  void* out;
  const int32_t* tiles;
  float* partial;
  int32_t heads, rank, rot, n_tiles, row_tiles, splits;
  float scale;
  int32_t dtype, device;
} vmi_hy_latent_attention_args;
VMI_HY_API int32_t vmi_hy_latent_row_tiles(int32_t row_dim, int32_t want, int32_t dtype);   /* 1, 2 or 4, at most `want` */
VMI_HY_API int vmi_hy_latent_attention(const vmi_hy_latent_attention_args* a, const vmi_hy_step* s, void* stream);

/* Linear attention with a matrix state per head, S [dim, vdim] float32 (csrc/hybrid_state.hip).  proj [T, ldp] begins with the
 * columns q [kv_heads dim] | k [kv_heads dim] | v [heads vdim]; head h uses q / k head h / (heads / kv_heads).
 *   VMI_HY_RETENTION  q and k rotated (first rot_n dimensions of a head), k / sqrt(dim_n), S <- d S + k v^T, o = S^T q; d per head
 *   VMI_HY_DELTA      q, k, v through a causal convolution and silu, q and k to unit length, q / sqrt(dim_n);
 *                     S <- g S (g per row), u = sigmoid(beta) (v - S^T k), S <- S + k u^T, o = S^T q,
 *                     g = exp(-rate_h softplus(z + dt_bias))
 * A step of single tokens (`single`) is one pass over the states; otherwise portions are cut into chunks of 16 rows whose inner
 * products are prepared independently (scratch: vmi_hy_state_scratch floats per (chunk, head)) and walked once per state.
 * out = o / rms(o) (over vdim_n) * norm_w (NULL: 1) * act(gate), per head.  A step of single tokens finishes its rows by itself where
 * one workgroup holds a head (vmi_hy_state_fuses); where not, o (float32 [T, heads vdim]) holds them in between. */
enum { VMI_HY_RETENTION = 0, VMI_HY_DELTA = 1 };
enum { VMI_HY_ACT_SIGMOID = 0, VMI_HY_ACT_SILU = 1 };
typedef struct {
  const void* proj;
  const void* beta;        /* [T, ldp] one column per head, before the sigmoid */
  const void* z;           /* [T, ldz] heads dim columns */
  const float* conv_w;     /* [taps][2 kv_heads dim + heads vdim] */
  const float* rate;       /* [heads]: DELTA exp(A_log) */
  const float* dt_bias;    /* [heads dim] */
  const float* decay;      /* [heads]: RETENTION */
  const float* log2_decay; /* [heads] */
  const float* turns;      /* [T][rot_n / 2][2]: what vmi_hy_rotations wrote */
  float* state;            /* [slots][heads][dim][vdim] */
  void* tail;              /* [slots][2][taps - 1][2 kv_heads dim + heads vdim] element type */
  float* o;                /* single and not fused */
  float* scratch;          /* not single */
  void* out;               /* [T, ldo] heads vdim columns */
  const void* gate;        /* [T, ldg] heads vdim columns */
  const float* norm_w;     /* [vdim] or NULL */
  int64_t ldp, ldz, ldo, ldg;
  int32_t heads, kv_heads, dim, vdim, dim_n, vdim_n, taps, rot_n, kind, single, act;
  float eps;
  int32_t dtype, device;
} vmi_hy_state_args;
/* out [T][half][2] = cos, sin of tok_pos[t] * freq[i]: once per step for all layers of one set of frequencies */
VMI_HY_API int vmi_hy_rotations(const double* freq, int32_t half, float* out, const vmi_hy_step* s, int32_t device, void* stream);
VMI_HY_API int64_t vmi_hy_state_scratch(int32_t kind, int32_t dim, int32_t vdim);
VMI_HY_API int32_t vmi_hy_state_fuses(int32_t dim, int32_t vdim);
VMI_HY_API int vmi_hy_state(const vmi_hy_state_args* a, const vmi_hy_step* s, void* stream);

/* Grouped-query softmax attention over a paged cache of rows [kv_heads][dim | vdim] (csrc/hybrid_attention.hip).
 * prep: proj [T, ldp] = q [heads dim] | k [kv_heads dim] | v [kv_heads vdim]; q and k over their root mean square (dim_n true
 * sizes), q to q [T, heads dim], k and v to the token's cache row. */
typedef struct {
  const void* proj;
  void* q;
  void* cache;            /* [pages][page_size][kv_heads (dim + vdim)] element type */
  int64_t ldp;
  int32_t heads, kv_heads, dim, vdim, dim_n;
  float eps;
  int32_t dtype, device;
} vmi_hy_kv_prep_args;
VMI_HY_API int vmi_hy_kv_prep(const vmi_hy_kv_prep_args* a, const vmi_hy_step* s, void* stream);

/* score = scale q . k + bias[h][min(i - j, bias_n - 1)]; token i sees the j <= i of its own chunk of `chunk` tokens (0: all);
 * sink[h] adds exp(sink) to the denominator; out = softmax . v * sigmoid(gate[t, h]).  bias, sink and gate may be NULL; bias and
 * sink come times log2(e).  Query rows of an entry and key head are (token, head of the group) pairs, head fastest, in tiles of
 * 16 * row_tiles (1 or 4, vmi_hy_attention_row_tiles): tiles [n_tiles][2] = (entry, first row), entry -1: none.  splits > 1: a tile's keys are dealt to that
 * many workgroups, partial float32 [splits][T * heads][vdim + 2]. */
typedef struct {
  const void* q;
  const void* cache;
  void* out;
  const float* bias;
  const float* sink;
  const void* gate;
  const int32_t* tiles;
  float* partial;
  int64_t ldo, ldg;
  int32_t heads, kv_heads, dim, vdim, bias_n, chunk, n_tiles, row_tiles, splits;
  float scale;
  int32_t dtype, device;
} vmi_hy_attention_args;
VMI_HY_API int32_t vmi_hy_attention_row_tiles(int32_t dim, int32_t vdim, int32_t want, int32_t dtype);
VMI_HY_API int vmi_hy_attention(const vmi_hy_attention_args* a, const vmi_hy_step* s, void* stream);

VMI_HY_API const char* vmi_hybrid_last_error(void);
VMI_HY_API int32_t vmi_hybrid_abi_version(void);
VMI_HY_API const char* vmi_hybrid_target_arch(void);

#ifdef __cplusplus
}
#endif
#endif
