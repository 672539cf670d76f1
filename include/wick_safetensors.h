/* wick_safetensors.h -- read-only access to a model folder: config.json and model.safetensors.
 *
 * The counterpart of wick_gguf.h for models that come as a folder: config.json says which architecture it is and with what sizes,
 * model.safetensors (8-byte little-endian header length, a JSON header name -> {dtype, shape, data_offsets}, the data) holds the
 * tensors.  Every tensor's byte range is checked against its shape and the file.  Nothing here touches the GPU.
 *
 * Every call returns 0 on success or a negative status (the values of wick_gguf_status); the message of the last failure on the
 * calling thread is wick_safetensors_last_error().  Pointers handed out stay valid until wick_safetensors_close.
 */
#ifndef WICK_SAFETENSORS_H
#define WICK_SAFETENSORS_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum { WICK_SAFETENSORS_BF16 = 0, WICK_SAFETENSORS_F32 = 1, WICK_SAFETENSORS_I32 = 2 };

typedef struct wick_safetensors wick_safetensors;

const char *wick_safetensors_last_error(void);
/* Opens DIR/config.json and DIR/model.safetensors (mapped read-only). */
int wick_safetensors_open(const char *dir, wick_safetensors **out);
void wick_safetensors_close(wick_safetensors *s);
/* config.json's "architecture" (NUL-terminated). */
const char *wick_safetensors_architecture(const wick_safetensors *s);
/* The text of config.json. */
const char *wick_safetensors_config(const wick_safetensors *s, size_t *nbytes);
uint64_t wick_safetensors_tensor_count(const wick_safetensors *s);
const char *wick_safetensors_tensor_name(const wick_safetensors *s, uint64_t index);
/* dims: room for 8 entries, outermost first; any out pointer may be null. */
int wick_safetensors_tensor(const wick_safetensors *s, const char *name, int *dtype, uint32_t *n_dims, uint64_t *dims, const void **data,
                            size_t *nbytes);

#ifdef __cplusplus
}
#endif
#endif /* WICK_SAFETENSORS_H */
